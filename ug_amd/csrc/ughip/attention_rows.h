// Attention of many positions over keys and values in memory, the scores never leaving registers; shared by the kinds of attention
// that bring their operands into this form.
//   A wave owns 32 queries, a workgroup 128; keys come in tiles of 64 through LDS.  The scores are computed transposed, S^T = K Q^T
//   (32 x 32 tiles), which leaves lane l with query l % 32 as its column: the running maximum and sum are one exchange with lane
//   l ^ 32, and the weights sit where the second product, O^T = V^T P^T, wants its right operand (the order in which keys take
//   part in it is the order the accumulator layout gives; V is read in the same order).  Values come transposed for that.  Two such
//   groups of waves take turns with the tiles of keys where registers allow it.
//   bf16 operands: v_mfma_f32_32x32x16_bf16, a weight as two bf16 terms (16 bits of it); f32: v_mfma_f32_32x32x2_f32.
#pragma once
#include <hip/hip_runtime.h>

#include "bf16_split.h"
#include "layers.h"

namespace ughip {
namespace {  // every file that launches the kernel has its own

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));

// Queries come times scale * log2(e): the weights are powers of two of the scores.  q [heads][q_rows][DQ], k [kv_heads][k_rows][DQ],
// v [kv_heads vdim][v_stride] (one row per value element, position along it); zeros past a query's and a key's last element and past
// the last query.
struct AttRowsArgs {
  const void* q;
  const void* k;
  const void* v;
  void* dst;
  size_t v_stride, dst_stride;
  int t, pos, vdim, q_rows, k_rows;
  int kv_heads;  // key head of query head h: h / (heads / kv_heads)
  int window;    // > 0: a position sees itself and the window - 1 positions in front of it
  bool dst_bf16;
};

template <typename T>
__device__ __forceinline__ T to_elem(float v) {
  if constexpr (sizeof(T) == 2) return bf16_rne(v);
  else return v;
}

template <typename T>
__device__ __forceinline__ void mfma_chunk(const u32x4_t& a, const u32x4_t& b, f32x16& acc) {
  if constexpr (sizeof(T) == 2) {
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
  } else {
    const f32x4_t x = __builtin_bit_cast(f32x4_t, a), y = __builtin_bit_cast(f32x4_t, b);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.x, y.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.y, y.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.z, y.z, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(x.w, y.w, acc, 0, 0, 0);
  }
}

constexpr int ATT_KT = 64, ATT_QT = 128;
// Two groups of four waves share the queries and take every second tile of keys, where the registers of two waves per SIMD hold the
// tiles; their results meet at the end.
template <typename T, int DQ, int DV>
constexpr int attention_rows_groups() {
  return sizeof(T) == 2 && DQ <= 192 && DV <= 128 ? 2 : 1;
}
template <typename T, int DQ, int DV>
constexpr int attention_rows_threads() {
  return 256 * attention_rows_groups<T, DQ, DV>();
}
// A tile's bytes, and whether LDS holds two per group: the next one goes in while this one is multiplied.
template <typename T, int DQ, int DV>
constexpr int attention_rows_tile_bytes() {
  return ATT_KT * (DQ * (int)sizeof(T) + 16) + DV * (ATT_KT * (int)sizeof(T) + 16);
}
template <typename T, int DQ, int DV>
constexpr bool attention_rows_twice() {
  return 2 * attention_rows_groups<T, DQ, DV>() * attention_rows_tile_bytes<T, DQ, DV>() <= 160 * 1024;
}
template <typename T, int DQ, int DV>
constexpr int attention_rows_lds_bytes() {
  return (attention_rows_twice<T, DQ, DV>() ? 2 : 1) * attention_rows_groups<T, DQ, DV>() * attention_rows_tile_bytes<T, DQ, DV>();
}

// DQ >= dim + rot and DV >= vdim, the surplus is zeros.  T: uint16_t (bf16) or float.
template <typename T, int DQ, int DV>
__global__ void __launch_bounds__((attention_rows_threads<T, DQ, DV>())) attention_rows_kernel(AttRowsArgs a) {
  constexpr int E = 16 / sizeof(T), QC = DQ / E, K_ROW = DQ * sizeof(T) + 16, V_ROW = ATT_KT * sizeof(T) + 16, VC = ATT_KT / E;
  constexpr int NK = ATT_KT * QC / 256, NV = DV * VC / 256;  // 16-byte pieces of a tile per thread
  constexpr bool AHEAD = NK + NV <= 16;                   // the next tile waits in registers while this one is multiplied
  static_assert(ATT_KT * QC % 256 == 0 && DV * VC % 256 == 0, "whole pieces per thread");
  extern __shared__ __attribute__((aligned(16))) char lds[];
  constexpr int GROUPS = attention_rows_groups<T, DQ, DV>();
  const int group = threadIdx.x >> 8, tid = threadIdx.x & 255;
  constexpr int TILE = attention_rows_tile_bytes<T, DQ, DV>();
  constexpr bool TWICE = attention_rows_twice<T, DQ, DV>();
  char* const tiles = lds + group * (TWICE ? 2 : 1) * TILE;
  char* Ks = tiles;                // [ATT_KT][DQ]
  char* Vs = Ks + ATT_KT * K_ROW;  // [DV][ATT_KT]
  // consecutive workgroups (dealt round robin to the chip's eight parts) take different key heads: those that share one meet in a cache
  const int per = gridDim.x / a.kv_heads, kv = blockIdx.x % a.kv_heads, head = kv * per + blockIdx.x / a.kv_heads;
  const int qb = gridDim.y - 1 - blockIdx.y;  // the longest rows first
  const int lane = tid & 63, wave = tid >> 6, col = lane & 31, hf = lane >> 5;
  const int i_mine = qb * ATT_QT + wave * 32 + col, p_mine = a.pos + min(i_mine, a.t - 1);
  // the wave's queries as the right operand of S^T: chunk 2 c + hf of query `col` (rows up to q_rows exist, zeros past t)
  u32x4_t qf[QC / 2];
  {
    const char* qr = static_cast<const char*>(a.q) + ((size_t)head * a.q_rows + i_mine) * DQ * sizeof(T) + hf * 16;
#pragma unroll
    for (int c = 0; c < QC / 2; ++c) qf[c] = *reinterpret_cast<const u32x4_t*>(qr + c * 32);
  }
  f32x16 o[DV / 32];
#pragma unroll
  for (int i = 0; i < DV / 32; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[i][e] = 0.f;
  float mx = -INFINITY, sum = 0.f;
  const int s_all = a.pos + a.t, last_q = min(a.t, (qb + 1) * ATT_QT), keys = a.pos + last_q, first_p = a.pos + qb * ATT_QT + wave * 32;
  const int k_begin = a.window ? max(0, a.pos + qb * ATT_QT - a.window + 1) / ATT_KT * ATT_KT : 0, oldest = a.window ? p_mine - a.window : -1;  // keys > oldest are seen
  const char* k_head = static_cast<const char*>(a.k) + (size_t)kv * a.k_rows * DQ * sizeof(T);
  const T* v_head = static_cast<const T*>(a.v) + (size_t)kv * a.vdim * a.v_stride;
  u32x4_t kr[NK], vr[NV];
  auto fetch = [&](int k0) {
#pragma unroll
    for (int u = 0; u < NK; ++u) kr[u] = *reinterpret_cast<const u32x4_t*>(k_head + (size_t)k0 * DQ * sizeof(T) + (tid + u * 256) * 16);
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      // rows are padded to whole tiles and 16-byte aligned; every lane loads (no branches between loads)
      const int x = tid + u * 256, vc = x / VC;
      vr[u] = *reinterpret_cast<const u32x4_t*>(v_head + (size_t)(vc < a.vdim ? vc : 0) * a.v_stride + k0 + x % VC * E);
    }
  };
  // what of a piece of values is none: columns past the last one, positions past the last one (never written)
  auto value_piece = [&](const u32x4_t& piece, int vc, int kp) {
    T v[E];
    __builtin_memcpy(v, &piece, 16);
#pragma unroll
    for (int e = 0; e < E; ++e) v[e] = vc < a.vdim && kp + e < s_all ? v[e] : T(0);
    u32x4_t out;
    __builtin_memcpy(&out, v, 16);
    return out;
  };
  const int k_mine = k_begin + group * ATT_KT;
  auto place = [&](int k0, char* kt) {
    char* vt = kt + ATT_KT * K_ROW;
#pragma unroll
    for (int u = 0; u < NK; ++u) {
      const int x = tid + u * 256;
      *reinterpret_cast<u32x4_t*>(kt + x / QC * K_ROW + x % QC * 16) = kr[u];
    }
    const bool whole = k0 + ATT_KT <= s_all && DV == a.vdim;
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      const int x = tid + u * 256;
      *reinterpret_cast<u32x4_t*>(vt + x / VC * V_ROW + x % VC * 16) = whole ? vr[u] : value_piece(vr[u], x / VC, k0 + x % VC * E);
    }
  };
  if (AHEAD && k_mine < keys) fetch(k_mine);
  if constexpr (TWICE) {
    if (!AHEAD && k_mine < keys) fetch(k_mine);
    if (k_mine < keys) place(k_mine, tiles);
    if (AHEAD && k_mine + GROUPS * ATT_KT < keys) fetch(k_mine + GROUPS * ATT_KT);
  }
  for (int k0 = k_mine; k0 - group * ATT_KT < keys; k0 += GROUPS * ATT_KT) {
    const bool there = GROUPS == 1 || k0 < keys;  // (the last tile of an odd number is the first group's alone)
    const int k_next = k0 + GROUPS * ATT_KT;
    if constexpr (TWICE) {
      __syncthreads();  // (this tile is there, and the one before has been read)
      if (k_next < keys) {
        if (!AHEAD) fetch(k_next);
        place(k_next, tiles + (Ks == tiles ? TILE : 0));
        if (AHEAD && k_next + GROUPS * ATT_KT < keys) fetch(k_next + GROUPS * ATT_KT);
      }
    } else {
      __syncthreads();
      if (there) {
        if (!AHEAD) fetch(k0);
        place(k0, tiles);
      }
      __syncthreads();
      if (AHEAD && k_next < keys) fetch(k_next);
    }
    const char* const Kc = Ks;
    const char* const Vc = Vs;
    if constexpr (TWICE) Ks = Ks == tiles ? tiles + TILE : tiles, Vs = Ks + ATT_KT * K_ROW;
    if (!there) continue;
    if (k0 > first_p + 31 || (a.window && k0 + ATT_KT - 1 <= first_p - a.window)) continue;  // nothing in this tile is visible to the wave's queries
    f32x16 s[2];
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int e = 0; e < 16; ++e) s[b][e] = 0.f;
#pragma unroll
    for (int c = 0; c < QC / 2; ++c)
#pragma unroll
      for (int b = 0; b < 2; ++b) mfma_chunk<T>(*reinterpret_cast<const u32x4_t*>(Kc + (b * 32 + col) * K_ROW + hf * 16 + c * 32), qf[c], s[b]);
    // element e of s[b]: key k0 + 32 b + 8 (e / 4) + 4 hf + e % 4, query `col`
    float top = mx;
    if (k0 + ATT_KT - 1 > first_p || (a.window && k0 <= first_p + 31 - a.window)) {  // some keys of the tile are not visible to some of the wave's queries
#pragma unroll
      for (int b = 0; b < 2; ++b)
#pragma unroll
        for (int e = 0; e < 16; ++e) {
          const int key = k0 + 32 * b + 8 * (e >> 2) + 4 * hf + (e & 3);
          s[b][e] = key <= p_mine && key > oldest ? s[b][e] : -INFINITY;
        }
    }
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int e = 0; e < 16; ++e) top = fmaxf(top, s[b][e]);
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    // the weights' base follows the maximum only when that has left it well behind: up to 2^8 they lose nothing
    const bool behind = top > mx + 8.f;
    if (__any(behind)) {
      const float alpha = behind ? exp2f(mx - top) : 1.f;
      sum *= alpha;
#pragma unroll
      for (int i = 0; i < DV / 32; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e) o[i][e] *= alpha;
      mx = behind ? top : mx;
    }
    const float base = mx == -INFINITY ? 0.f : mx;
    float part = 0.f;
#pragma unroll
    for (int b = 0; b < 2; ++b)
#pragma unroll
      for (int e = 0; e < 16; ++e) {
        s[b][e] = __builtin_amdgcn_exp2f(s[b][e] - base);
        part += s[b][e];
      }
    sum += part + __shfl_xor(part, 32, 64);
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      if constexpr (sizeof(T) == 2) {
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          bf16x8 hi, lo;
#pragma unroll
          for (int e = 0; e < 8; ++e) {
            hi[e] = (__bf16)s[b][8 * u + e];
            lo[e] = (__bf16)(s[b][8 * u + e] - (float)hi[e]);
          }
          bf16x8 vf[DV / 32];
#pragma unroll
          for (int i = 0; i < DV / 32; ++i) {
            const char* p = Vc + (i * 32 + col) * V_ROW + (b * 32 + 16 * u + 4 * hf) * 2;
            const uint2 v0 = *reinterpret_cast<const uint2*>(p), v1 = *reinterpret_cast<const uint2*>(p + 16);
            vf[i] = __builtin_bit_cast(bf16x8, u32x4_t{v0.x, v0.y, v1.x, v1.y});
          }
#pragma unroll
          for (int i = 0; i < DV / 32; ++i) o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[i], hi, o[i], 0, 0, 0);
#pragma unroll
          for (int i = 0; i < DV / 32; ++i) o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(vf[i], lo, o[i], 0, 0, 0);
        }
      } else {
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int i = 0; i < DV / 32; ++i) {
            const f32x4_t v = *reinterpret_cast<const f32x4_t*>(Vc + (i * 32 + col) * V_ROW + (b * 32 + 8 * u + 4 * hf) * 4);
            o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(v.x, s[b][4 * u], o[i], 0, 0, 0);
            o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(v.y, s[b][4 * u + 1], o[i], 0, 0, 0);
            o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(v.z, s[b][4 * u + 2], o[i], 0, 0, 0);
            o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(v.w, s[b][4 * u + 3], o[i], 0, 0, 0);
          }
      }
    }
  }
  if constexpr (GROUPS == 2) {
    constexpr int N = DV / 32 * 4;
    static_assert(4 * 64 * (N * 16 + 8) <= attention_rows_lds_bytes<T, DQ, DV>(), "a group's results fit where the tiles were");
    f32x4_t* other = reinterpret_cast<f32x4_t*>(lds) + wave * N * 64 + lane;
    float* ms = reinterpret_cast<float*>(lds + 4 * 64 * N * 16) + (wave * 64 + lane) * 2;
    __syncthreads();
    if (group == 1) {
#pragma unroll
      for (int i = 0; i < DV / 32; ++i)
#pragma unroll
        for (int q = 0; q < 4; ++q) other[(i * 4 + q) * 64] = f32x4_t{o[i][4 * q], o[i][4 * q + 1], o[i][4 * q + 2], o[i][4 * q + 3]};
      ms[0] = mx, ms[1] = sum;
    }
    __syncthreads();
    if (group == 1) return;
    const float m2 = ms[0], s2 = ms[1], top = fmaxf(mx, m2), base = top == -INFINITY ? 0.f : top, f1 = exp2f(mx - base), f2 = exp2f(m2 - base);
    sum = f1 * sum + f2 * s2;
#pragma unroll
    for (int i = 0; i < DV / 32; ++i)
#pragma unroll
      for (int q = 0; q < 4; ++q) {
        const f32x4_t v = other[(i * 4 + q) * 64];
#pragma unroll
        for (int e = 0; e < 4; ++e) o[i][4 * q + e] = f1 * o[i][4 * q + e] + f2 * v[e];
      }
  }
  if (i_mine >= a.t) return;
  const float inv = 1.f / sum;
  const size_t at = (size_t)i_mine * a.dst_stride + (size_t)head * a.vdim;
#pragma unroll
  for (int i = 0; i < DV / 32; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int vc = i * 32 + 8 * (e >> 2) + 4 * hf + (e & 3);
      if (vc < a.vdim) {
        if (a.dst_bf16) static_cast<uint16_t*>(a.dst)[at + vc] = bf16_rne(o[i][e] * inv);
        else static_cast<float*>(a.dst)[at + vc] = o[i][e] * inv;
      }
    }
}

}  // namespace
}  // namespace ughip
