// Attention of query heads that share key / value heads in groups (ughip_layers.h), over caches this file owns the layout of: keys
// [kv_heads][cap][DQ] with the head size padded to one the kernels are built for, values transposed [kv_heads vdim][cap], both in the
// type the products read (BF16 or F32).  Queries and keys may be rotated in neighbouring pairs on the way, queries multiplied by a
// factor per position, and a window may limit what a position sees.
//
// Many positions: attention_place_kernel writes keys and values into the caches and the queries as attention_rows.h wants them.
// Few positions (attention_split_kernel): the 32 rows of a wave are (position, query head) pairs of one key head, and what is dealt to
//   waves and workgroups are tiles of 32 keys, read from the caches straight into MFMA operands; the waves' parts meet in LDS, the
//   workgroups' (if there are several per key head) in a second launch.  The scores come out transposed as in attention_rows.h.  With
//   bf16 caches a query is two bf16 terms, and so is a weight.  One position: the wave that meets the new key makes it from the
//   projected row and leaves it in the caches; nobody else reads that place.
#include <hip/hip_runtime.h>

#include <type_traits>

#include "attention_rows.h"
#include "bf16_split.h"
#include "layers.h"

using namespace ughip;

namespace {

// How a head's elements become the operand: `rot` elements in pairs (2 i, 2 i + 1) turned by the angles of the position, the rest as
// they are, all times `mul`.
struct Turn {
  const float* cos;  // of the position, rot / 2 values; null: nothing is rotated
  const float* sin;
  int rot;
  float mul;
};
// elements c .. c + N - 1 (c even) of a head of `dim`, zeros past its end; VEC: they are there (or none is) and 16-byte aligned, and a
// rotated part ends between pieces
template <int N, bool VEC = false>
__device__ __forceinline__ void turned(const float* head, int c, int dim, const Turn& t, float (&out)[N]) {
  if constexpr (VEC) {
    const bool there = c < dim, turns = t.cos && c < t.rot;
    float x[N], co[N / 2], si[N / 2];
#pragma unroll
    for (int e = 0; e < N; e += 4) __builtin_memcpy(x + e, __builtin_assume_aligned(head + (there ? c : 0) + e, 16), 16);
    const size_t at = turns ? c >> 1 : 0;
#pragma unroll
    for (int e = 0; e < N / 2; e += 2) {
      co[e] = 1.f, co[e + 1] = 1.f, si[e] = si[e + 1] = 0.f;
      if (t.cos) __builtin_memcpy(co + e, __builtin_assume_aligned(t.cos + at + e, 8), 8), __builtin_memcpy(si + e, __builtin_assume_aligned(t.sin + at + e, 8), 8);
    }
#pragma unroll
    for (int e = 0; e < N; e += 2) {
      const float u = there ? x[e] : 0.f, v = there ? x[e + 1] : 0.f, cc = turns ? co[e / 2] : 1.f, ss = turns ? si[e / 2] : 0.f;
      out[e] = (u * cc - v * ss) * t.mul;
      out[e + 1] = (v * cc + u * ss) * t.mul;
    }
    return;
  }
#pragma unroll
  for (int e = 0; e < N; e += 2) {
    const int d = c + e;
    const float u = d < dim ? head[d] : 0.f, v = d + 1 < dim ? head[d + 1] : 0.f;
    if (t.cos && d < t.rot) {
      const float co = t.cos[d >> 1], si = t.sin[d >> 1];
      out[e] = (u * co - v * si) * t.mul;
      out[e + 1] = (v * co + u * si) * t.mul;
    } else {
      out[e] = u * t.mul;
      out[e + 1] = v * t.mul;
    }
  }
}
template <typename T, int N>
__device__ __forceinline__ u32x4_t packed(const float (&v)[N]) {
  static_assert(N * sizeof(T) == 16, "one 16-byte piece");
  T e[N];
#pragma unroll
  for (int i = 0; i < N; ++i) e[i] = to_elem<T>(v[i]);
  u32x4_t out;
  __builtin_memcpy(&out, e, 16);
  return out;
}

struct GroupedArgs {
  const float* qkv;  // rows [heads dim | kv_heads dim | kv_heads vdim]
  void* kc;
  void* vc;
  void* qp;  // packed queries
  const float* cos;
  const float* sin;
  const float* temp;
  size_t row, cap;
  int t, pos, heads, kv_heads, dim, vdim, rot, q_rows;
  float scale2;  // scale * log2(e), a part of every query: the weights are powers of two of the scores
};
__device__ __forceinline__ Turn turn_of(const GroupedArgs& a, int p, bool query) {
  const size_t at = (size_t)p * (a.rot >> 1);
  return Turn{a.rot ? a.cos + at : nullptr, a.rot ? a.sin + at : nullptr, a.rot, query ? (a.temp ? a.temp[p] * a.scale2 : a.scale2) : 1.f};
}

constexpr int VT = 64;  // positions and value elements of a transposed tile

// blockIdx.y: first the query heads (none when q_rows is 0), then the key heads, then blocks of VT value elements of every value head.
template <typename T, int DQ, bool VEC>
__global__ void __launch_bounds__(256) attention_place_kernel(GroupedArgs a) {
  constexpr int E = 16 / sizeof(T), CH = DQ / E;
  __shared__ T tile[VT][VT + 2];
  const int nq = a.q_rows ? a.heads : 0, y = blockIdx.y;
  if (y < nq + a.kv_heads) {
    const bool is_q = y < nq;
    const int head = is_q ? y : y - nq, rows = is_q ? a.q_rows : a.t;
    const size_t e0 = (size_t)blockIdx.x * 256 + threadIdx.x;
    const int r = (int)(e0 / CH), c = (int)(e0 % CH) * E;
    if (r >= rows) return;
    u32x4_t piece = {0, 0, 0, 0};
    if (r < a.t) {
      float v[E];
      turned<E, VEC>(a.qkv + (size_t)r * a.row + (size_t)(is_q ? head : a.heads + head) * a.dim, c, a.dim, turn_of(a, a.pos + r, is_q), v);
      piece = packed<T>(v);
    }
    T* out = is_q ? static_cast<T*>(a.qp) + ((size_t)head * a.q_rows + r) * DQ + c : static_cast<T*>(a.kc) + ((size_t)head * a.cap + a.pos + r) * DQ + c;
    *reinterpret_cast<u32x4_t*>(out) = piece;
    return;
  }
  const int blocks = (a.vdim + VT - 1) / VT, kv = (y - nq - a.kv_heads) / blocks, v0 = (y - nq - a.kv_heads) % blocks * VT, r0 = blockIdx.x * VT;
  if (r0 >= a.t) return;
  const int x = threadIdx.x & 63, z = threadIdx.x >> 6;
  const float* src = a.qkv + (size_t)(a.heads + a.kv_heads) * a.dim + (size_t)kv * a.vdim + v0;
#pragma unroll 4
  for (int r = z; r < VT; r += 4)
    if (r0 + r < a.t && v0 + x < a.vdim) tile[r][x] = to_elem<T>(src[(size_t)(r0 + r) * a.row + x]);
  __syncthreads();
  T* out = static_cast<T*>(a.vc) + ((size_t)kv * a.vdim + v0) * a.cap + a.pos + r0;
#pragma unroll 4
  for (int v = z; v < VT; v += 4)
    if (r0 + x < a.t && v0 + v < a.vdim) out[(size_t)v * a.cap + x] = tile[x][v];
}

struct SplitArgs {
  GroupedArgs g;
  void* dst;
  float* acc;  // [splits][kv_heads rows][vdim]
  float* ml;   // [splits][kv_heads rows][2]
  size_t dst_stride;
  int rows, row_blocks, splits, window;  // rows: (position, head) pairs per key head
  bool dst_bf16;
};
constexpr int SK = 32;

// NW waves.  APPEND: one position, whose key and value come from the projected row.
template <typename T, int DQ, int DV, int NW, bool APPEND>
__global__ void __launch_bounds__(64 * NW) attention_split_kernel(SplitArgs a) {
  constexpr int E = 16 / sizeof(T), QC = DQ / E, NV = sizeof(T) == 2 ? 2 : 4;  // NV: 16-byte value operands of a tile and 32 value elements
  constexpr bool BF = sizeof(T) == 2;
  constexpr int Q_ROW = DQ + E;
  extern __shared__ __attribute__((aligned(16))) float parts[];
  const GroupedArgs& g = a.g;
  const int kv = blockIdx.x % g.kv_heads, rb = blockIdx.x / g.kv_heads, split = blockIdx.y, per = g.heads / g.kv_heads;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, col = lane & 31, hf = lane >> 5;
  const int r_last = min(a.rows, rb * 32 + 32) - 1, r_mine = min(rb * 32 + col, r_last), p_mine = g.pos + r_mine / per;
  const int first = g.pos + rb * 32 / per, last = g.pos + r_last / per, s_all = g.pos + g.t;
  const int tile0 = a.window ? max(0, first - a.window + 1) / SK : 0, tiles = last / SK + 1 - tile0, share = (tiles + a.splits - 1) / a.splits;
  const int k_stop = min(tile0 + tiles, tile0 + (split + 1) * share) * SK, oldest = a.window ? p_mine - a.window : -1;
  const T* keys = static_cast<const T*>(g.kc) + (size_t)kv * g.cap * DQ;
  const T* values = static_cast<const T*>(g.vc) + (size_t)kv * g.vdim * g.cap;
  u32x4_t kf[QC / 2], vf[DV / 32][NV];
  auto fetch = [&](int k0) {  // (the caches hold whole tiles)
#pragma unroll
    for (int c = 0; c < QC / 2; ++c) kf[c] = *reinterpret_cast<const u32x4_t*>(keys + (size_t)(k0 + col) * DQ + (2 * c + hf) * E);
#pragma unroll
    for (int i = 0; i < DV / 32; ++i) {
      const int v = i * 32 + col;
      const T* row = values + (size_t)(v < g.vdim ? v : 0) * g.cap + k0 + 4 * hf;
#pragma unroll
      for (int u = 0; u < NV; ++u) {
        if constexpr (BF) {
          const uint2 x = *reinterpret_cast<const uint2*>(row + 16 * u), y = *reinterpret_cast<const uint2*>(row + 16 * u + 8);
          vf[i][u] = u32x4_t{x.x, x.y, y.x, y.y};
        } else {
          vf[i][u] = *reinterpret_cast<const u32x4_t*>(row + 8 * u);
        }
      }
    }
  };
  int k0 = (tile0 + split * share + wave) * SK;
  if (k0 < k_stop) fetch(k0);
  // the queries (and the new key and value) through LDS, a pair of elements per thread and turn
  const int live = r_last + 1 - rb * 32;
  T* q_hi = reinterpret_cast<T*>(parts);
  T* q_lo = q_hi + (size_t)live * Q_ROW;  // (bf16 only)
  T* k_new = q_hi + (size_t)live * Q_ROW * (BF ? 2 : 1);
  T* v_new = k_new + DQ;
  for (int x = threadIdx.x; x < (live + (APPEND ? 1 : 0)) * (DQ / 2); x += 64 * NW) {
    const int r = x / (DQ / 2), d = x % (DQ / 2) * 2, row = min(rb * 32 + r, r_last);
    const bool query = r < live;
    const float* head = g.qkv + (size_t)(row / per) * g.row + (size_t)(query ? kv * per + row % per : g.heads + kv) * g.dim;
    float v[2];
    turned<2>(head, d, g.dim, turn_of(g, g.pos + row / per, query), v);
    T* to = query ? q_hi + r * Q_ROW + d : k_new + d;
    to[0] = to_elem<T>(v[0]), to[1] = to_elem<T>(v[1]);
    if constexpr (BF) {
      if (query) {
        q_lo[r * Q_ROW + d] = to_elem<T>(v[0] - bf16_to_f32(to[0]));
        q_lo[r * Q_ROW + d + 1] = to_elem<T>(v[1] - bf16_to_f32(to[1]));
      }
    }
  }
  if constexpr (APPEND)
    for (int v = threadIdx.x; v < DV; v += 64 * NW) v_new[v] = to_elem<T>(v < g.vdim ? g.qkv[(size_t)(g.heads + g.kv_heads) * g.dim + (size_t)kv * g.vdim + v] : 0.f);
  __syncthreads();
  const int q_at = (r_mine - rb * 32) * Q_ROW + hf * E;  // chunk 2 c + hf of row `col`: 2 c E further
  if constexpr (APPEND) {
    // the workgroup that meets the new key leaves it in the caches
    if ((tile0 + split * share) * SK <= g.pos && g.pos < k_stop) {
      T* krow = static_cast<T*>(g.kc) + ((size_t)kv * g.cap + g.pos) * DQ;
      for (int x = threadIdx.x; x < QC; x += 64 * NW) *reinterpret_cast<u32x4_t*>(krow + x * E) = *reinterpret_cast<const u32x4_t*>(k_new + x * E);
      for (int v = threadIdx.x; v < g.vdim; v += 64 * NW) static_cast<T*>(g.vc)[((size_t)kv * g.vdim + v) * g.cap + g.pos] = v_new[v];
    }
  }
  f32x16 o[DV / 32];
#pragma unroll
  for (int i = 0; i < DV / 32; ++i)
#pragma unroll
    for (int e = 0; e < 16; ++e) o[i][e] = 0.f;
  float mx = -INFINITY, sum = 0.f;
  for (; k0 < k_stop; k0 += NW * SK) {
    if constexpr (APPEND) {
      if (k0 + SK > g.pos) {  // the new position's tile
        const bool mine = k0 + col == g.pos;
#pragma unroll
        for (int c = 0; c < QC / 2; ++c) {
          const u32x4_t piece = *reinterpret_cast<const u32x4_t*>(k_new + (2 * c + hf) * E);
          kf[c] = mine ? piece : kf[c];
        }
#pragma unroll
        for (int i = 0; i < DV / 32; ++i) {
          const T now = v_new[i * 32 + col];
#pragma unroll
          for (int u = 0; u < NV; ++u) {
            T e[E];
            __builtin_memcpy(e, &vf[i][u], 16);
#pragma unroll
            for (int x = 0; x < E; ++x) {
              const int p = k0 + (BF ? 16 * u + 8 * (x >> 2) : 8 * u) + 4 * hf + (x & 3);
              e[x] = p < g.pos ? e[x] : p == g.pos ? now : T(0);
            }
            __builtin_memcpy(&vf[i][u], e, 16);
          }
        }
      }
    } else if (k0 + SK > s_all) {  // places past the last position were never written
#pragma unroll
      for (int i = 0; i < DV / 32; ++i)
#pragma unroll
        for (int u = 0; u < NV; ++u) {
          T e[E];
          __builtin_memcpy(e, &vf[i][u], 16);
#pragma unroll
          for (int x = 0; x < E; ++x) e[x] = k0 + (BF ? 16 * u + 8 * (x >> 2) : 8 * u) + 4 * hf + (x & 3) < s_all ? e[x] : T(0);
          __builtin_memcpy(&vf[i][u], e, 16);
        }
    }
    f32x16 s, s2;
#pragma unroll
    for (int e = 0; e < 16; ++e) s[e] = s2[e] = 0.f;
    asm volatile("" ::: "memory");  // (the queries' operands are read where they are used: they would not fit the registers)
#pragma unroll
    for (int c = 0; c < QC / 2; ++c) {
      mfma_chunk<T>(kf[c], *reinterpret_cast<const u32x4_t*>(q_hi + q_at + 2 * c * E), s);
      if constexpr (BF) mfma_chunk<T>(kf[c], *reinterpret_cast<const u32x4_t*>(q_lo + q_at + 2 * c * E), s2);
    }
    // element e: key k0 + 8 (e / 4) + 4 hf + e % 4, row `col`
    float top = mx;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int key = k0 + 8 * (e >> 2) + 4 * hf + (e & 3);
      s[e] = key <= p_mine && key > oldest ? s[e] + s2[e] : -INFINITY;
      top = fmaxf(top, s[e]);
    }
    top = fmaxf(top, __shfl_xor(top, 32, 64));
    const float alpha = top > mx ? __builtin_amdgcn_exp2f(mx - top) : 1.f, base = top == -INFINITY ? 0.f : top;
    mx = top;
    float part = 0.f;
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      s[e] = __builtin_amdgcn_exp2f(s[e] - base);
      part += s[e];
    }
    sum = sum * alpha + part + __shfl_xor(part, 32, 64);
#pragma unroll
    for (int i = 0; i < DV / 32; ++i)
#pragma unroll
      for (int e = 0; e < 16; ++e) o[i][e] *= alpha;
#pragma unroll
    for (int u = 0; u < NV; ++u) {
      if constexpr (BF) {
        bf16x8 hi, lo;
#pragma unroll
        for (int e = 0; e < 8; ++e) {
          hi[e] = (__bf16)s[8 * u + e];
          lo[e] = (__bf16)(s[8 * u + e] - (float)hi[e]);
        }
#pragma unroll
        for (int i = 0; i < DV / 32; ++i) {
          o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, vf[i][u]), hi, o[i], 0, 0, 0);
          o[i] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, vf[i][u]), lo, o[i], 0, 0, 0);
        }
      } else {
#pragma unroll
        for (int i = 0; i < DV / 32; ++i) {
          const f32x4_t v = __builtin_bit_cast(f32x4_t, vf[i][u]);
#pragma unroll
          for (int x = 0; x < 4; ++x) o[i] = __builtin_amdgcn_mfma_f32_32x32x2f32(v[x], s[4 * u + x], o[i], 0, 0, 0);
        }
      }
    }
    if (k0 + NW * SK < k_stop) fetch(k0 + NW * SK);
  }
  // the waves' parts: [wave][row][DV + 4], then every wave's maximum and sum per row
  __syncthreads();  // (what was staged there has been read)
  constexpr int P = DV + 4;
  float* ml = parts + (size_t)NW * live * P;
  if (col < live) {
    float* mine = parts + ((size_t)wave * live + col) * P;
#pragma unroll
    for (int i = 0; i < DV / 32; ++i)
#pragma unroll
      for (int q = 0; q < 4; ++q) *reinterpret_cast<f32x4_t*>(mine + i * 32 + 8 * q + 4 * hf) = f32x4_t{o[i][4 * q], o[i][4 * q + 1], o[i][4 * q + 2], o[i][4 * q + 3]};
    if (hf == 0) ml[(wave * live + col) * 2] = mx, ml[(wave * live + col) * 2 + 1] = sum;
  }
  __syncthreads();
  for (int x = threadIdx.x; x < live * g.vdim; x += 64 * NW) {
    const int r = x / g.vdim, v = x - r * g.vdim, row = rb * 32 + r;
    float m[NW], top = -INFINITY;
#pragma unroll
    for (int w = 0; w < NW; ++w) top = fmaxf(top, m[w] = ml[(w * live + r) * 2]);
    const float base = top == -INFINITY ? 0.f : top;
    float l = 0.f, val = 0.f;
#pragma unroll
    for (int w = 0; w < NW; ++w) {
      const float f = __builtin_amdgcn_exp2f(m[w] - base);
      l += f * ml[(w * live + r) * 2 + 1];
      val += f * parts[((size_t)w * live + r) * P + v];
    }
    if (a.splits == 1) {
      const size_t at = (size_t)(row / per) * a.dst_stride + (size_t)(kv * per + row % per) * g.vdim + v;
      if (a.dst_bf16) static_cast<uint16_t*>(a.dst)[at] = bf16_rne(val / l);
      else static_cast<float*>(a.dst)[at] = val / l;
    } else {
      const size_t at = (size_t)split * g.kv_heads * a.rows + (size_t)kv * a.rows + row;
      a.acc[at * g.vdim + v] = val;
      if (v == 0) a.ml[at * 2] = top, a.ml[at * 2 + 1] = l;
    }
  }
}

// A workgroup per (position, head): its splits (up to 64) added up.
__global__ void __launch_bounds__(256) attention_merge_kernel(SplitArgs a) {
  __shared__ float fac[64];
  __shared__ float part[256];
  const GroupedArgs& g = a.g;
  const int per = g.heads / g.kv_heads, kv = blockIdx.x / a.rows, row = blockIdx.x - kv * a.rows;
  const size_t step = (size_t)g.kv_heads * a.rows, mine = (size_t)kv * a.rows + row;
  if (threadIdx.x < 64) {
    const int s = threadIdx.x;
    const float m = s < a.splits ? a.ml[(s * step + mine) * 2] : -INFINITY, l = s < a.splits ? a.ml[(s * step + mine) * 2 + 1] : 0.f;
    const float top = wave_max(m), f = __builtin_amdgcn_exp2f(m - top);  // every position sees itself: top is finite
    fac[s] = f / wave_sum(f * l);
  }
  __syncthreads();
  const int nc = g.vdim <= 64 ? 64 : g.vdim <= 128 ? 128 : 256, share = 256 / nc, v = threadIdx.x % nc, z = threadIdx.x / nc;
  float val = 0.f;
  if (v < g.vdim) {
#pragma unroll 8
    for (int s = z; s < a.splits; s += share) val += fac[s] * a.acc[(s * step + mine) * g.vdim + v];
  }
  part[threadIdx.x] = val;
  __syncthreads();
  if (z != 0 || v >= g.vdim) return;
  for (int k = 1; k < share; ++k) val += part[k * nc + v];
  const size_t at = (size_t)(row / per) * a.dst_stride + (size_t)(kv * per + row % per) * g.vdim + v;
  if (a.dst_bf16) static_cast<uint16_t*>(a.dst)[at] = bf16_rne(val);
  else static_cast<float*>(a.dst)[at] = val;
}

constexpr size_t HEAD_MAX = 256;
// The sizes the kernels are built for: a head's padded query / key size and the value size of its accumulators.
struct Built {
  int dq, dv;
};
Built built_for(size_t dim, size_t vdim) {
  if (dim <= 64 && vdim <= 64) return {64, 64};
  if (dim <= 128 && vdim <= 128) return {128, 128};
  if (dim <= 192 && vdim <= 128) return {192, 128};
  return {256, 256};
}
template <typename F>
int with_sizes(const Built& b, F&& f) {
  using std::integral_constant;
  if (b.dq == 64) return f(integral_constant<int, 64>{}, integral_constant<int, 64>{});
  if (b.dq == 128) return f(integral_constant<int, 128>{}, integral_constant<int, 128>{});
  if (b.dq == 192) return f(integral_constant<int, 192>{}, integral_constant<int, 128>{});
  return f(integral_constant<int, 256>{}, integral_constant<int, 256>{});
}

template <typename T, int DQ>
int place(ughip_device* dev, const GroupedArgs& g) {
  const size_t pieces = (size_t)(g.q_rows > g.t ? g.q_rows : g.t) * (DQ * sizeof(T) / 16), tiles = ((size_t)g.t + VT - 1) / VT;
  const size_t x = (pieces + 255) / 256 > tiles ? (pieces + 255) / 256 : tiles;
  const int y = (g.q_rows ? g.heads : 0) + g.kv_heads + g.kv_heads * ((g.vdim + VT - 1) / VT);
  if (y > 65535) return set_error(UGHIP_ERR_UNSUPPORTED, "grouped_attention: too many heads");
  auto whole = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  const bool vec = g.dim % 8 == 0 && g.rot % 8 == 0 && g.row % 4 == 0 && whole(g.qkv);
  if (vec) attention_place_kernel<T, DQ, true><<<dim3((unsigned)x, (unsigned)y), 256, 0, dev->stream>>>(g);
  else attention_place_kernel<T, DQ, false><<<dim3((unsigned)x, (unsigned)y), 256, 0, dev->stream>>>(g);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

template <typename T, int DQ, int DV>
int attend_many(ughip_device* dev, GroupedArgs g, AttRowsArgs r) {
  g.q_rows = (g.t + ATT_QT - 1) / ATT_QT * ATT_QT;
  if (int rc = rows_scratch(dev, (size_t)g.heads * g.q_rows * DQ * sizeof(T), &g.qp)) return rc;
  if (int rc = place<T, DQ>(dev, g)) return rc;
  r.q = g.qp, r.q_rows = g.q_rows, r.k_rows = (int)g.cap;
  constexpr int bytes = attention_rows_lds_bytes<T, DQ, DV>();
  static_assert(bytes <= 160 * 1024, "tile does not fit LDS");
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(attention_rows_kernel<T, DQ, DV>), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
  UGHIP_HIPCHK(attr);
  attention_rows_kernel<T, DQ, DV><<<dim3((unsigned)g.heads, (unsigned)(g.q_rows / ATT_QT)), attention_rows_threads<T, DQ, DV>(), bytes, dev->stream>>>(r);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

template <typename T, int DQ, int DV>
int attend_few(ughip_device* dev, SplitArgs a) {
  constexpr int NW = DV <= 128 && DQ * sizeof(T) <= 384 ? 8 : 4;
  const GroupedArgs& g = a.g;
  if (g.t > 1)
    if (int rc = place<T, DQ>(dev, g)) return rc;
  a.rows = g.t * (g.heads / g.kv_heads), a.row_blocks = (a.rows + 31) / 32;
  const int groups = g.kv_heads * a.row_blocks;
  int seen = g.pos + g.t;
  if (a.window && seen > a.window + g.t - 1) seen = a.window + g.t - 1;
  const int tiles = (seen + SK - 1) / SK + 1;
  // a tile per wave; a second launch pays from some tiles per wave on
  int splits = tiles <= 2 * NW + 1 ? 1 : (tiles + NW - 1) / NW, most = 512 / groups;
  if (most > 64) most = 64;
  if (splits > most) splits = most;
  if (splits < 1) splits = 1;
  a.splits = splits;
  if (splits > 1) {
    const size_t rows = (size_t)splits * g.kv_heads * a.rows, n_ml = (rows * 2 + 63) & ~(size_t)63;
    void* ws = nullptr;
    if (int rc = rows_scratch(dev, (n_ml + rows * g.vdim) * sizeof(float), &ws)) return rc;
    a.ml = static_cast<float*>(ws), a.acc = a.ml + n_ml;
  }
  const int live = a.rows < 32 ? a.rows : 32;
  const size_t staged = ((size_t)live * (DQ + 16 / sizeof(T)) * (sizeof(T) == 2 ? 2 : 1) + DQ + DV) * sizeof(T), met = (size_t)NW * live * (DV + 4 + 2) * sizeof(float);
  const size_t lds = staged > met ? staged : met;
  auto go = [&](auto kernel) {
    if (lds > 60 * 1024)
      if (hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); e != hipSuccess) return e;
    kernel<<<dim3((unsigned)groups, (unsigned)splits), 64 * NW, lds, dev->stream>>>(a);
    return hipGetLastError();
  };
  UGHIP_HIPCHK(g.t == 1 ? go(attention_split_kernel<T, DQ, DV, NW, true>) : go(attention_split_kernel<T, DQ, DV, NW, false>));
  if (splits > 1) {
    attention_merge_kernel<<<(unsigned)(g.kv_heads * a.rows), 256, 0, dev->stream>>>(a);
    UGHIP_HIPCHK(hipGetLastError());
  }
  return UGHIP_OK;
}

constexpr size_t FEW = 16;  // positions

}  // namespace

extern "C" int ughip_grouped_attention_cache(size_t kv_heads, size_t dim, size_t vdim, size_t capacity, size_t* rows, size_t* k_elems, size_t* v_elems) {
  if (!rows || !k_elems || !v_elems) return set_error(UGHIP_ERR_INVALID, "grouped_attention_cache: null argument");
  if (kv_heads == 0 || dim == 0 || vdim == 0 || dim > HEAD_MAX || vdim > HEAD_MAX)
    return set_error(UGHIP_ERR_UNSUPPORTED, "grouped_attention: heads of %zu and %zu elements (1 to %zu)", dim, vdim, HEAD_MAX);
  *rows = (capacity + ATT_KT - 1) / ATT_KT * ATT_KT;
  *k_elems = kv_heads * *rows * built_for(dim, vdim).dq, *v_elems = kv_heads * vdim * *rows;
  return UGHIP_OK;
}

extern "C" int ughip_grouped_attention(ughip_device* dev, const ughip_attention* p) {
  const char* what = "grouped_attention";
  if (!dev || !p || !p->k_cache || !p->v_cache) return set_error(UGHIP_ERR_INVALID, "%s: null argument", what);
  if (p->heads == 0 || p->kv_heads == 0 || p->heads % p->kv_heads != 0 || p->heads > 32767) return set_error(UGHIP_ERR_INVALID, "%s: %zu heads on %zu", what, p->heads, p->kv_heads);
  size_t rows, k_elems, v_elems;
  if (int rc = ughip_grouped_attention_cache(p->kv_heads, p->dim, p->vdim, p->capacity, &rows, &k_elems, &v_elems)) return rc;
  const int type = p->k_cache->dtype;
  if (type != UGHIP_F32 && type != UGHIP_BF16) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: caches are F32 or BF16", what);
  if (int rc = check_buf(dev, p->k_cache, k_elems, type, what)) return rc;
  if (int rc = check_buf(dev, p->v_cache, v_elems, type, what)) return rc;
  const size_t s = p->pos + p->t, row = (p->heads + p->kv_heads) * p->dim + p->kv_heads * p->vdim;
  if (s > p->capacity || s > 0x3fffffffull) return set_error(UGHIP_ERR_BOUNDS, "%s: %zu positions exceed the cache's %zu", what, s, p->capacity);
  if (p->window > 0x3fffffffull) return set_error(UGHIP_ERR_INVALID, "%s: a window of %zu", what, p->window);
  if (int rc = check_view(dev, p->qkv, p->t, row, UGHIP_F32, what)) return rc;
  if (p->rot) {
    if (p->rot % 2 != 0 || p->rot > p->dim) return set_error(UGHIP_ERR_INVALID, "%s: %zu rotated elements of %zu", what, p->rot, p->dim);
    if (s > p->table_rows) return set_error(UGHIP_ERR_BOUNDS, "%s: positions up to %zu, tables for %zu", what, s, p->table_rows);
    for (const ughip_slice* q : {p->cos, p->sin})
      if (int rc = check_buf(dev, q, p->table_rows * (p->rot / 2), UGHIP_F32, what)) return rc;
  }
  if (p->q_factor)
    if (int rc = check_buf(dev, p->q_factor, s, UGHIP_F32, what)) return rc;
  if (int rc = check_view(dev, p->dst, p->t, p->heads * p->vdim, -1, what)) return rc;
  const bool bf16 = p->dst.s->dtype == UGHIP_BF16;
  if (!bf16 && p->dst.s->dtype != UGHIP_F32) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: the result is F32 or BF16", what);
  if (p->t == 0) return UGHIP_OK;
  if ((p->t + ATT_QT - 1) / ATT_QT > 65535) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: too many positions", what);
  if (int rc = device_activate(dev)) return rc;
  GroupedArgs g{};
  g.qkv = view_ptr<float>(p->qkv), g.kc = p->k_cache->ptr, g.vc = p->v_cache->ptr, g.cos = buf_ptr<float>(p->cos), g.sin = buf_ptr<float>(p->sin);
  g.temp = buf_ptr<float>(p->q_factor), g.row = p->qkv.stride, g.cap = rows;
  g.t = (int)p->t, g.pos = (int)p->pos, g.heads = (int)p->heads, g.kv_heads = (int)p->kv_heads, g.dim = (int)p->dim, g.vdim = (int)p->vdim, g.rot = (int)p->rot;
  void* dst = static_cast<char*>(p->dst.s->ptr) + p->dst.offset * (bf16 ? 2 : 4);
  g.scale2 = p->scale * 1.4426950408889634f;
  const Built built = built_for(p->dim, p->vdim);
  const int window = p->window < s ? (int)p->window : 0;  // (one that nothing has left yet is none)
  if (p->t <= FEW) {
    SplitArgs a{};
    a.g = g, a.dst = dst, a.dst_stride = p->dst.stride, a.window = window, a.dst_bf16 = bf16;
    return with_sizes(built, [&](auto dq, auto dv) {
      return type == UGHIP_BF16 ? attend_few<uint16_t, decltype(dq)::value, decltype(dv)::value>(dev, a) : attend_few<float, decltype(dq)::value, decltype(dv)::value>(dev, a);
    });
  }
  AttRowsArgs r{};
  r.k = g.kc, r.v = g.vc, r.dst = dst, r.v_stride = rows, r.dst_stride = p->dst.stride, r.t = g.t, r.pos = g.pos, r.vdim = g.vdim, r.kv_heads = g.kv_heads, r.window = window;
  r.dst_bf16 = bf16;
  return with_sizes(built, [&](auto dq, auto dv) {
    return type == UGHIP_BF16 ? attend_many<uint16_t, decltype(dq)::value, decltype(dv)::value>(dev, g, r) : attend_many<float, decltype(dq)::value, decltype(dv)::value>(dev, g, r);
  });
}
