// Attention over latents (ughip_layers.h): the cache of a layer is one row per position, [normed latent (rank) | rotated key part
// (rot)], shared by all heads.
//
// Many positions: keys and values are expanded by products before, the kernel of attention_rows.h does the rest.
// Few positions (absorb, split, merge): the up-projection of the keys is folded into the query, that of the values into the
//   result, so that a head's keys and values are both the cache rows as they are.  16 (position, head) pairs per workgroup against
//   tiles of 32 cache rows in LDS, v_mfma_f32_16x16x4_f32; the cache is split over workgroups, a last launch adds the parts up.
#include <hip/hip_runtime.h>

#include <type_traits>

#include "attention_rows.h"
#include "bf16_split.h"
#include "layers.h"

using namespace ughip;

namespace {

// element e of a rotated part of `rot` elements at a table row: pairs (i, i + rot / 2)
__device__ __forceinline__ float rotated(const float* part, int e, int rot, const float* cos, const float* sin) {
  const int half = rot >> 1, i = e < half ? e : e - half;
  const float u = part[i], v = part[i + half], c = cos[i], s = sin[i];
  return e < half ? u * c - v * s : v * c + u * s;
}

struct AppendArgs {
  const float* kv;  // null: nothing to append
  size_t kv_stride;
  const float* w;
  float eps;
  const float* cos;
  const float* sin;
  float* cache;
  size_t pos;
  int rank, rot;
};

__device__ __forceinline__ void append_row(const AppendArgs& a, int i, float* red) {
  const float* row = a.kv + (size_t)i * a.kv_stride;
  const size_t p = a.pos + i;
  float ss = 0.f;
  for (int c = threadIdx.x; c < a.rank; c += 256) ss += row[c] * row[c];
  ss = block_sum<4>(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)a.rank + a.eps);
  float* out = a.cache + p * (a.rank + a.rot);
  for (int c = threadIdx.x; c < a.rank; c += 256) out[c] = row[c] * inv * a.w[c];
  for (int e = threadIdx.x; e < a.rot; e += 256) out[a.rank + e] = rotated(row + a.rank, e, a.rot, a.cos + p * (a.rot / 2), a.sin + p * (a.rot / 2));
}

__global__ void __launch_bounds__(256) latent_append_kernel(AppendArgs a) {
  __shared__ float red[4];
  append_row(a, blockIdx.x, red);
}

struct PackArgs {
  const float* q;
  const void* k;
  const float* cache;
  const float* cos;
  const float* sin;
  void* qp;
  void* kp;
  size_t q_stride;
  int t, pos, heads, dim, rot, rank, q_rows, k_rows;
  float q_mul;
  bool q_vec;  // a head's query starts on 16 bytes
};

// The operands of the scores as the kernel below reads them: [heads][rows][DQ], queries rotated, keys with the shared rotated part
// behind each head's own, zeros past the last element and the last position.  A thread makes 16 bytes.
template <typename T, int DQ>
__global__ void __launch_bounds__(256) latent_pack_kernel(PackArgs a) {
  constexpr int E = 16 / sizeof(T), CH = DQ / E;
  const size_t e0 = (size_t)blockIdx.x * 256 + threadIdx.x, all = (size_t)(a.q_rows + a.k_rows) * CH;
  if (e0 >= all) return;
  const int head = blockIdx.y, row = (int)(e0 / CH), c = (int)(e0 % CH) * E;
  const bool is_q = row < a.q_rows;
  const int r = is_q ? row : row - a.q_rows, p = is_q ? a.pos + r : r;
  T v[E];
  if (is_q ? r < a.t : r < a.pos + a.t) {
    const float* qr = is_q ? a.q + (size_t)r * a.q_stride + (size_t)head * (a.dim + a.rot) : nullptr;
    const T* kr = static_cast<const T*>(a.k) + (size_t)r * a.heads * a.dim + (size_t)head * a.dim;
    const float* rr = a.cache + (size_t)r * (a.rank + a.rot) + a.rank;
    if (a.dim % 8 == 0 && !is_q && c < a.dim) {  // a whole piece of a head's own key
      __builtin_memcpy(v, __builtin_assume_aligned(kr + c, 16), 16);
    } else if (a.dim % 8 == 0 && is_q && c < a.dim && a.q_vec) {
#pragma unroll
      for (int e = 0; e < E; e += 4) {
        const f32x4_t f = *reinterpret_cast<const f32x4_t*>(qr + c + e);
#pragma unroll
        for (int i = 0; i < 4; ++i) v[e + i] = to_elem<T>(f[i] * a.q_mul);
      }
    } else
#pragma unroll
    for (int e = 0; e < E; ++e) {
      const int d = c + e;
      if (d < a.dim) v[e] = is_q ? to_elem<T>(qr[d] * a.q_mul) : kr[d];
      else if (d < a.dim + a.rot)
        v[e] = to_elem<T>(is_q ? rotated(qr + a.dim, d - a.dim, a.rot, a.cos + (size_t)p * (a.rot / 2), a.sin + (size_t)p * (a.rot / 2)) * a.q_mul : rr[d - a.dim]);
      else v[e] = T(0);
    }
  } else {
#pragma unroll
    for (int e = 0; e < E; ++e) v[e] = T(0);
  }
  T* out = static_cast<T*>(is_q ? a.qp : a.kp) + ((size_t)head * (is_q ? a.q_rows : a.k_rows) + r) * DQ + c;
  u32x4_t chunk;
  __builtin_memcpy(&chunk, v, 16);
  *reinterpret_cast<u32x4_t*>(out) = chunk;
}

template <typename T, int DQ, int DV>
int launch_rows(ughip_device* dev, AttRowsArgs a, PackArgs pk) {
  constexpr int bytes = attention_rows_lds_bytes<T, DQ, DV>();
  static_assert(bytes <= 160 * 1024, "tile does not fit LDS");
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(attention_rows_kernel<T, DQ, DV>), hipFuncAttributeMaxDynamicSharedMemorySize, bytes);
  UGHIP_HIPCHK(attr);
  pk.q_rows = (pk.t + ATT_QT - 1) / ATT_QT * ATT_QT, pk.k_rows = (pk.pos + pk.t + ATT_KT - 1) / ATT_KT * ATT_KT;
  const size_t q_bytes = (size_t)pk.heads * pk.q_rows * DQ * sizeof(T), k_bytes = (size_t)pk.heads * pk.k_rows * DQ * sizeof(T);
  void* ws = nullptr;
  if (int rc = rows_scratch(dev, q_bytes + k_bytes, &ws)) return rc;
  pk.qp = ws, pk.kp = static_cast<char*>(ws) + q_bytes;
  a.q = pk.qp, a.k = pk.kp, a.q_rows = pk.q_rows, a.k_rows = pk.k_rows, a.kv_heads = pk.heads, a.window = 0;
  constexpr int CH = DQ * (int)sizeof(T) / 16;
  const size_t pieces = (size_t)(pk.q_rows + pk.k_rows) * CH;
  latent_pack_kernel<T, DQ><<<dim3((unsigned)((pieces + 255) / 256), (unsigned)pk.heads), 256, 0, dev->stream>>>(pk);
  UGHIP_HIPCHK(hipGetLastError());
  attention_rows_kernel<T, DQ, DV><<<dim3((unsigned)pk.heads, (unsigned)(pk.q_rows / ATT_QT)), attention_rows_threads<T, DQ, DV>(), bytes, dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
template <typename T>
int launch_rows_any(ughip_device* dev, const AttRowsArgs& a, const PackArgs& pk) {
  const int dq = pk.dim + pk.rot;
  if (dq <= 64 && a.vdim <= 64) return launch_rows<T, 64, 64>(dev, a, pk);
  if (dq <= 128 && a.vdim <= 128) return launch_rows<T, 128, 128>(dev, a, pk);
  if (dq <= 192 && a.vdim <= 128) return launch_rows<T, 192, 128>(dev, a, pk);
  return launch_rows<T, 256, 256>(dev, a, pk);
}

// ---- few positions ----------------------------------------------------------------------------------------------------------
// Four consecutive elements of a matrix row (V4: they are there and aligned).
template <bool V4>
__device__ __forceinline__ f32x4_t load4(const float* p, int left) {
  if constexpr (V4) return *reinterpret_cast<const f32x4_t*>(p);
  f32x4_t v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (i < left) v[i] = p[i];
  return v;
}
template <bool V4>
__device__ __forceinline__ f32x4_t load4(const uint16_t* p, int left) {
  if constexpr (V4) {
    const uint2 v = *reinterpret_cast<const uint2*>(p);
    return f32x4_t{__uint_as_float(v.x << 16), __uint_as_float(v.x & 0xffff0000u), __uint_as_float(v.y << 16), __uint_as_float(v.y & 0xffff0000u)};
  }
  f32x4_t v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int i = 0; i < 4; ++i)
    if (i < left) v[i] = bf16_to_f32(p[i]);
  return v;
}

// qa[(i heads + h), 0 .. rank) = scale * sum_d q_h[d] w_uk[h dim + d, :], then the rotated part (scaled too).  A workgroup takes a
// head and 128 columns; eight groups of 32 threads share d.  One workgroup more than there are heads appends the step's row.
template <typename WT, bool V4>
__global__ void __launch_bounds__(256) latent_absorb_kernel(const float* __restrict__ q, size_t q_stride, const WT* __restrict__ w, AppendArgs ap, float* __restrict__ qa,
                                                            int heads, int dim, float scale) {
  __shared__ float part[8][128];
  __shared__ float red[4];
  const int h = blockIdx.x, c0 = blockIdx.y * 128, cg = threadIdx.x & 31, dg = threadIdx.x >> 5, rank = ap.rank, rot = ap.rot, L = rank + rot;
  const int i = blockIdx.z;
  if (h == heads) {
    if (blockIdx.y == 0) append_row(ap, i, red);
    return;
  }
  const float* qr = q + (size_t)i * q_stride + (size_t)h * (dim + rot);
  float* out = qa + ((size_t)i * heads + h) * L;
  f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
  const int c = c0 + cg * 4;
  if (c < rank) {
    const WT* wr = w + (size_t)h * dim * rank + c;
#pragma unroll 8
    for (int d = dg; d < dim; d += 8) {
      const float qv = qr[d];
      const f32x4_t v = load4<V4>(wr + (size_t)d * rank, rank - c);
      acc.x += qv * v.x;
      acc.y += qv * v.y;
      acc.z += qv * v.z;
      acc.w += qv * v.w;
    }
  }
#pragma unroll
  for (int e = 0; e < 4; ++e) part[dg][cg * 4 + e] = acc[e];
  __syncthreads();
  if (threadIdx.x < 128 && c0 + (int)threadIdx.x < rank) {
    float v = 0.f;
#pragma unroll
    for (int g = 0; g < 8; ++g) v += part[g][threadIdx.x];
    out[c0 + threadIdx.x] = v * scale;
  }
  if (blockIdx.y == 0) {
    const size_t p = (ap.pos + i) * (rot / 2);
    for (int e = threadIdx.x; e < rot; e += 256) out[rank + e] = rotated(qr + dim, e, rot, ap.cos + p, ap.sin + p) * scale;
  }
}

struct SplitArgs {
  const float* qa;
  const float* cache;
  float* acc;  // [splits, rows, rank]
  float* ml;   // [splits, rows, 2]
  int rows, heads, pos, keys, rank, L, tiles_per_split;
};

constexpr int SK = 32, S_ROW = SK + 4, SPLIT_WAVES = 16, SPLIT_PARTS = SPLIT_WAVES / 2;
__host__ __device__ inline int split_row(int L) { return ((L + 15) & ~15) + 4; }
inline size_t split_lds_bytes(int L) { return ((size_t)(SK + 16) * split_row(L) + SPLIT_PARTS * 16 * S_ROW + 48) * sizeof(float); }

// N rows of L floats (rows from `left` on and columns from L on are zeros) through registers to LDS, a row per wave and turn.
// NC > 0: rows of L % 4 == 0 elements in NC pieces of 16 bytes per lane, all on their way at once.
template <int N, int NC>
struct RowsAhead {
  static constexpr int TURNS = N / SPLIT_WAVES;
  f32x4_t v[TURNS][NC ? NC : 1];
  const float* from;
  int rows;
  __device__ void load(const float* src, int L, int left) {
    from = src, rows = left;
    if constexpr (NC != 0) {
      const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
      for (int u = 0; u < TURNS; ++u)
#pragma unroll
        for (int b = 0; b < NC; ++b) {
          const int r = wave + u * SPLIT_WAVES, c = b * 256 + lane * 4;
          v[u][b] = *reinterpret_cast<const f32x4_t*>(src + (r < left && c < L ? (size_t)r * L + c : 0));  // every lane loads: no branches between loads
        }
    }
  }
  __device__ void store(float* lds, int ld, int L, int Lp) const {
    const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
#pragma unroll
    for (int u = 0; u < TURNS; ++u) {
      const int r = wave + u * SPLIT_WAVES;
      if constexpr (NC != 0) {
#pragma unroll
        for (int b = 0; b < NC; ++b) {
          const int c = b * 256 + lane * 4;
          if (c < Lp) *reinterpret_cast<f32x4_t*>(lds + r * ld + c) = r < rows && c < L ? v[u][b] : f32x4_t{0.f, 0.f, 0.f, 0.f};
        }
      } else {
        for (int c = lane; c < Lp; c += 64) lds[r * ld + c] = r < rows && c < L ? from[(size_t)r * L + c] : 0.f;
      }
    }
  }
};

// NT: 16-column tiles of the result per wave; NC as in RowsAhead, the next tile on its way while this one is multiplied
template <int NT, int NC>
__global__ void __launch_bounds__(64 * SPLIT_WAVES) latent_split_kernel(SplitArgs a) {
  extern __shared__ __attribute__((aligned(16))) float sl[];
  const int ld = split_row(a.L), Lp = (a.L + 15) & ~15;
  float* Ks = sl;                     // [SK][ld]
  float* Qs = Ks + SK * ld;           // [16][ld]
  float* Sp = Qs + 16 * ld;           // [SPLIT_PARTS][16][S_ROW] parts of the scores
  float* Ps = Sp;                     // [16][S_ROW] weights, in place of the first part
  float* mrow = Sp + SPLIT_PARTS * 16 * S_ROW;  // running maximum, sum, and this tile's factor
  float* lrow = mrow + 16;
  float* arow = lrow + 16;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, g = lane >> 4;
  const int r0 = blockIdx.x * 16, split = blockIdx.y;
  const int k_begin = split * a.tiles_per_split * SK, k_stop = min(a.keys, k_begin + a.tiles_per_split * SK);
  RowsAhead<SK, NC> ahead;
  {
    RowsAhead<16, NC> queries;
    queries.load(a.qa + (size_t)r0 * a.L, a.L, a.rows - r0);
    ahead.load(a.cache + (size_t)k_begin * a.L, a.L, k_stop - k_begin);
    queries.store(Qs, ld, a.L, Lp);
  }
  if (threadIdx.x < 16) mrow[threadIdx.x] = -INFINITY, lrow[threadIdx.x] = 0.f;
  f32x4_t acc[NT];
#pragma unroll
  for (int i = 0; i < NT; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
  for (int k0 = k_begin; k0 < k_stop; k0 += SK) {
    __syncthreads();
    ahead.store(Ks, ld, a.L, Lp);
    if (k0 + SK < k_stop) ahead.load(a.cache + (size_t)(k0 + SK) * a.L, a.L, k_stop - k0 - SK);
    __syncthreads();
    {  // wave: 16 keys (wave % 2), every SPLIT_PARTS-th run of 16 elements (from wave / 2)
      f32x4_t s = {0.f, 0.f, 0.f, 0.f}, s2 = s;  // two chains
      const int kb = (wave & 1) * 16;
      for (int c = (wave >> 1) * 16; c < Lp; c += 16 * SPLIT_PARTS) {
        const f32x4_t x = *reinterpret_cast<const f32x4_t*>(Qs + j * ld + c + 4 * g), y = *reinterpret_cast<const f32x4_t*>(Ks + (kb + j) * ld + c + 4 * g);
        s = __builtin_amdgcn_mfma_f32_16x16x4f32(x.x, y.x, s, 0, 0, 0);
        s2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.y, y.y, s2, 0, 0, 0);
        s = __builtin_amdgcn_mfma_f32_16x16x4f32(x.z, y.z, s, 0, 0, 0);
        s2 = __builtin_amdgcn_mfma_f32_16x16x4f32(x.w, y.w, s2, 0, 0, 0);
      }
      s += s2;
#pragma unroll
      for (int e = 0; e < 4; ++e) Sp[((wave >> 1) * 16 + 4 * g + e) * S_ROW + kb + j] = s[e];
    }
    __syncthreads();
    if (wave < 4) {  // row 4 wave + g, keys j and j + 16
      const int r = 4 * wave + g, limit = a.pos + (r0 + r) / a.heads;
      float s0 = 0.f, s1 = 0.f;
#pragma unroll
      for (int x = 0; x < SPLIT_PARTS; ++x) s0 += Sp[(x * 16 + r) * S_ROW + j], s1 += Sp[(x * 16 + r) * S_ROW + j + 16];
      if (k0 + j > limit || k0 + j >= k_stop) s0 = -INFINITY;
      if (k0 + j + 16 > limit || k0 + j + 16 >= k_stop) s1 = -INFINITY;
      float top = fmaxf(s0, s1);
      for (int d = 8; d; d >>= 1) top = fmaxf(top, __shfl_xor(top, d, 64));
      const float before = mrow[r];
      top = fmaxf(top, before);
      const float base = top == -INFINITY ? 0.f : top;  // nothing of this split is visible to the row so far
      const float p0 = expf(s0 - base), p1 = expf(s1 - base), alpha = expf(before - base);
      float part = p0 + p1;
      for (int d = 8; d; d >>= 1) part += __shfl_xor(part, d, 64);
      Ps[r * S_ROW + j] = p0;
      Ps[r * S_ROW + j + 16] = p1;
      if (j == 0) {
        mrow[r] = top;
        lrow[r] = lrow[r] * alpha + part;
        arow[r] = alpha;
      }
    }
    __syncthreads();
    float al[4];
#pragma unroll
    for (int e = 0; e < 4; ++e) al[e] = arow[4 * g + e];
    float pf[SK / 4];
#pragma unroll
    for (int kk = 0; kk < SK / 4; ++kk) pf[kk] = Ps[j * S_ROW + 4 * kk + g];
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      const int c0 = (wave + SPLIT_WAVES * i) * 16;
      if (c0 >= a.rank) continue;  // uniform over the wave (columns up to Lp exist in LDS)
#pragma unroll
      for (int e = 0; e < 4; ++e) acc[i][e] *= al[e];
#pragma unroll
      for (int kk = 0; kk < SK / 4; ++kk) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(pf[kk], Ks[(4 * kk + g) * ld + c0 + j], acc[i], 0, 0, 0);
    }
  }
  __syncthreads();
#pragma unroll
  for (int i = 0; i < NT; ++i) {
    const int c = (wave + SPLIT_WAVES * i) * 16 + j;
    if (c >= a.rank) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = r0 + 4 * g + e;
      if (r < a.rows) a.acc[((size_t)split * a.rows + r) * a.rank + c] = acc[i][e];
    }
  }
  if (threadIdx.x < 16 && r0 + (int)threadIdx.x < a.rows) {
    float* o = a.ml + ((size_t)split * a.rows + r0 + threadIdx.x) * 2;
    o[0] = mrow[threadIdx.x];
    o[1] = lrow[threadIdx.x];
  }
}

// The parts of one (position, head) added up, then 16 elements of the head's result through the values' up-projection.
constexpr int MERGE_V = 16, MERGE_WAVES = 16, MERGE_THREADS = 64 * MERGE_WAVES, SPLITS_MAX = 128;
template <typename WT, bool V4>
__global__ void __launch_bounds__(MERGE_THREADS) latent_merge_kernel(const float* __restrict__ acc, const float* __restrict__ ml, const WT* __restrict__ w, float* __restrict__ dst,
                                                           size_t dst_stride, int rows, int splits, int heads, int rank, int vdim) {
  extern __shared__ __attribute__((aligned(16))) float lat[];  // [rank], zeros up to a multiple of 256
  __shared__ float fac[SPLITS_MAX];
  __shared__ f32x4_t part[MERGE_THREADS];
  const int h = blockIdx.x, i = blockIdx.y, v0 = blockIdx.z * MERGE_V, row = i * heads + h;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  f32x4_t held[MERGE_V / MERGE_WAVES][2];  // the first 512 elements of the wave's matrix rows, asked for before anything else
#pragma unroll
  for (int u = 0; u < MERGE_V / MERGE_WAVES; ++u)
#pragma unroll
    for (int b = 0; b < 2; ++b) {
      const int v = v0 + wave + MERGE_WAVES * u, c = b * 256 + lane * 4;
      held[u][b] = v < vdim && c < rank ? load4<V4>(w + ((size_t)h * vdim + v) * rank + c, rank - c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    }
  if (wave == 0) {
    float m[SPLITS_MAX / 64], l[SPLITS_MAX / 64], top = -INFINITY, sum = 0.f;
#pragma unroll
    for (int u = 0; u < SPLITS_MAX / 64; ++u) {
      const int s = lane + 64 * u;
      m[u] = s < splits ? ml[((size_t)s * rows + row) * 2] : -INFINITY, l[u] = s < splits ? ml[((size_t)s * rows + row) * 2 + 1] : 0.f;
      top = fmaxf(top, m[u]);
    }
    for (int d = 32; d; d >>= 1) top = fmaxf(top, __shfl_xor(top, d, 64));
#pragma unroll
    for (int u = 0; u < SPLITS_MAX / 64; ++u) m[u] = expf(m[u] - top), sum += m[u] * l[u];
    for (int d = 32; d; d >>= 1) sum += __shfl_xor(sum, d, 64);
#pragma unroll
    for (int u = 0; u < SPLITS_MAX / 64; ++u) fac[lane + 64 * u] = m[u] / sum;
  }
  __syncthreads();
  const int padded = (rank + 255) & ~255;
  const float* mine = acc + (size_t)row * rank;
  const size_t step = (size_t)rows * rank;
  if (V4 && rank <= 1024) {
    // four columns per thread, the splits dealt to as many threads per column as there are
    const int nc = padded / 4, share = MERGE_THREADS / nc, c = (threadIdx.x % nc) * 4, g = threadIdx.x / nc;  // nc: 64, 128, 192 or 256; a share of 4 to 16
    f32x4_t v = {0.f, 0.f, 0.f, 0.f};
    if (c < rank && g < share) {
#pragma unroll 16
      for (int s = g; s < splits; s += share) v += *reinterpret_cast<const f32x4_t*>(mine + s * step + c) * fac[s];
    }
    part[threadIdx.x] = v;
    __syncthreads();
    if (g == 0) {
      for (int k = 1; k < share; ++k) v += part[k * nc + threadIdx.x];
      *reinterpret_cast<f32x4_t*>(lat + c) = v;
    }
  } else {
    for (int c = threadIdx.x; c < padded; c += MERGE_THREADS) {
      float v = 0.f;
      if (c < rank) {
#pragma unroll 16
        for (int s = 0; s < splits; ++s) v += fac[s] * mine[s * step + c];
      }
      lat[c] = v;
    }
  }
  __syncthreads();
#pragma unroll
  for (int u = 0; u < MERGE_V / MERGE_WAVES; ++u) {
    const int v = v0 + wave + MERGE_WAVES * u;
    if (v >= vdim) break;
    const WT* wr = w + ((size_t)h * vdim + v) * rank;
    float s = 0.f;
    for (int c = lane * 4; c < rank; c += 256) {
      const f32x4_t a = c < 256 ? held[u][0] : c < 512 ? held[u][1] : load4<V4>(wr + c, rank - c), b = *reinterpret_cast<const f32x4_t*>(lat + c);
      s += a.x * b.x;
      s += a.y * b.y;
      s += a.z * b.z;
      s += a.w * b.w;
    }
    s = wave_sum(s);
    if (lane == 0) dst[(size_t)i * dst_stride + (size_t)h * vdim + v] = s;
  }
}

int check_tables(const ughip_device* dev, const ughip_slice* cos, const ughip_slice* sin, size_t table_rows, size_t pos, size_t t, size_t rot, const char* what) {
  if (rot == 0 || rot % 2 != 0) return set_error(UGHIP_ERR_INVALID, "%s: a rotated part of %zu elements", what, rot);
  if (pos + t > table_rows) return set_error(UGHIP_ERR_BOUNDS, "%s: positions up to %zu, tables for %zu", what, pos + t, table_rows);
  for (const ughip_slice* s : {cos, sin})
    if (int rc = check_buf(dev, s, table_rows * (rot / 2), UGHIP_F32, what)) return rc;
  return UGHIP_OK;
}

}  // namespace

extern "C" int ughip_latent_append(ughip_device* dev, ughip_view kv, const ughip_slice* w, float eps, const ughip_slice* cos, const ughip_slice* sin, size_t table_rows,
                                   ughip_slice* cache, size_t cap, size_t pos, size_t t, size_t rank, size_t rot) {
  const char* what = "latent_append";
  if (!dev) return set_error(UGHIP_ERR_INVALID, "%s: null device", what);
  if (rank == 0 || rank > 65536) return set_error(UGHIP_ERR_INVALID, "%s: rank %zu", what, rank);
  if (int rc = check_view(dev, kv, t, rank + rot, UGHIP_F32, what)) return rc;
  if (int rc = check_buf(dev, w, rank, UGHIP_F32, what)) return rc;
  if (int rc = check_tables(dev, cos, sin, table_rows, pos, t, rot, what)) return rc;
  if (pos + t > cap) return set_error(UGHIP_ERR_BOUNDS, "%s: %zu rows exceed the cache's %zu", what, pos + t, cap);
  if (int rc = check_buf(dev, cache, cap * (rank + rot), UGHIP_F32, what)) return rc;
  if (t == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  latent_append_kernel<<<(unsigned)t, 256, 0, dev->stream>>>(
      AppendArgs{view_ptr<float>(kv), kv.stride, buf_ptr<float>(w), eps, buf_ptr<float>(cos), buf_ptr<float>(sin), static_cast<float*>(cache->ptr), pos, (int)rank, (int)rot});
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_latent_attention_rows(ughip_device* dev, ughip_view q, const ughip_slice* k, const ughip_slice* v_t, size_t v_stride, const ughip_slice* cache,
                                           const ughip_slice* cos, const ughip_slice* sin, size_t table_rows, ughip_view dst, size_t t, size_t pos, size_t heads, size_t dim,
                                           size_t rot, size_t vdim, size_t rank, float scale) {
  const char* what = "latent_attention_rows";
  if (!dev || !k || !v_t) return set_error(UGHIP_ERR_INVALID, "%s: null argument", what);
  if (heads == 0 || dim == 0 || vdim == 0 || rank == 0 || dim + rot > 256 || vdim > 256 || heads > 65535)
    return set_error(UGHIP_ERR_UNSUPPORTED, "%s: heads %zu of %zu + %zu and %zu elements (built for up to 256)", what, heads, dim, rot, vdim);
  const size_t s = pos + t;
  if (s > 0x3fffffffull || v_stride % 64 != 0 || v_stride < s) return set_error(UGHIP_ERR_INVALID, "%s: %zu positions, value rows of %zu (whole tiles of 64)", what, s, v_stride);
  if (k->dtype != v_t->dtype || (k->dtype != UGHIP_F32 && k->dtype != UGHIP_BF16)) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: keys and values are both F32 or both BF16", what);
  if (int rc = check_view(dev, q, t, heads * (dim + rot), UGHIP_F32, what)) return rc;
  if (int rc = check_buf(dev, k, s * heads * dim, -1, what)) return rc;
  if (int rc = check_buf(dev, v_t, heads * vdim * v_stride, -1, what)) return rc;
  if (int rc = check_buf(dev, cache, s * (rank + rot), UGHIP_F32, what)) return rc;
  if (int rc = check_tables(dev, cos, sin, table_rows, pos, t, rot, what)) return rc;
  if (int rc = check_view(dev, dst, t, heads * vdim, -1, what)) return rc;
  const bool bf16 = dst.s->dtype == UGHIP_BF16;
  if (!bf16 && dst.s->dtype != UGHIP_F32) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: the result is F32 or BF16", what);
  if (t == 0) return UGHIP_OK;
  if ((t + ATT_QT - 1) / ATT_QT > 65535) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: too many positions", what);
  if (int rc = device_activate(dev)) return rc;
  AttRowsArgs a{};
  a.v = v_t->ptr, a.dst = static_cast<char*>(dst.s->ptr) + dst.offset * (bf16 ? 2 : 4), a.v_stride = v_stride, a.dst_stride = dst.stride;
  a.t = (int)t, a.pos = (int)pos, a.vdim = (int)vdim, a.dst_bf16 = bf16;
  PackArgs pk{};
  pk.q = view_ptr<float>(q), pk.k = k->ptr, pk.cache = buf_ptr<float>(cache), pk.cos = buf_ptr<float>(cos), pk.sin = buf_ptr<float>(sin), pk.q_stride = q.stride;
  pk.t = (int)t, pk.pos = (int)pos, pk.heads = (int)heads, pk.dim = (int)dim, pk.rot = (int)rot, pk.rank = (int)rank;
  pk.q_mul = scale * 1.4426950408889634f;  // the weights are powers of two
  pk.q_vec = (dim + rot) % 4 == 0 && q.stride % 4 == 0 && (reinterpret_cast<uintptr_t>(pk.q) & 15) == 0;
  return k->dtype == UGHIP_BF16 ? launch_rows_any<uint16_t>(dev, a, pk) : launch_rows_any<float>(dev, a, pk);
}

extern "C" int ughip_latent_attention_absorbed(ughip_device* dev, ughip_view q, ughip_view kv, const ughip_slice* kv_norm, float eps, const ughip_slice* w_uk,
                                               const ughip_slice* w_uv, ughip_slice* cache, size_t cap, const ughip_slice* cos, const ughip_slice* sin, size_t table_rows,
                                               ughip_view dst, size_t t, size_t pos, size_t heads, size_t dim, size_t rot, size_t vdim, size_t rank, float scale) {
  const char* what = "latent_attention_absorbed";
  if (!dev || !w_uk || !w_uv) return set_error(UGHIP_ERR_INVALID, "%s: null argument", what);
  if (heads == 0 || dim == 0 || vdim == 0 || rank == 0 || heads > 65535 || t > 65535) return set_error(UGHIP_ERR_INVALID, "%s: bad shape", what);
  const size_t s = pos + t, L = rank + rot, rows = t * heads;
  if (s > 0x3fffffffull || rows > 0x3fffffffull) return set_error(UGHIP_ERR_INVALID, "%s: %zu positions", what, s);
  if (rank > 1024 || split_lds_bytes((int)L) > 160 * 1024) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: latents of %zu + %zu elements", what, rank, rot);
  if (w_uk->dtype != w_uv->dtype || (w_uk->dtype != UGHIP_F32 && w_uk->dtype != UGHIP_BF16)) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: matrices are both F32 or both BF16", what);
  if (int rc = check_view(dev, q, t, heads * (dim + rot), UGHIP_F32, what)) return rc;
  if (int rc = check_buf(dev, w_uk, heads * dim * rank, -1, what)) return rc;
  if (int rc = check_buf(dev, w_uv, heads * vdim * rank, -1, what)) return rc;
  if (s > cap) return set_error(UGHIP_ERR_BOUNDS, "%s: %zu rows exceed the cache's %zu", what, s, cap);
  if (int rc = check_buf(dev, cache, cap * L, UGHIP_F32, what)) return rc;
  if (kv.s) {
    if (int rc = check_view(dev, kv, t, L, UGHIP_F32, what)) return rc;
    if (int rc = check_buf(dev, kv_norm, rank, UGHIP_F32, what)) return rc;
  }
  if (int rc = check_tables(dev, cos, sin, table_rows, pos, t, rot, what)) return rc;
  if (int rc = check_view(dev, dst, t, heads * vdim, UGHIP_F32, what)) return rc;
  if (t == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  const size_t tiles = (s + SK - 1) / SK, row_blocks = (rows + 15) / 16;
  size_t splits = row_blocks >= 256 ? 1 : 256 / row_blocks;
  if (splits > SPLITS_MAX) splits = SPLITS_MAX;
  if (splits > tiles) splits = tiles;
  const size_t per = (tiles + splits - 1) / splits;
  splits = (tiles + per - 1) / per;
  auto up = [](size_t v) { return (v + 63) & ~(size_t)63; };
  const size_t n_qa = up(rows * L), n_ml = up(splits * rows * 2), n_acc = splits * rows * rank;
  void* ws = nullptr;
  if (int rc = rows_scratch(dev, (n_qa + n_ml + n_acc) * sizeof(float), &ws)) return rc;
  float* qa = static_cast<float*>(ws);
  SplitArgs a{qa, buf_ptr<float>(cache), qa + n_qa + n_ml, qa + n_qa, (int)rows, (int)heads, (int)pos, (int)s, (int)rank, (int)L, (int)per};
  const AppendArgs ap{view_ptr<float>(kv), kv.stride, buf_ptr<float>(kv_norm), eps, buf_ptr<float>(cos), buf_ptr<float>(sin), static_cast<float*>(cache->ptr), pos, (int)rank, (int)rot};
  const dim3 g1((unsigned)(heads + (kv.s ? 1 : 0)), (unsigned)((rank + 127) / 128), (unsigned)t);
  const bool bf = w_uk->dtype == UGHIP_BF16, v4 = rank % 4 == 0;
  auto absorb = [&](auto* w, auto vec) {
    latent_absorb_kernel<std::remove_const_t<std::remove_pointer_t<decltype(w)>>, decltype(vec)::value>
        <<<g1, 256, 0, dev->stream>>>(view_ptr<float>(q), q.stride, w, ap, qa, (int)heads, (int)dim, scale);
  };
  if (bf && v4) absorb(buf_ptr<uint16_t>(w_uk), std::true_type{});
  else if (bf) absorb(buf_ptr<uint16_t>(w_uk), std::false_type{});
  else if (v4) absorb(buf_ptr<float>(w_uk), std::true_type{});
  else absorb(buf_ptr<float>(w_uk), std::false_type{});
  UGHIP_HIPCHK(hipGetLastError());
  const dim3 g2((unsigned)row_blocks, (unsigned)splits);
  const size_t lds = split_lds_bytes((int)L);
  auto split_go = [&](auto kernel) {
    if (lds > 64 * 1024)
      if (hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); e != hipSuccess) return e;
    kernel<<<g2, 64 * SPLIT_WAVES, lds, dev->stream>>>(a);
    return hipSuccess;
  };
  auto split_any = [&](auto nc) {
    constexpr int NC = decltype(nc)::value;
    return rank <= 256 ? split_go(latent_split_kernel<1, NC>) : rank <= 512 ? split_go(latent_split_kernel<2, NC>) : split_go(latent_split_kernel<4, NC>);
  };
  using std::integral_constant;
  const size_t nc = L % 4 ? 0 : (((L + 15) & ~(size_t)15) + 255) / 256;  // at most 3: the rows' bytes in LDS are limited above
  UGHIP_HIPCHK(nc == 0 ? split_any(integral_constant<int, 0>{}) : nc == 1 ? split_any(integral_constant<int, 1>{}) : nc == 2 ? split_any(integral_constant<int, 2>{})
                                                                                                                           : split_any(integral_constant<int, 3>{}));
  UGHIP_HIPCHK(hipGetLastError());
  const dim3 g3((unsigned)heads, (unsigned)t, (unsigned)((vdim + MERGE_V - 1) / MERGE_V));
  const size_t lds3 = ((rank + 255) & ~(size_t)255) * sizeof(float);
  auto merge = [&](auto* w, auto vec) {
    latent_merge_kernel<std::remove_const_t<std::remove_pointer_t<decltype(w)>>, decltype(vec)::value>
        <<<g3, MERGE_THREADS, lds3, dev->stream>>>(a.acc, a.ml, w, view_ptr<float>(dst), dst.stride, (int)rows, (int)splits, (int)heads, (int)rank, (int)vdim);
  };
  if (bf && v4) merge(buf_ptr<uint16_t>(w_uv), std::true_type{});
  else if (bf) merge(buf_ptr<uint16_t>(w_uv), std::false_type{});
  else if (v4) merge(buf_ptr<float>(w_uv), std::true_type{});
  else merge(buf_ptr<float>(w_uv), std::false_type{});
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
