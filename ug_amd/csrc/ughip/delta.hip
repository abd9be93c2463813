// A gated delta rule with a decay per key channel (ughip_layers.h).
//
//   S_i = diag(g_i) S_{i-1} + k_i u_i^T,   u_i = beta_i (v_i - (diag(g_i) S_{i-1})^T k_i),   o_i = S_i^T q_i
//
// Several positions run in chunks of C.  With G_i = g_1 g_2 .. g_i inside a chunk (per channel, from the chunk's start) and S the state in
// front of it:
//   A_ij = beta_i sum_c k_ic k_jc (G_i / G_j)_c (j < i),   P_ij = sum_c q_ic k_jc (G_i / G_j)_c (j <= i)
//   (I + A) U = beta V - (beta G K) S,   o_i = (G_i q_i)^T S + sum_{j <= i} P_ij u_j,   S' = diag(G_C) S + sum_j (G_C / G_j k_j) u_j^T
//   delta_prepare  (all chunks at once)  W and V' with (I + A) W = beta G K, (I + A) V' = beta V; P; G q; G_C / G k
//   delta_scan     (chunks in order)     U = V' - W S, then S'; leaves U and the S in front of every chunk
//   delta_out      (all chunks at once)  o, normed and gated
// A quotient G_i / G_j is never taken as one: with strong decays both are too small for f32.  The logarithms are summed inside blocks of
// 16 rows; between two blocks the quotient is split at the later block's start into two factors <= 1; inside a block it is the product of
// G_i and 1 / G_j from the block's start as long as the latter stays small, and an exponential per pair otherwise.
// The triangular system is solved by blocks: the inverses of its diagonal blocks by substitution, the rest as products.
// The products are v_mfma_f32_16x16x4_f32 (lane l: row or column l % 16, k = l / 16; result element e: row 4 (l / 16) + e, column
// l % 16).  Four of them take k = 4 (l / 16) + e as element e of a lane's 16 bytes, on both sides: a left operand is then 16 bytes of a
// row, and a result is a right operand as it is.  That is how the state stays in registers over the scan (every wave holds all
// channels of 16 columns; what a wave updates of them goes round through LDS), and the layout U and the states are left in.
#include <hip/hip_runtime.h>

#include <type_traits>

#include "bf16_split.h"
#include "layers.h"

using namespace ughip;

namespace {

constexpr float UNIT_EPS = 1e-6f, LOG2E = 1.4426950408889634f;

__device__ __forceinline__ f32x4_t mfma16(float x, float y, f32x4_t acc) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, acc, 0, 0, 0); }
// acc += x y over 16 elements of k
__device__ __forceinline__ f32x4_t mfma16x16(const f32x4_t& x, const f32x4_t& y, f32x4_t acc) {
  acc = mfma16(x.x, y.x, acc);
  acc = mfma16(x.y, y.y, acc);
  acc = mfma16(x.z, y.z, acc);
  return mfma16(x.w, y.w, acc);
}
// acc[i] += x[i] y[i], the chains side by side: a product that waits for the one before it leaves the pipe idle
template <int N>
__device__ __forceinline__ void mfma16x16_each(const f32x4_t (&x)[N], const f32x4_t (&y)[N], f32x4_t (&acc)[N]) {
#pragma unroll
  for (int e = 0; e < 4; ++e)
#pragma unroll
    for (int i = 0; i < N; ++i) acc[i] = mfma16(x[i][e], y[i][e], acc[i]);
}
// Where element (row, k) of a left operand lies in its tile, and a tile's lane.
__device__ __forceinline__ int left_at(int row, int k) { return ((k >> 2) * 16 + row) * 4 + (k & 3); }
__device__ __forceinline__ float* tile_at(float* tiles, size_t tile, int lane) { return tiles + (tile * 64 + lane) * 4; }
__device__ __forceinline__ f32x4_t tile_of(const float* tiles, size_t tile, int lane) { return *reinterpret_cast<const f32x4_t*>(tiles + (tile * 64 + lane) * 4); }
__device__ __forceinline__ float exact_sigmoid(float z) { return 1.f / (1.f + expf(-z)); }
__device__ __forceinline__ f32x4_t exp2_4(const f32x4_t& v) {
  return f32x4_t{__builtin_amdgcn_exp2f(v.x), __builtin_amdgcn_exp2f(v.y), __builtin_amdgcn_exp2f(v.z), __builtin_amdgcn_exp2f(v.w)};
}

struct DeltaArgs {
  const float* qkv;  // rows behind the convolution
  const float* b;
  const float* a;
  const float* z;
  const float* a_log;
  const float* dt_bias;
  const float* norm;
  float* s;
  void* dst;
  size_t qkv_stride, b_stride, a_stride, z_stride, dst_stride;
  int t, heads, kv_heads, dim, vdim, dp, vp, chunks;  // dp: dim rounded up to 64, vp: vdim rounded up to 16
  float eps;
  bool fresh, dst_bf16;
  // What lies between the launches, per (chunk, head): tiles of 16 x 16 as the lanes of a wave hold them, 16 bytes each.  Left operands
  // (lane l: row l % 16, elements 4 (l / 16) .. + 3 of k):
  float* w;      // [C / 16][dp / 16]: W, rows are positions
  float* kd;     // [dp / 16][C / 16]: G_C / G k, rows are channels
  float* qg;     // [C / 16][dp / 16]: G q
  float* p;      // [C / 16][C / 16]: P, tiles above the diagonal are not there
  // right operands and results (lane l: column l % 16, rows 4 (l / 16) .. + 3):
  float* v;      // [vp / 16][C / 16]: V'
  float* u;      // [vp / 16][C / 16]: U
  float* s0;     // [vp / 16][dp / 16]: the state in front of the chunk
  float* gam;    // G_C of every channel
};

template <int C>
__host__ __device__ constexpr size_t prepare_lds_floats(int dp) {
  return (size_t)3 * C * (dp + 4) + (size_t)C * (C + 4) + C;
}

// four elements of a row, zeros from `left` on
template <bool VEC>
__device__ __forceinline__ f32x4_t four(const float* p, int left) {
  if constexpr (VEC) return *reinterpret_cast<const f32x4_t*>(p);
  f32x4_t v = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
  for (int e = 0; e < 4; ++e)
    if (e < left) v[e] = p[e];
  return v;
}

template <int C>
constexpr int prepare_threads() {
  return C == 64 ? 512 : 256;
}
template <int C, bool VEC>
__global__ void __launch_bounds__((prepare_threads<C>())) delta_prepare_kernel(DeltaArgs a) {
  constexpr int NB = C / 16, NT = prepare_threads<C>(), NW = NT / 64;
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int dp = a.dp, ds = dp + 4, chunk = blockIdx.x, h = blockIdx.y, g = h / (a.heads / a.kv_heads), row0 = chunk * C, rows = min(C, a.t - row0), d = a.dim;
  float* K = lds;             // [C][ds]
  float* Q = K + C * ds;      // [C][ds]
  float* B = Q + C * ds;      // [C][ds]: log2 of the decays, summed from the start of a block of 16 rows
  float* A = B + C * ds;      // [C][C + 4]: A, then the inverses of I + A in the diagonal blocks
  float* beta = A + C * (C + 4);
  constexpr int as = C + 4;
  const size_t at = (size_t)chunk * a.heads + h;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, kg = lane >> 4;
  const int d4 = dp / 4;
  const float neg = -expf(a.a_log[h]) * LOG2E;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  for (int e = threadIdx.x; e < C * d4; e += NT) {
    const int r = e / d4, c = (e - r * d4) * 4;
    f32x4_t k = zero, q = zero, l = zero;
    if (r < rows && c < d) {
      const float* row = a.qkv + (size_t)(row0 + r) * a.qkv_stride + (size_t)g * d + c;
      q = four<VEC>(row, d - c), k = four<VEC>(row + (size_t)a.kv_heads * d, d - c);
      l = four<VEC>(a.a + (size_t)(row0 + r) * a.a_stride + (size_t)h * d + c, d - c);
      const f32x4_t bias = four<VEC>(a.dt_bias + (size_t)h * d + c, d - c);
#pragma unroll
      for (int x = 0; x < 4; ++x) l[x] = c + x < d ? neg * softplus_f(l[x] + bias[x]) : 0.f;
    }
    *reinterpret_cast<f32x4_t*>(K + r * ds + c) = k;
    *reinterpret_cast<f32x4_t*>(Q + r * ds + c) = q;
    *reinterpret_cast<f32x4_t*>(B + r * ds + c) = l;
  }
  if (threadIdx.x < C) beta[threadIdx.x] = (int)threadIdx.x < rows ? exact_sigmoid(a.b[(size_t)(row0 + threadIdx.x) * a.b_stride + h]) : 0.f;
  __syncthreads();
  // unit vectors: 16 lanes per row
  const float q_scale = 1.f / sqrtf((float)d);
  for (int r = wave * 4 + kg; r < C; r += 4 * NW) {
#pragma unroll
    for (int m = 0; m < 2; ++m) {
      float* row = (m ? Q : K) + r * ds;
      float ss = 0.f;
      for (int c = j * 4; c < dp; c += 64) {
        const f32x4_t v = *reinterpret_cast<const f32x4_t*>(row + c);
        ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
      }
      const float f = (m ? q_scale : 1.f) / sqrtf(row_sum16(ss) + UNIT_EPS);
      for (int c = j * 4; c < dp; c += 64) *reinterpret_cast<f32x4_t*>(row + c) *= f;
    }
  }
  for (int x = threadIdx.x; x < dp * NB; x += NT) {
    float* col = B + (x / dp) * 16 * ds + x % dp;
    float s = 0.f;
#pragma unroll
    for (int r = 0; r < 16; ++r) col[r * ds] = s += col[r * ds];
  }
  __syncthreads();

  float* P = a.p + at * C * C;
  auto row4 = [&](const float* m, int r, int c) { return *reinterpret_cast<const f32x4_t*>(m + r * ds + c); };
  // a pair of blocks per wave and turn, those of a block with itself first
  for (int n = wave; n < NB * (NB + 1) / 2; n += NW) {
    int I = n, J = n;
    if (n >= NB) {
      I = 1;
      for (J = n - NB; J >= I; ++I) J -= I;
    }
    if (J < I) {
      f32x4_t acc[4] = {zero, zero, zero, zero};
      for (int c = 4 * kg; c < dp; c += 32) {
        f32x4_t x[4], y[4];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const int cc = c + 16 * u;  // dp is a multiple of 64
          const f32x4_t left = exp2_4(row4(B, 16 * I + j, cc));
          f32x4_t rest = row4(B, 16 * J + 15, cc) - row4(B, 16 * J + j, cc);
          for (int M = J + 1; M < I; ++M) rest += row4(B, 16 * M + 15, cc);
          y[2 * u] = y[2 * u + 1] = row4(K, 16 * J + j, cc) * exp2_4(rest);
          x[2 * u] = row4(K, 16 * I + j, cc) * left;
          x[2 * u + 1] = row4(Q, 16 * I + j, cc) * left;
        }
        mfma16x16_each(x, y, acc);
      }
      const f32x4_t ak = acc[0] + acc[2], aq = acc[1] + acc[3];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 16 * I + 4 * kg + e;
        A[i * as + 16 * J + j] = ak[e] * beta[i];
        P[(I * NB + J) * 256 + left_at(4 * kg + e, j)] = aq[e];
      }
      continue;
    }

    float least = 0.f;
    for (int c = lane; c < dp; c += 64) least = fminf(least, B[(16 * I + 15) * ds + c]);
    least = -wave_max(-least);
    if (least > -64.f) {  // the same for the whole wave
      f32x4_t acc[4] = {zero, zero, zero, zero};
      for (int c = 4 * kg; c < dp; c += 32) {
        f32x4_t x[4], y[4];
#pragma unroll
        for (int u = 0; u < 2; ++u) {
          const int cc = c + 16 * u;
          const f32x4_t l = row4(B, 16 * I + j, cc), k = row4(K, 16 * I + j, cc), left = exp2_4(l);
          y[2 * u] = y[2 * u + 1] = k * exp2_4(-l);
          x[2 * u] = k * left;
          x[2 * u + 1] = row4(Q, 16 * I + j, cc) * left;
        }
        mfma16x16_each(x, y, acc);
      }
      const f32x4_t ak = acc[0] + acc[2], aq = acc[1] + acc[3];
#pragma unroll
      for (int e = 0; e < 4; ++e) {
        const int i = 4 * kg + e, row = 16 * I + i;
        A[row * as + 16 * I + j] = j < i ? ak[e] * beta[row] : 0.f;
        P[(I * NB + I) * 256 + left_at(i, j)] = j <= i ? aq[e] : 0.f;
      }
      continue;
    }
    // row 16 I + j against rows 16 I + 4 kg ..
    float ak[4] = {0.f, 0.f, 0.f, 0.f}, aq[4] = {0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int c = 0; c < dp; c += 4) {
      const f32x4_t ki = row4(K, 16 * I + j, c), qi = row4(Q, 16 * I + j, c), bi = row4(B, 16 * I + j, c);
#pragma unroll
      for (int x = 0; x < 4; ++x) {
        const f32x4_t kj = row4(K, 16 * I + 4 * kg + x, c);
        f32x4_t diff = bi - row4(B, 16 * I + 4 * kg + x, c);
#pragma unroll
        for (int y = 0; y < 4; ++y) diff[y] = fminf(diff[y], 0.f);  // (positive only where the pair does not count)
        const f32x4_t m = kj * exp2_4(diff), k = m * ki, q = m * qi;
        ak[x] += (k.x + k.y) + (k.z + k.w);
        aq[x] += (q.x + q.y) + (q.z + q.w);
      }
    }
    const float bt = beta[16 * I + j];
#pragma unroll
    for (int x = 0; x < 4; ++x) {
      const int jj = 4 * kg + x;
      A[(16 * I + j) * as + 16 * I + jj] = jj < j ? ak[x] * bt : 0.f;
      P[(I * NB + I) * 256 + left_at(j, jj)] = jj <= j ? aq[x] : 0.f;
    }
  }
  __syncthreads();

  // the inverses of the diagonal blocks, a column per lane
  if (wave < NB && lane < 16) {
    float* block = A + 16 * wave * as + 16 * wave;
    float x[16];
#pragma unroll
    for (int i = 0; i < 16; ++i) {
      float v = i == lane ? 1.f : 0.f;
#pragma unroll
      for (int m = 0; m < i; ++m) v -= block[i * as + m] * x[m];
      x[i] = v;
    }
#pragma unroll
    for (int i = 0; i < 16; ++i) block[i * as + lane] = x[i];
  }
  __syncthreads();
  // (I + A) X = right-hand side, 16 columns per wave and turn: first the channels of beta G K, then the columns of beta V
  {
    f32x4_t m[NB][NB];
#pragma unroll
    for (int I = 0; I < NB; ++I)
#pragma unroll
      for (int J = 0; J <= I; ++J) m[I][J] = *reinterpret_cast<const f32x4_t*>(A + (16 * I + j) * as + 16 * J + 4 * kg);
    const float* values = a.qkv + (size_t)row0 * a.qkv_stride + (size_t)2 * a.kv_heads * d + (size_t)h * a.vdim;
    const int kt = dp / 16, all = kt + a.vp / 16;
    f32x4_t ahead[NB];
    auto fetch = [&](int tile) {
      if (tile < kt || tile >= all) return;  // uniform over the wave
      const int c = (tile - kt) * 16 + j;
      const float* col = values + (c < a.vdim ? c : 0);
#pragma unroll
      for (int I = 0; I < NB; ++I)
#pragma unroll
        for (int e = 0; e < 4; ++e) ahead[I][e] = col[(size_t)min(16 * I + 4 * kg + e, rows - 1) * a.qkv_stride];
    };
    fetch(wave);
    for (int tile = wave; tile < all; tile += NW) {
      f32x4_t x[NB];
      const int c = (tile < kt ? tile : tile - kt) * 16 + j;
      if (tile < kt) {
        float before = 0.f;  // blocks in front of this one
#pragma unroll
        for (int I = 0; I < NB; ++I) {
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int row = 16 * I + 4 * kg + e;
            x[I][e] = beta[row] * K[row * ds + c] * __builtin_amdgcn_exp2f(before + B[row * ds + c]);
          }
          before += B[(16 * I + 15) * ds + c];
        }
      } else {
        const float on = c < a.vdim ? 1.f : 0.f;
#pragma unroll
        for (int I = 0; I < NB; ++I)
#pragma unroll
          for (int e = 0; e < 4; ++e) x[I][e] = on * beta[16 * I + 4 * kg + e] * ahead[I][e];  // (beta is 0 past the last row)
      }
      fetch(tile + NW);
      float* W = a.w + at * C * dp;
      float* V = a.v + at * C * a.vp;
#pragma unroll
      for (int I = 0; I < NB; ++I) {
        f32x4_t acc[NB];
#pragma unroll
        for (int J = 0; J < I; ++J) acc[J] = zero;
#pragma unroll
        for (int e = 0; e < 4; ++e)
#pragma unroll
          for (int J = 0; J < I; ++J) acc[J] = mfma16(m[I][J][e], x[J][e], acc[J]);
#pragma unroll
        for (int J = 0; J < I; ++J) x[I] -= acc[J];
        x[I] = mfma16x16(m[I][I], x[I], zero);
        if (tile < kt) {
#pragma unroll
          for (int e = 0; e < 4; ++e) W[(I * kt + tile) * 256 + left_at(4 * kg + e, j)] = x[I][e];
        } else {
          *reinterpret_cast<f32x4_t*>(tile_at(V, (tile - kt) * NB + I, lane)) = x[I];
        }
      }
    }
  }
  // G q, and G_C / G k
  float* QG = a.qg + at * C * dp;
  for (int e = threadIdx.x; e < C * d4; e += NT) {
    const int tile = e / 64, r = tile / (dp / 16) * 16 + (e & 15), c = tile % (dp / 16) * 16 + (e >> 4 & 3) * 4;
    f32x4_t l = row4(B, r, c);
    for (int M = 0; M < r / 16; ++M) l += row4(B, 16 * M + 15, c);
    *reinterpret_cast<f32x4_t*>(QG + 4 * e) = row4(Q, r, c) * exp2_4(l);
  }
  float* KD = a.kd + at * C * dp;
  for (int e = threadIdx.x; e < C * d4; e += NT) {
    const int tile = e / 64, c = tile / NB * 16 + (e & 15), r = tile % NB * 16 + (e >> 4 & 3) * 4;
    float after = 0.f;
    for (int M = r / 16 + 1; M < NB; ++M) after += B[(16 * M + 15) * ds + c];
    const float end = B[(r | 15) * ds + c];
    f32x4_t v;
#pragma unroll
    for (int x = 0; x < 4; ++x) v[x] = K[(r + x) * ds + c] * __builtin_amdgcn_exp2f((end - B[(r + x) * ds + c]) + after);
    *reinterpret_cast<f32x4_t*>(KD + 4 * e) = v;
  }
  for (int c = threadIdx.x; c < dp; c += NT) {
    float all = 0.f;
#pragma unroll
    for (int M = 0; M < NB; ++M) all += B[(16 * M + 15) * ds + c];
    a.gam[at * dp + c] = __builtin_amdgcn_exp2f(all);
  }
}

// A workgroup takes a head and 16 columns of its state, dp = 16 NT.  Wave w updates the channel tiles w, w + 4, ..
template <int C, int NT>
__global__ void __launch_bounds__(256) delta_scan_kernel(DeltaArgs a) {
  constexpr int NB = C / 16, MINE = NT / 4, dp = 16 * NT;
  static_assert(NT % 4 == 0, "whole tiles per wave");
  __shared__ f32x4_t Us[NB][64];
  __shared__ f32x4_t Ss[NT][64];
  const int h = blockIdx.x, ct = blockIdx.y, p0 = ct * 16, vp = a.vp;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), j = lane & 15, kg = lane >> 4;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  const bool col_there = p0 + j < a.vdim;
  float* state = a.s + (size_t)h * a.dim * a.vdim + p0 + j;
  f32x4_t mine[MINE];
#pragma unroll
  for (int m = 0; m < MINE; ++m) {
    mine[m] = zero;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int c = 16 * (wave + 4 * m) + 4 * kg + e;
      if (!a.fresh && c < a.dim && col_there) mine[m][e] = state[(size_t)c * a.vdim];
    }
    Ss[wave + 4 * m][lane] = mine[m];
  }
  // what a chunk brings, on its way from two chunks before
  struct Held {
    f32x4_t wf[NT], v0, kf[MINE][NB], gm[MINE];
  } held[2];
  const int ub = NB == 4 ? wave : wave % NB;  // the block of 16 rows whose U the wave makes (with fewer blocks than waves: some twice)
  // (loads go out between the products: all at once they would wait for each other's turn)
  auto fetch_w = [&](Held& t, int chunk, int n0, int n1) {
    const float* w = a.w + ((size_t)min(chunk, a.chunks - 1) * a.heads + h) * C * dp;
#pragma unroll
    for (int n = n0; n < n1; ++n) t.wf[n] = tile_of(w, ub * NT + n, lane);
  };
  auto fetch_v = [&](Held& t, int chunk) { t.v0 = tile_of(a.v + ((size_t)min(chunk, a.chunks - 1) * a.heads + h) * C * vp, ct * NB + ub, lane); };
  auto fetch_k = [&](Held& t, int chunk, int m) {
    const size_t at = (size_t)min(chunk, a.chunks - 1) * a.heads + h;
    const int n = wave + 4 * m;
    t.gm[m] = *reinterpret_cast<const f32x4_t*>(a.gam + at * dp + 16 * n + 4 * kg);
#pragma unroll
    for (int b = 0; b < NB; ++b) t.kf[m][b] = tile_of(a.kd + at * C * dp, n * NB + b, lane);
  };
#pragma unroll
  for (int x = 0; x < 2; ++x) {
    fetch_w(held[x], x, 0, NT);
    fetch_v(held[x], x);
#pragma unroll
    for (int m = 0; m < MINE; ++m) fetch_k(held[x], x, m);
  }
  __syncthreads();
  auto go = [&](Held& t, int chunk) {
    const size_t at = ((size_t)chunk * a.heads + h) * (vp / 16) + ct;
    {
      f32x4_t acc[4] = {zero, zero, zero, zero};
#pragma unroll
      for (int n = 0; n < NT; n += 4) {
        const f32x4_t x[4] = {t.wf[n], t.wf[n + 1], t.wf[n + 2], t.wf[n + 3]}, y[4] = {Ss[n][lane], Ss[n + 1][lane], Ss[n + 2][lane], Ss[n + 3][lane]};
        mfma16x16_each(x, y, acc);
        fetch_w(t, chunk + 2, n, n + 4);
      }
      const f32x4_t u = t.v0 - ((acc[0] + acc[1]) + (acc[2] + acc[3]));
      Us[ub][lane] = u;
      *reinterpret_cast<f32x4_t*>(tile_at(a.u, at * NB + ub, lane)) = u;
    }
    fetch_v(t, chunk + 2);
    __syncthreads();
    f32x4_t uf[NB];
#pragma unroll
    for (int b = 0; b < NB; ++b) uf[b] = Us[b][lane];
#pragma unroll
    for (int m = 0; m < MINE; ++m) {
      *reinterpret_cast<f32x4_t*>(tile_at(a.s0, at * NT + wave + 4 * m, lane)) = mine[m];
      mine[m] = t.gm[m] * mine[m];
    }
#pragma unroll
    for (int m = 0; m < MINE; m += 2) {  // four chains: two tiles, even and odd blocks
      const int m2 = m + 1 < MINE ? m + 1 : m;
      f32x4_t acc[4] = {mine[m], zero, m + 1 < MINE ? mine[m2] : zero, zero};
#pragma unroll
      for (int b = 0; b < NB; b += 2) {
        const int b2 = b + 1 < NB ? b + 1 : b;
        const f32x4_t x[4] = {t.kf[m][b], b + 1 < NB ? t.kf[m][b2] : zero, m + 1 < MINE ? t.kf[m2][b] : zero, m + 1 < MINE && b + 1 < NB ? t.kf[m2][b2] : zero};
        const f32x4_t y[4] = {uf[b], uf[b2], uf[b], uf[b2]};
        mfma16x16_each(x, y, acc);
      }
      mine[m] = acc[0] + acc[1];
      fetch_k(t, chunk + 2, m);
      if (m + 1 < MINE) {
        mine[m2] = acc[2] + acc[3];
        fetch_k(t, chunk + 2, m2);
      }
    }
#pragma unroll
    for (int m = 0; m < MINE; ++m) Ss[wave + 4 * m][lane] = mine[m];
    __syncthreads();
  };
#pragma unroll 1
  for (int chunk = 0; chunk < a.chunks; chunk += 2) {
    go(held[0], chunk);
    if (chunk + 1 < a.chunks) go(held[1], chunk + 1);
  }
#pragma unroll
  for (int m = 0; m < MINE; ++m)
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int c = 16 * (wave + 4 * m) + 4 * kg + e;
      if (c < a.dim && col_there) state[(size_t)c * a.vdim] = mine[m][e];
    }
}

// A wave takes 16 positions of a chunk and a head; NT, NV: tiles of channels and of columns.
template <int C, int NT, int NV>
__global__ void __launch_bounds__(C * 4) delta_out_kernel(DeltaArgs a) {
  constexpr int NB = C / 16;
  constexpr int dp = 16 * NT;
  const int chunk = blockIdx.x, h = blockIdx.y, vt = a.vp / 16, row0 = chunk * C, rows = min(C, a.t - row0);
  const int lane = threadIdx.x & 63, I = __builtin_amdgcn_readfirstlane(threadIdx.x >> 6), j = lane & 15, kg = lane >> 4;
  if (16 * I >= rows) return;
  const size_t at = (size_t)chunk * a.heads + h;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  f32x4_t qf[NT], pf[NB], o[NV];
#pragma unroll
  for (int n = 0; n < NT; ++n) qf[n] = tile_of(a.qg + at * C * dp, I * NT + n, lane);
#pragma unroll
  for (int b = 0; b < NB; ++b) pf[b] = tile_of(a.p + at * C * C, I * NB + (b <= I ? b : 0), lane);
  float ss[4] = {0.f, 0.f, 0.f, 0.f};
  f32x4_t sf[2][NT], uf[2][NB];  // a column tile's state and U, on their way one tile ahead
  auto fetch = [&](int x, int v) {
    const size_t tile = at * vt + min(v, vt - 1);
#pragma unroll
    for (int n = 0; n < NT; ++n) sf[x][n] = tile_of(a.s0, tile * NT + n, lane);
#pragma unroll
    for (int b = 0; b < NB; ++b) uf[x][b] = tile_of(a.u, tile * NB + b, lane);
  };
  fetch(0, 0);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    o[v] = zero;
    if (v >= vt) continue;
    fetch((v + 1) & 1, v + 1);
    f32x4_t acc[4] = {zero, zero, zero, zero};
#pragma unroll
    for (int n = 0; n < NT; n += 4) {
      const f32x4_t x[4] = {qf[n], qf[n + 1], qf[n + 2], qf[n + 3]}, y[4] = {sf[v & 1][n], sf[v & 1][n + 1], sf[v & 1][n + 2], sf[v & 1][n + 3]};
      mfma16x16_each(x, y, acc);
    }
#pragma unroll
    for (int b = 0; b < NB; ++b)
      if (b <= I) acc[b] = mfma16x16(pf[b], uf[v & 1][b], acc[b]);
    o[v] = (acc[0] + acc[1]) + (acc[2] + acc[3]);  // columns past vdim are zeros
#pragma unroll
    for (int e = 0; e < 4; ++e) ss[e] += o[v][e] * o[v][e];
  }
  float inv[4];
#pragma unroll
  for (int e = 0; e < 4; ++e) inv[e] = 1.f / sqrtf(row_sum16(ss[e]) / (float)a.vdim + a.eps);
#pragma unroll
  for (int v = 0; v < NV; ++v) {
    const int c = 16 * v + j;
    if (c >= a.vdim) continue;
    const float w = a.norm[c];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int r = 16 * I + 4 * kg + e;
      if (r >= rows) continue;
      const float y = o[v][e] * inv[e] * w * sigmoid_f(a.z[(size_t)(row0 + r) * a.z_stride + (size_t)h * a.vdim + c]);
      const size_t to = (size_t)(row0 + r) * a.dst_stride + (size_t)h * a.vdim + c;
      if (a.dst_bf16) static_cast<uint16_t*>(a.dst)[to] = bf16_rne(y);
      else static_cast<float*>(a.dst)[to] = y;
    }
  }
}

// ---- one position -------------------------------------------------------------------------------------------------------------
// A workgroup takes a head and COLS columns of its state: it convolves those columns and the head's q and k (again in every workgroup:
// a few hundred channels), makes the head's decays, then 8 threads per column walk the state.  The ring's slot of this position is one
// that no tap of this position reads, so the rows go in while other workgroups still convolve.
constexpr int COLS = 32, GROUPS = 8, HELD = 16;
struct DeltaStepArgs {
  const float* qkv;  // this position's inputs of the convolution
  const float* b;
  const float* a_in;
  const float* z_in;
  const float* taps;
  float* ring;
  const float* a_log;
  const float* dt_bias;
  const void* w_a;
  const void* w_z;
  float* s;
  float* out;
  int before, slot;  // positions in front of this one, as far as the taps care; the ring's row of this position
  int n_taps, heads, kv_heads, dim, vdim, a_rank, z_rank, channels;
  bool fresh;
};

// TAPS > 0: that many, everything asked for at once.
template <int TAPS>
__device__ __forceinline__ float conv_one(const DeltaStepArgs& a, int c) {
  const float* taps = a.taps + (size_t)c * a.n_taps;
  if constexpr (TAPS > 0) {
    float w[TAPS], x[TAPS];
#pragma unroll
    for (int j = 0; j < TAPS; ++j) {
      const int row = a.slot + 1 + j;  // of the position TAPS - 1 - j back
      w[j] = taps[j];
      x[j] = j + 1 < TAPS ? a.ring[(size_t)(row < TAPS ? row : row - TAPS) * a.channels + c] : a.qkv[c];
    }
    float v = 0.f;
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
      v += TAPS - 1 - j <= a.before ? w[j] * x[j] : 0.f;
    return silu_f(v);
  }
  float v = 0.f;
  for (int j = 0; j + 1 < a.n_taps; ++j) {
    const int row = a.slot + 1 + j;
    if (a.n_taps - 1 - j <= a.before) v += taps[j] * a.ring[(size_t)(row < a.n_taps ? row : row - a.n_taps) * a.channels + c];
  }
  return silu_f(v + taps[a.n_taps - 1] * a.qkv[c]);
}

// Eight elements of a matrix row.
template <typename WT>
struct Piece8;
template <>
struct Piece8<uint16_t> {
  u32x4_t v;
  __device__ void load(const uint16_t* p) { v = *reinterpret_cast<const u32x4_t*>(p); }
  __device__ float dot(const float* x) const {
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) s += __uint_as_float(v[e] << 16) * x[2 * e] + __uint_as_float(v[e] & 0xffff0000u) * x[2 * e + 1];
    return s;
  }
};
template <>
struct Piece8<float> {
  f32x4_t u, v;
  __device__ void load(const float* p) { u = *reinterpret_cast<const f32x4_t*>(p), v = *reinterpret_cast<const f32x4_t*>(p + 4); }
  __device__ float dot(const float* x) const {
    float s = 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e) s += u[e] * x[e] + v[e] * x[4 + e];
    return s;
  }
};
// Eight lanes' part of a row's product with x from element k0 on: lane l takes every eighth piece of 8 (V8: rows of whole aligned pieces).
template <typename WT, bool V8>
__device__ __forceinline__ float row_part(const WT* row, const float* x, int k0, int n, int l) {
  float s = 0.f;
  for (int k = k0 + l * 8; k < n; k += 64) {
    if constexpr (V8) {
      Piece8<WT> w;
      w.load(row + k);
      s += w.dot(x + k);
    } else {
#pragma unroll
      for (int e = 0; e < 8; ++e)
        if (k + e < n) {
          if constexpr (sizeof(WT) == 2) s += bf16_to_f32(row[k + e]) * x[k + e];
          else s += row[k + e] * x[k + e];
        }
    }
  }
  return s;
}

constexpr int ROUNDS = 5, PIECES = 2;  // of the decays' and gates' rows, asked for before anything else: 160 rows of up to 128 elements
template <typename WT, bool V8, int TAPS>
__global__ void __launch_bounds__(256) delta_step_kernel(DeltaStepArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int d = a.dim, h = blockIdx.x, p0 = blockIdx.y * COLS, per = a.heads / a.kv_heads, g = h / per, gd = a.kv_heads * d;
  float* q = lds;
  float* k = q + d;
  float* decay = k + d;
  float* a_in = decay + d;
  float* z_in = a_in + a.a_rank;
  __shared__ float vs[COLS], part[GROUPS][COLS + 1], scale[2];
  const int tid = threadIdx.x, col = tid & (COLS - 1), grp = tid / COLS, p = p0 + col, lane = tid & 63, wave = tid >> 6;
  const int mine = min(COLS, a.vdim - p0), l8 = tid & 7, row8 = tid >> 3;
  // the decays' rows, then the gates'; eight lanes to a row
  auto row_of = [&](int r) {
    const bool gate = r >= d;
    return gate ? static_cast<const WT*>(a.w_z) + (size_t)(h * a.vdim + p0 + r - d) * a.z_rank : static_cast<const WT*>(a.w_a) + (size_t)(h * d + r) * a.a_rank;
  };
  Piece8<WT> pre[V8 ? ROUNDS : 1][PIECES];
  const int r_mine = row8 + 32 * l8;  // the row whose decay (or gate) this lane finishes
  const float bias = a.dt_bias[h * d + min(r_mine, d - 1)];
  if constexpr (V8) {
#pragma unroll
    for (int u = 0; u < ROUNDS; ++u) {
      const int r = min(row8 + 32 * u, d + mine - 1), n = r >= d ? a.z_rank : a.a_rank;
#pragma unroll
      for (int b = 0; b < PIECES; ++b) pre[u][b].load(row_of(r) + (b * 64 + l8 * 8 < n ? b * 64 + l8 * 8 : 0));
    }
  }
  float* S = a.s + (size_t)h * d * a.vdim + p;
  const bool there = p < a.vdim;
  float held[HELD];  // the first of the state's rows (lanes without a place in it load another's)
  {
    const float* Sl = a.s + (size_t)h * d * a.vdim + (there ? p : 0);
#pragma unroll
    for (int u = 0; u < HELD; ++u) held[u] = Sl[(size_t)min(grp + GROUPS * u, d - 1) * a.vdim];
  }
  __builtin_amdgcn_sched_barrier(0);
  float* slot = a.ring + (size_t)a.slot * a.channels;
  const bool first = h % per == 0 && blockIdx.y == 0;  // stores the key head's rows
  for (int i = tid; i < 2 * d; i += 256) {
    const int c = (i < d ? 0 : gd - d) + g * d + i;
    lds[i] = conv_one<TAPS>(a, c);
    if (first) slot[c] = a.qkv[c];
  }
  if (tid < COLS && there) {
    const int c = 2 * gd + h * a.vdim + p;
    vs[tid] = conv_one<TAPS>(a, c);
    slot[c] = a.qkv[c];
  }
  for (int i = tid; i < a.a_rank; i += 256) a_in[i] = a.a_in[i];
  for (int i = tid; i < a.z_rank; i += 256) z_in[i] = a.z_in[i];
  if (a.fresh) {  // nothing is known of the state's memory
#pragma unroll
    for (int u = 0; u < HELD; ++u) held[u] = 0.f;
  }
  const float neg = -expf(a.a_log[h]), beta = exact_sigmoid(a.b[h]);
  __syncthreads();
  if (wave < 2) {
    const float* row = wave ? k : q;
    float ss = 0.f;
    for (int c = lane; c < d; c += 64) ss += row[c] * row[c];
    ss = wave_sum(ss);
    if (lane == 0) scale[wave] = 1.f / sqrtf(ss + UNIT_EPS) * (wave ? 1.f : 1.f / sqrtf((float)d));
  }
  auto over8 = [&](float s) {
    s += __shfl_xor(s, 4, 64);
    s += __shfl_xor(s, 2, 64);
    return s + __shfl_xor(s, 1, 64);
  };
  auto finish = [&](int r, float s, float b) {
    if (r >= d + mine) return;
    if (r >= d) a.out[(size_t)a.heads * a.vdim + h * a.vdim + p0 + r - d] = s;
    else decay[r] = expf(neg * softplus_f(s + b));
  };
  if constexpr (V8) {
    float s_mine = 0.f;
#pragma unroll
    for (int u = 0; u < ROUNDS; ++u) {
      const int rr = min(row8 + 32 * u, d + mine - 1), n = rr >= d ? a.z_rank : a.a_rank;
      const float* x = rr >= d ? z_in : a_in;
      float s = 0.f;
#pragma unroll
      for (int b = 0; b < PIECES; ++b)
        if (b * 64 + l8 * 8 < n) s += pre[u][b].dot(x + b * 64 + l8 * 8);
      if (n > PIECES * 64) s += row_part<WT, V8>(row_of(rr), x, PIECES * 64, n, l8);
      s = over8(s);
      if (l8 == u) s_mine = s;
    }
    if (l8 < ROUNDS) finish(r_mine, s_mine, bias);
  }
  for (int r = row8 + (V8 ? 32 * ROUNDS : 0); r < d + mine; r += 32) {  // a row's eight lanes stay together
    const bool gate = r >= d;
    const float s = over8(row_part<WT, V8>(row_of(r), gate ? z_in : a_in, 0, gate ? a.z_rank : a.a_rank, l8));
    if (l8 == 0) finish(r, s, gate ? 0.f : a.dt_bias[h * d + r]);
  }
  __syncthreads();
  const float ks = scale[1], qs = scale[0];
  float sk = 0.f;
#pragma unroll
  for (int u = 0; u < HELD; ++u) {
    const int c = grp + GROUPS * u;
    if (c >= d) break;
    held[u] *= decay[c];
    sk += held[u] * (k[c] * ks);
  }
  if (there && !a.fresh)
    for (int c = grp + GROUPS * HELD; c < d; c += GROUPS) sk += S[(size_t)c * a.vdim] * decay[c] * (k[c] * ks);
  part[grp][col] = sk;
  __syncthreads();
  float all = 0.f;
#pragma unroll
  for (int i = 0; i < GROUPS; ++i) all += part[i][col];
  __syncthreads();
  const float u_new = there ? beta * (vs[col] - all) : 0.f;
  float o = 0.f;
#pragma unroll
  for (int u = 0; u < HELD; ++u) {
    const int c = grp + GROUPS * u;
    if (c >= d) break;
    const float v = held[u] + k[c] * ks * u_new;
    if (there) S[(size_t)c * a.vdim] = v;
    o += v * (q[c] * qs);
  }
  if (there)
    for (int c = grp + GROUPS * HELD; c < d; c += GROUPS) {
      float v = k[c] * ks * u_new;
      if (!a.fresh) v += S[(size_t)c * a.vdim] * decay[c];
      S[(size_t)c * a.vdim] = v;
      o += v * (q[c] * qs);
    }
  part[grp][col] = o;
  __syncthreads();
  if (grp == 0 && there) {
    float v = 0.f;
#pragma unroll
    for (int i = 0; i < GROUPS; ++i) v += part[i][col];
    a.out[h * a.vdim + p] = v;
  }
}

constexpr size_t SIZE_MAX_ = 256;

int check_delta(const ughip_device* dev, const ughip_delta* p, const char* what) {
  if (!dev || !p) return set_error(UGHIP_ERR_INVALID, "%s: null argument", what);
  if (p->heads == 0 || p->kv_heads == 0 || p->dim == 0 || p->vdim == 0 || p->heads % p->kv_heads != 0 || p->heads > 65535)
    return set_error(UGHIP_ERR_INVALID, "%s: %zu heads on %zu, of %zu and %zu elements", what, p->heads, p->kv_heads, p->dim, p->vdim);
  if (p->dim > SIZE_MAX_ || p->vdim > SIZE_MAX_) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: heads of %zu and %zu elements (built for up to %zu)", what, p->dim, p->vdim, SIZE_MAX_);
  if (int rc = check_buf(dev, p->a_log, p->heads, UGHIP_F32, what)) return rc;
  if (int rc = check_buf(dev, p->dt_bias, p->heads * p->dim, UGHIP_F32, what)) return rc;
  return check_buf(dev, p->s, p->heads * p->dim * p->vdim, UGHIP_F32, what);
}

template <int C, bool VEC>
int prepare(ughip_device* dev, const DeltaArgs& a) {
  const size_t bytes = prepare_lds_floats<C>(a.dp) * sizeof(float);
  static const hipError_t attr = hipFuncSetAttribute(reinterpret_cast<const void*>(delta_prepare_kernel<C, VEC>), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  UGHIP_HIPCHK(attr);
  delta_prepare_kernel<C, VEC><<<dim3((unsigned)a.chunks, (unsigned)a.heads), prepare_threads<C>(), bytes, dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
template <int C, int NT>
int scan_out(ughip_device* dev, const DeltaArgs& a) {
  delta_scan_kernel<C, NT><<<dim3((unsigned)a.heads, (unsigned)(a.vp / 16)), 256, 0, dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  const dim3 grid((unsigned)a.chunks, (unsigned)a.heads);
  if (a.vp <= 128) delta_out_kernel<C, NT, 8><<<grid, C * 4, 0, dev->stream>>>(a);
  else delta_out_kernel<C, NT, 16><<<grid, C * 4, 0, dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
template <int C>
int run_chunks(ughip_device* dev, const DeltaArgs& a, bool vec) {
  if (int rc = vec ? prepare<C, true>(dev, a) : prepare<C, false>(dev, a)) return rc;
  return a.dp == 64 ? scan_out<C, 4>(dev, a) : a.dp == 128 ? scan_out<C, 8>(dev, a) : a.dp == 192 ? scan_out<C, 12>(dev, a) : scan_out<C, 16>(dev, a);
}

}  // namespace

extern "C" int ughip_delta_rows(ughip_device* dev, const ughip_delta* p) {
  const char* what = "delta_rows";
  if (int rc = check_delta(dev, p, what)) return rc;
  const size_t H = p->heads, G = p->kv_heads, d = p->dim, vd = p->vdim;
  if (int rc = check_view(dev, p->qkv, p->t, 2 * G * d + H * vd, UGHIP_F32, what)) return rc;
  if (int rc = check_view(dev, p->b, p->t, H, UGHIP_F32, what)) return rc;
  if (int rc = check_view(dev, p->a, p->t, H * d, UGHIP_F32, what)) return rc;
  if (int rc = check_view(dev, p->z, p->t, H * vd, UGHIP_F32, what)) return rc;
  if (int rc = check_buf(dev, p->norm, vd, UGHIP_F32, what)) return rc;
  if (int rc = check_view(dev, p->dst, p->t, H * vd, -1, what)) return rc;
  const bool bf16 = p->dst.s->dtype == UGHIP_BF16;
  if (!bf16 && p->dst.s->dtype != UGHIP_F32) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: the result is F32 or BF16", what);
  if (p->t == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  const int dp = (int)((d + 63) / 64 * 64), vp = (int)((vd + 15) / 16 * 16);
  // chunks of 64 where a chunk's keys, queries and decays fit LDS, shorter ones for fewer positions
  const int C = p->t <= 16 ? 16 : p->t <= 32 || dp > 128 ? 32 : 64;
  const size_t c = C, per = c * dp * 3 + c * vp * 2 + c * c + dp + (size_t)dp * vp;  // floats per (chunk, head)
  // what lies between the launches stays within 1 GiB
  size_t span = (p->t + c - 1) / c, most = ((size_t)1 << 28) / (per * H);
  if (most < 1) most = 1;
  if (span > most) span = most;
  void* ws = nullptr;
  if (int rc = rows_scratch(dev, span * H * per * sizeof(float), &ws)) return rc;
  auto a16 = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  const bool vec = d % 4 == 0 && p->qkv.stride % 4 == 0 && p->a.stride % 4 == 0 && a16(view_ptr<float>(p->qkv)) && a16(view_ptr<float>(p->a));
  for (size_t r0 = 0; r0 < p->t; r0 += span * c) {
    const size_t rows = p->t - r0 < span * c ? p->t - r0 : span * c;
    DeltaArgs a{};
    a.qkv = view_ptr<float>(p->qkv) + r0 * p->qkv.stride, a.b = view_ptr<float>(p->b) + r0 * p->b.stride, a.a = view_ptr<float>(p->a) + r0 * p->a.stride;
    a.z = view_ptr<float>(p->z) + r0 * p->z.stride, a.a_log = buf_ptr<float>(p->a_log), a.dt_bias = buf_ptr<float>(p->dt_bias), a.norm = buf_ptr<float>(p->norm);
    a.s = static_cast<float*>(p->s->ptr), a.dst = static_cast<char*>(p->dst.s->ptr) + (p->dst.offset + r0 * p->dst.stride) * (bf16 ? 2 : 4);
    a.qkv_stride = p->qkv.stride, a.b_stride = p->b.stride, a.a_stride = p->a.stride, a.z_stride = p->z.stride, a.dst_stride = p->dst.stride;
    a.t = (int)rows, a.heads = (int)H, a.kv_heads = (int)G, a.dim = (int)d, a.vdim = (int)vd, a.dp = dp, a.vp = vp, a.chunks = (int)((rows + c - 1) / c);
    a.eps = p->eps, a.fresh = p->pos == 0 && r0 == 0, a.dst_bf16 = bf16;
    const size_t n = (size_t)a.chunks * H;
    float* w = static_cast<float*>(ws);
    auto take = [&](size_t floats) {
      float* at = w;
      w += n * floats;
      return at;
    };
    a.w = take(c * dp), a.v = take(c * vp), a.kd = take(c * dp), a.qg = take(c * dp), a.p = take(c * c), a.gam = take(dp), a.s0 = take((size_t)dp * vp), a.u = take(c * vp);
    if (int rc = C == 16 ? run_chunks<16>(dev, a, vec) : C == 32 ? run_chunks<32>(dev, a, vec) : run_chunks<64>(dev, a, vec)) return rc;
  }
  return UGHIP_OK;
}

extern "C" int ughip_delta_step(ughip_device* dev, const ughip_delta* p) {
  const char* what = "delta_step";
  if (int rc = check_delta(dev, p, what)) return rc;
  const size_t H = p->heads, G = p->kv_heads, d = p->dim, vd = p->vdim, ch = 2 * G * d + H * vd;
  if (p->n_taps == 0 || p->n_taps > 1024) return set_error(UGHIP_ERR_INVALID, "%s: %zu taps", what, p->n_taps);
  if (p->a_rank == 0 || p->z_rank == 0 || p->a_rank > 4096 || p->z_rank > 4096) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: ranks %zu and %zu", what, p->a_rank, p->z_rank);
  auto row = [&](size_t off, size_t n) { return check_view(dev, ughip_view{const_cast<ughip_slice*>(p->p), off, n}, 1, n, UGHIP_F32, what); };
  if (int rc = row(p->qkv_offset, ch)) return rc;
  if (int rc = row(p->b_offset, H)) return rc;
  if (int rc = row(p->a_offset, p->a_rank)) return rc;
  if (int rc = row(p->z_offset, p->z_rank)) return rc;
  if (int rc = check_buf(dev, p->taps, ch * p->n_taps, UGHIP_F32, what)) return rc;
  if (int rc = check_buf(dev, p->ring, ch * p->n_taps, UGHIP_F32, what)) return rc;
  if (!p->w_a || !p->w_z || p->w_a->dtype != p->w_z->dtype || (p->w_a->dtype != UGHIP_F32 && p->w_a->dtype != UGHIP_BF16))
    return set_error(UGHIP_ERR_UNSUPPORTED, "%s: matrices are both F32 or both BF16", what);
  if (int rc = check_buf(dev, p->w_a, H * d * p->a_rank, -1, what)) return rc;
  if (int rc = check_buf(dev, p->w_z, H * vd * p->z_rank, -1, what)) return rc;
  if (int rc = check_view(dev, ughip_view{p->out, p->dst_offset, 2 * H * vd}, 1, 2 * H * vd, UGHIP_F32, what)) return rc;
  if (p->out == p->p) return set_error(UGHIP_ERR_INVALID, "%s: out aliases p", what);
  if (int rc = device_activate(dev)) return rc;
  const float* in = buf_ptr<float>(p->p);
  DeltaStepArgs a{in + p->qkv_offset, in + p->b_offset, in + p->a_offset, in + p->z_offset, buf_ptr<float>(p->taps), static_cast<float*>(p->ring->ptr), buf_ptr<float>(p->a_log),
                  buf_ptr<float>(p->dt_bias), p->w_a->ptr, p->w_z->ptr, static_cast<float*>(p->s->ptr), static_cast<float*>(p->out->ptr) + p->dst_offset,
                  (int)(p->pos < p->n_taps ? p->pos : p->n_taps), (int)(p->pos % p->n_taps), (int)p->n_taps, (int)H, (int)G, (int)d, (int)vd, (int)p->a_rank, (int)p->z_rank, (int)ch, p->pos == 0};
  const bool v8 = p->a_rank % 8 == 0 && p->z_rank % 8 == 0 && (reinterpret_cast<uintptr_t>(a.w_a) & 15) == 0 && (reinterpret_cast<uintptr_t>(a.w_z) & 15) == 0;
  const size_t lds = (3 * d + p->a_rank + p->z_rank) * sizeof(float);
  auto go = [&](auto kernel) { kernel<<<dim3((unsigned)H, (unsigned)((vd + COLS - 1) / COLS)), 256, lds, dev->stream>>>(a); };
  const bool bf = p->w_a->dtype == UGHIP_BF16;
  auto taps = [&](auto type, auto whole) {
    using WT = decltype(type);
    constexpr bool V8 = decltype(whole)::value;
    p->n_taps == 4 ? go(delta_step_kernel<WT, V8, 4>) : p->n_taps == 3 ? go(delta_step_kernel<WT, V8, 3>) : p->n_taps == 2 ? go(delta_step_kernel<WT, V8, 2>) : go(delta_step_kernel<WT, V8, 0>);
  };
  if (bf) v8 ? taps(uint16_t(), std::true_type{}) : taps(uint16_t(), std::false_type{});
  else v8 ? taps(float(), std::true_type{}) : taps(float(), std::false_type{});
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
