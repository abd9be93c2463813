// A state-space recurrence (Mamba-2's) behind a causal convolution (ughip_layers.h).
//
//   S_t = exp(a_t) S_{t-1} + d_t B_t x_t^T,   y_t = S_t^T C_t + skip x_t,   a_t = -exp(a_log) d_t, d_t = softplus(dt_t + bias)
//
// Several positions run in chunks of Q.  With A_i = a_1 + .. + a_i inside a chunk:
//   ssm_chunk_decays  d_i and A_i
//   ssm_chunk_state   what a chunk adds to the state: sum_j B_j (exp(A_Q - A_j) d_j x_j)^T
//   ssm_chunk_scan    the state in front of every chunk, S <- exp(A_Q) S + that, in place              (elementwise, chunks in order)
//   ssm_chunk_out     y_i = sum_{j <= i} exp(A_i - A_j) d_j (C_i . B_j) x_j + exp(A_i) S^T C_i + skip x_i
// Every exponent is <= 0.  A workgroup takes a chunk and some heads of one group: B, C and the products C_i . B_j are the group's
// and are made once, then the heads follow one after the other, the next head's x (and state) on their way to registers while
// this one is multiplied.  The products are v_mfma_f32_16x16x4_f32 on f32 tiles in LDS (lane l: row or column l % 16, k = l / 16;
// result element e: row 4 (l / 16) + e, column l % 16), four independent column tiles at a time.
#include <hip/hip_runtime.h>

#include "layers.h"

using namespace ughip;

namespace {

struct SsmArgs {
  const float* xbc;
  const float* dt;
  const float* dt_bias;
  const float* a_log;
  const float* skip;
  float* s;        // [heads, state, vdim]
  float* chunk_s;  // [chunks, heads, state, vdim]
  float* cum;      // [chunks, heads, 64]: A_i, and
  float* step;     // d_i (0 past the last row, where A_i stays)
  float* dst;
  size_t xbc_stride, dt_stride, dst_stride;
  int t, heads, vdim, groups, state, q, chunks;
  bool fresh;
};

// A thread takes four channels (V) of ROWS_CONV rows, the taps' rows sliding through registers; any channel count otherwise.
constexpr int ROWS_CONV = 8;
template <int TAPS>
__global__ void __launch_bounds__(256) conv_silu_rows4_kernel(const float* __restrict__ x, size_t x_stride, const float* __restrict__ taps, const float* __restrict__ bias,
                                                              const float* __restrict__ ring, long long pos, int t, int channels, float* __restrict__ dst, size_t dst_stride) {
  const int c = (blockIdx.x * 256 + threadIdx.x) * 4, i0 = blockIdx.y * ROWS_CONV;
  if (c >= channels) return;
  auto row = [&](int r) -> f32x4_t {
    if (r >= 0) return r < t ? *reinterpret_cast<const f32x4_t*>(x + (size_t)r * x_stride + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (pos + r >= 0) return *reinterpret_cast<const f32x4_t*>(ring + (size_t)((pos + r) % TAPS) * channels + c);
    return f32x4_t{0.f, 0.f, 0.f, 0.f};
  };
  float w[4][TAPS];
#pragma unroll
  for (int e = 0; e < 4; ++e)
#pragma unroll
    for (int j = 0; j < TAPS; ++j) w[e][j] = taps[(size_t)(c + e) * TAPS + j];
  const f32x4_t b = bias ? *reinterpret_cast<const f32x4_t*>(bias + c) : f32x4_t{0.f, 0.f, 0.f, 0.f};
  f32x4_t in[ROWS_CONV + TAPS - 1];
#pragma unroll
  for (int j = 0; j < ROWS_CONV + TAPS - 1; ++j) in[j] = row(i0 - (TAPS - 1) + j);
#pragma unroll
  for (int i = 0; i < ROWS_CONV; ++i) {
    if (i0 + i >= t) break;
    f32x4_t v = b;
#pragma unroll
    for (int j = 0; j < TAPS; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e) v[e] += w[e][j] * in[i + j][e];
#pragma unroll
    for (int e = 0; e < 4; ++e) v[e] = silu_f(v[e]);
    *reinterpret_cast<f32x4_t*>(dst + (size_t)(i0 + i) * dst_stride + c) = v;
  }
}

__global__ void __launch_bounds__(256) conv_silu_rows_kernel(const float* __restrict__ x, size_t x_stride, const float* __restrict__ taps, const float* __restrict__ bias,
                                                             int n_taps, const float* __restrict__ ring, long long pos, int t, int channels, float* __restrict__ dst,
                                                             size_t dst_stride) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= channels) return;
  for (int i = blockIdx.y; i < t; i += gridDim.y) {
    float v = bias ? bias[c] : 0.f;
    for (int j = 0; j < n_taps; ++j) {
      const int r = i - (n_taps - 1) + j;
      float in = 0.f;
      if (r >= 0) in = x[(size_t)r * x_stride + c];
      else if (pos + r >= 0) in = ring[(size_t)((pos + r) % n_taps) * channels + c];
      v += taps[(size_t)c * n_taps + j] * in;
    }
    dst[(size_t)i * dst_stride + c] = silu_f(v);
  }
}

__global__ void __launch_bounds__(256) conv_ring_store_kernel(const float* __restrict__ x, size_t x_stride, int n_taps, float* __restrict__ ring, long long pos, int t,
                                                              int channels) {
  const int c = blockIdx.x * 256 + threadIdx.x;
  const int i = t - 1 - (int)blockIdx.y;
  if (c >= channels || i < 0) return;
  ring[(size_t)((pos + i) % n_taps) * channels + c] = x[(size_t)i * x_stride + c];
}

// One wave per chunk and head (q <= 64).
__global__ void __launch_bounds__(256) ssm_chunk_decays_kernel(SsmArgs a) {
  const int i = threadIdx.x & 63, h = blockIdx.y * 4 + (threadIdx.x >> 6), row0 = blockIdx.x * a.q;
  if (h >= a.heads) return;
  float dv = 0.f;
  if (i < a.q && row0 + i < a.t) dv = softplus_f(a.dt[(size_t)(row0 + i) * a.dt_stride + h] + a.dt_bias[h]);
  float s = -expf(a.a_log[h]) * dv;
  for (int k = 1; k < 64; k <<= 1) {
    const float o = __shfl_up(s, k, 64);
    if (i >= k) s += o;
  }
  const size_t at = ((size_t)blockIdx.x * a.heads + h) * 64 + i;
  a.cum[at] = s, a.step[at] = dv;
}

__device__ __forceinline__ f32x4_t mfma16(float x, float y, f32x4_t acc) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, acc, 0, 0, 0); }

constexpr int PB = 64, PS = PB + 4;  // columns of vdim at a time, and the stride of their rows in LDS

__device__ __host__ inline int pad16(int v) { return (v + 15) & ~15; }
// row stride of LDS tiles of `state` columns: a multiple of 16 plus 4, so that 16 rows x 4 neighbours spread over the banks
__device__ __host__ inline int row_n(int state) { return pad16(state) + 4; }

// `rows` x `cols` (cols <= 4 * width4) of a row-major matrix, zeros outside, through registers: N4 runs of four per thread.
template <int N4, bool VEC>
struct TileRegs {
  f32x4_t v[N4];
  int n_rows, n_cols;
  __device__ void load(const float* src, size_t stride, int rows, int cols, int width4, int total) {
    n_rows = rows, n_cols = cols;
#pragma unroll
    for (int u = 0; u < N4; ++u) {
      const int e = threadIdx.x + u * 256, r = e / width4, c = (e - r * width4) * 4;
      const bool ok = e < total && r < rows;
      const float* p = src + (size_t)(ok ? r : 0) * stride;
      if (VEC) {  // every lane loads (store() drops what is not there): with branches around loads the compiler waits for all of them at once
        v[u] = *reinterpret_cast<const f32x4_t*>(p + (c < cols ? c : 0));
      } else {
        v[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (ok && c + i < cols) v[u][i] = p[c + i];
      }
    }
  }
  // scale (may be null): row r times scale[r]
  __device__ void store(float* lds, int ld, int width4, int total, const float* scale = nullptr) const {
#pragma unroll
    for (int u = 0; u < N4; ++u) {
      const int e = threadIdx.x + u * 256, r = e / width4, c = (e - r * width4) * 4;
      if (e >= total) continue;
      f32x4_t w = v[u];
      if (VEC && (r >= n_rows || c >= n_cols)) w = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (scale) w *= scale[r];
      *reinterpret_cast<f32x4_t*>(lds + r * ld + c) = w;
    }
  }
};
template <bool VEC>
__device__ __forceinline__ void tile_to_lds(float* lds, int ld, const float* src, size_t stride, int rows, int cols, int width4, int total) {
  for (int base = 0; base < total; base += 256 * 4) {  // four loads per thread on their way at a time
    f32x4_t v[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int e = base + threadIdx.x + u * 256, r = e / width4, c = (e - r * width4) * 4;
      v[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      if (e >= total || r >= rows) continue;
      const float* p = src + (size_t)r * stride + c;
      if (VEC) {
        if (c < cols) v[u] = *reinterpret_cast<const f32x4_t*>(p);
      } else {
#pragma unroll
        for (int i = 0; i < 4; ++i)
          if (c + i < cols) v[u][i] = p[i];
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u) {
      const int e = base + threadIdx.x + u * 256, r = e / width4, c = (e - r * width4) * 4;
      if (e < total) *reinterpret_cast<f32x4_t*>(lds + r * ld + c) = v[u];
    }
  }
}

// What a workgroup walks: heads h0 .. h0 + n of a group, each in blocks of PB columns.
struct HeadWalk {
  int g, h0, items, blocks;
  __device__ HeadWalk(const SsmArgs& a) {
    const int per = a.heads / a.groups, each = (per + (int)gridDim.z - 1) / (int)gridDim.z;
    g = blockIdx.y;
    blocks = (a.vdim + PB - 1) / PB;
    const int first = (int)blockIdx.z * each, last = min(per, first + each);
    h0 = g * per + first;
    items = max(0, last - first) * blocks;
  }
  __device__ int head(int i) const { return h0 + i / blocks; }
  __device__ int col(int i) const { return i % blocks * PB; }
};

template <bool VEC>
__global__ void __launch_bounds__(256) ssm_chunk_state_kernel(SsmArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int q = a.q, chunk = blockIdx.x, row0 = chunk * q, rows = min(q, a.t - row0), N = a.state, ns = row_n(N), np = pad16(N), inner = a.heads * a.vdim;
  const HeadWalk hw(a);
  float* wgt = lds;
  float* Bs = lds + 64;       // [q][ns]
  float* Xs = Bs + q * ns;    // [q][PS]
  const float* xbc0 = a.xbc + (size_t)row0 * a.xbc_stride;
  tile_to_lds<VEC>(Bs, ns, xbc0 + inner + (size_t)hw.g * N, a.xbc_stride, rows, N, np / 4, q * np / 4);
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, kg = lane >> 4, tn = np / 16, xt = q * PB / 4;
  TileRegs<4, VEC> x;
  float weight = 0.f;  // of row `lane` (first wave)
  auto fetch = [&](int i) {
    x.load(xbc0 + (size_t)hw.head(i) * a.vdim + hw.col(i), a.xbc_stride, rows, min(PB, a.vdim - hw.col(i)), PB / 4, xt);
    if (wave == 0) {
      const size_t at = ((size_t)chunk * a.heads + hw.head(i)) * 64;
      weight = a.step[at + lane] * expf(a.cum[at + 63] - a.cum[at + lane]);
    }
  };
  if (hw.items) fetch(0);
  for (int it = 0; it < hw.items; ++it) {
    const int h = hw.head(it), p0 = hw.col(it), pw = min(PB, a.vdim - p0);
    __syncthreads();
    if (wave == 0) wgt[lane] = weight;
    __syncthreads();
    x.store(Xs, PS, PB / 4, xt, wgt);
    if (it + 1 < hw.items) fetch(it + 1);
    __syncthreads();
    float* out = a.chunk_s + ((size_t)chunk * a.heads + h) * N * a.vdim + p0;
    for (int n_tile = wave * 2; n_tile < tn; n_tile += 8) {  // two row tiles by four column tiles at a time
      const int n0 = n_tile * 16, n1 = min(n_tile + 1, tn - 1) * 16;
      f32x4_t acc[2][4];
#pragma unroll
      for (int u = 0; u < 4; ++u) acc[0][u] = acc[1][u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
      for (int k = kg; k < q; k += 4) {
        const float b0 = Bs[k * ns + n0 + j], b1 = Bs[k * ns + n1 + j];
#pragma unroll
        for (int u = 0; u < 4; ++u) {
          const float xv = Xs[k * PS + u * 16 + j];
          acc[0][u] = mfma16(b0, xv, acc[0][u]);
          acc[1][u] = mfma16(b1, xv, acc[1][u]);
        }
      }
#pragma unroll
      for (int v = 0; v < 2; ++v) {
        if (v == 1 && n_tile + 1 >= tn) break;
#pragma unroll
        for (int u = 0; u < 4; ++u)
#pragma unroll
          for (int e = 0; e < 4; ++e) {
            const int n = (v ? n1 : n0) + 4 * kg + e;
            if (n < N && u * 16 + j < pw) out[(size_t)n * a.vdim + u * 16 + j] = acc[v][u][e];
          }
      }
    }
  }
}

__global__ void __launch_bounds__(256) ssm_chunk_scan_kernel(SsmArgs a) {
  const int h = blockIdx.y;
  const size_t per = (size_t)a.state * a.vdim, e = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (e >= per) return;
  float s = a.fresh ? 0.f : a.s[h * per + e];
  for (int c = 0; c < a.chunks; ++c) {
    float* at = a.chunk_s + ((size_t)c * a.heads + h) * per + e;
    const float add = *at;
    *at = s;
    s = expf(a.cum[((size_t)c * a.heads + h) * 64 + 63]) * s + add;
  }
  a.s[h * per + e] = s;
}

template <bool VEC>
__global__ void __launch_bounds__(256) ssm_chunk_out_kernel(SsmArgs a) {
  extern __shared__ __attribute__((aligned(16))) float lds[];
  const int q = a.q, chunk = blockIdx.x, row0 = chunk * q, rows = min(q, a.t - row0), N = a.state, ns = row_n(N), np = pad16(N), gs = q + 4, inner = a.heads * a.vdim;
  const HeadWalk hw(a);
  float* cum = lds;
  float* d = lds + 64;
  float* Cs = lds + 128;      // [q][ns]
  float* Gs = Cs + q * ns;    // [q][gs]: C_i . B_j
  float* Bs = Gs + q * gs;    // [q][ns], then
  float* Xs = Bs;             // [q][PS]
  float* Ss = Xs + q * PS;    // [np][PS]
  const float* xbc0 = a.xbc + (size_t)row0 * a.xbc_stride;
  const float *b_src = xbc0 + inner + (size_t)hw.g * N, *c_src = xbc0 + inner + (size_t)(a.groups + hw.g) * N;
  const int bt = q * np / 4;
  if (bt <= 8 * 256) {
    TileRegs<8, VEC> b, c;  // both on their way at once
    b.load(b_src, a.xbc_stride, rows, N, np / 4, bt);
    c.load(c_src, a.xbc_stride, rows, N, np / 4, bt);
    b.store(Bs, ns, np / 4, bt);
    c.store(Cs, ns, np / 4, bt);
  } else {
    tile_to_lds<VEC>(Bs, ns, b_src, a.xbc_stride, rows, N, np / 4, bt);
    tile_to_lds<VEC>(Cs, ns, c_src, a.xbc_stride, rows, N, np / 4, bt);
  }
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, kg = lane >> 4, tq = q / 16, i0 = wave * 16, xt = q * PB / 4, st = np * PB / 4;
  TileRegs<4, VEC> x;
  TileRegs<8, VEC> s;
  float decays = 0.f;  // A of row `lane` (first wave), d of it (second)
  auto fetch = [&](int i) {
    const int pw = min(PB, a.vdim - hw.col(i));
    if (wave < 2) decays = (wave ? a.step : a.cum)[((size_t)chunk * a.heads + hw.head(i)) * 64 + lane];
    x.load(xbc0 + (size_t)hw.head(i) * a.vdim + hw.col(i), a.xbc_stride, rows, pw, PB / 4, xt);
    s.load(a.chunk_s + ((size_t)chunk * a.heads + hw.head(i)) * N * a.vdim + hw.col(i), a.vdim, N, pw, PB / 4, st);
  };
  if (hw.items) fetch(0);
  __syncthreads();
  if (wave < tq) {
    f32x4_t acc[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) acc[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 2
    for (int k = 4 * kg; k < np; k += 16) {  // k four elements per lane at a time: 16-byte reads
      const f32x4_t c = *reinterpret_cast<const f32x4_t*>(Cs + (i0 + j) * ns + k);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        if (u > wave) break;  // columns past the row tile are not used
        const f32x4_t b = *reinterpret_cast<const f32x4_t*>(Bs + (u * 16 + j) * ns + k);
        acc[u] = mfma16(c.x, b.x, acc[u]);
        acc[u] = mfma16(c.y, b.y, acc[u]);
        acc[u] = mfma16(c.z, b.z, acc[u]);
        acc[u] = mfma16(c.w, b.w, acc[u]);
      }
    }
#pragma unroll
    for (int u = 0; u < 4; ++u)
      if (u < tq)
#pragma unroll
        for (int e = 0; e < 4; ++e) Gs[(i0 + 4 * kg + e) * gs + u * 16 + j] = acc[u][e];
  }
  for (int it = 0; it < hw.items; ++it) {
    const int h = hw.head(it), p0 = hw.col(it), pw = min(PB, a.vdim - p0);
    __syncthreads();
    x.store(Xs, PS, PB / 4, xt);
    s.store(Ss, PS, PB / 4, st);
    for (int base = 2048; base < st; base += 2048) {  // states of more than 128 rows: the rest without prefetch
      const int r0 = base / (PB / 4);
      tile_to_lds<VEC>(Ss + r0 * PS, PS, a.chunk_s + (((size_t)chunk * a.heads + h) * N + r0) * a.vdim + p0, a.vdim, N - r0, pw, PB / 4, min(2048, st - base));
    }
    if (wave < 2) (wave ? d : cum)[lane] = decays;
    __syncthreads();
    if (it + 1 < hw.items) fetch(it + 1);
    if (wave >= tq) continue;  // q < 64: the waves without rows only move data
    f32x4_t in_chunk[4], from_s[4];
#pragma unroll
    for (int u = 0; u < 4; ++u) in_chunk[u] = from_s[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    const float ci = cum[i0 + j];
#pragma unroll 4
    for (int k = kg; k < i0 + 16; k += 4) {
      const float m = k <= i0 + j ? Gs[(i0 + j) * gs + k] * expf(ci - cum[k]) * d[k] : 0.f;
#pragma unroll
      for (int u = 0; u < 4; ++u) in_chunk[u] = mfma16(m, Xs[k * PS + u * 16 + j], in_chunk[u]);
    }
#pragma unroll 2
    for (int k = 4 * kg; k < np; k += 16) {
      const f32x4_t c = *reinterpret_cast<const f32x4_t*>(Cs + (i0 + j) * ns + k);
#pragma unroll
      for (int u = 0; u < 4; ++u) {
        from_s[u] = mfma16(c.x, Ss[k * PS + u * 16 + j], from_s[u]);
        from_s[u] = mfma16(c.y, Ss[(k + 1) * PS + u * 16 + j], from_s[u]);
        from_s[u] = mfma16(c.z, Ss[(k + 2) * PS + u * 16 + j], from_s[u]);
        from_s[u] = mfma16(c.w, Ss[(k + 3) * PS + u * 16 + j], from_s[u]);
      }
    }
    const float skip = a.skip[h];
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = i0 + 4 * kg + e;
      const float decay = expf(cum[i]);
      if (i >= rows) continue;
#pragma unroll
      for (int u = 0; u < 4; ++u)
        if (u * 16 + j < pw)
          a.dst[(size_t)(row0 + i) * a.dst_stride + (size_t)h * a.vdim + p0 + u * 16 + j] = in_chunk[u][e] + decay * from_s[u][e] + skip * Xs[i * PS + u * 16 + j];
    }
  }
}

// One position in one launch.  A workgroup takes a head and 16 of its columns: it convolves those columns and the head's B and
// C rows (again in every workgroup: a few hundred channels), then 16 threads per column walk the state.  The ring's slot of this
// position is one no tap of this position reads, so the rows go in while other workgroups still convolve.
constexpr int STEP_COLS = 16, STEP_ROWS = 8;
struct SsmStepArgs {
  const float* xbc;  // this position's inputs of the convolution
  const float* dt;
  const float* taps;
  const float* conv_bias;
  float* ring;
  const float* dt_bias;
  const float* a_log;
  const float* skip;
  float* s;
  float* dst;
  long long pos;
  int n_taps, heads, vdim, groups, state, channels;
};

__device__ __forceinline__ float conv_one(const SsmStepArgs& a, int c) {
  float v = a.conv_bias ? a.conv_bias[c] : 0.f;
  for (int j = 0; j + 1 < a.n_taps; ++j) {
    const long long p = a.pos - (a.n_taps - 1) + j;
    if (p >= 0) v += a.taps[(size_t)c * a.n_taps + j] * a.ring[(size_t)(p % a.n_taps) * a.channels + c];
  }
  return silu_f(v + a.taps[(size_t)c * a.n_taps + a.n_taps - 1] * a.xbc[c]);
}

__global__ void __launch_bounds__(256) ssm_step_kernel(SsmStepArgs a) {
  extern __shared__ float lds[];
  float* B = lds;
  float* C = lds + a.state;
  __shared__ float xs[STEP_COLS], part[16][STEP_COLS + 1];
  const int h = blockIdx.x, p0 = blockIdx.y * STEP_COLS, inner = a.heads * a.vdim, N = a.state, per = a.heads / a.groups, g = h / per;
  const bool first = h % per == 0 && blockIdx.y == 0;  // stores the group's B and C rows
  float* slot = a.ring + (size_t)(a.pos % a.n_taps) * a.channels;
  const int col = threadIdx.x & 15, ng = threadIdx.x >> 4, p = p0 + col;
  float* S = a.s + (size_t)h * N * a.vdim + p;
  float held[STEP_ROWS];  // the first of the state's rows, asked for before anything else
#pragma unroll
  for (int u = 0; u < STEP_ROWS; ++u) held[u] = a.pos && p < a.vdim && ng + 16 * u < N ? S[(size_t)(ng + 16 * u) * a.vdim] : 0.f;
  for (int i = threadIdx.x; i < 2 * N; i += 256) {
    const int c = inner + (i < N ? 0 : a.groups * N) + g * N + (i < N ? i : i - N);
    lds[i] = conv_one(a, c);
    if (first) slot[c] = a.xbc[c];
  }
  if (threadIdx.x < STEP_COLS && p0 + (int)threadIdx.x < a.vdim) {
    const int c = h * a.vdim + p0 + threadIdx.x;
    xs[threadIdx.x] = conv_one(a, c);
    slot[c] = a.xbc[c];
  }
  __syncthreads();
  const float d = softplus_f(a.dt[h] + a.dt_bias[h]), keep = expf(-expf(a.a_log[h]) * d);
  float y = 0.f;
  if (p < a.vdim) {
    const float dx = d * xs[col];
#pragma unroll
    for (int u = 0; u < STEP_ROWS; ++u) {
      const int n = ng + 16 * u;
      if (n >= N) break;
      const float v = keep * held[u] + dx * B[n];
      S[(size_t)n * a.vdim] = v;
      y += v * C[n];
    }
    for (int n = ng + 16 * STEP_ROWS; n < N; n += 16) {
      float v = dx * B[n];
      if (a.pos) v += keep * S[(size_t)n * a.vdim];
      S[(size_t)n * a.vdim] = v;
      y += v * C[n];
    }
  }
  part[ng][col] = y;
  __syncthreads();
  if (ng == 0 && p < a.vdim) {
    float v = 0.f;
#pragma unroll
    for (int i = 0; i < 16; ++i) v += part[i][col];
    a.dst[h * a.vdim + p] = v + a.skip[h] * xs[col];
  }
}

size_t state_lds_bytes(int q, int state) { return (size_t)(64 + q * row_n(state) + q * PS) * sizeof(float); }
size_t out_lds_bytes(int q, int state) {
  const size_t b = (size_t)q * row_n(state), xs = (size_t)(q + pad16(state)) * PS;
  return (128 + (size_t)q * row_n(state) + (size_t)q * (q + 4) + (b > xs ? b : xs)) * sizeof(float);
}

}  // namespace

extern "C" int ughip_conv_silu_rows(ughip_device* dev, ughip_view x, const ughip_slice* taps, const ughip_slice* bias, size_t n_taps, const ughip_slice* ring, size_t pos,
                                    size_t t, size_t channels, ughip_view dst) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "conv_silu_rows: null device");
  if (n_taps == 0 || n_taps > 1024) return set_error(UGHIP_ERR_INVALID, "conv_silu_rows: %zu taps", n_taps);
  if (int rc = check_view(dev, x, t, channels, UGHIP_F32, "conv_silu_rows x")) return rc;
  if (int rc = check_buf(dev, taps, channels * n_taps, UGHIP_F32, "conv_silu_rows taps")) return rc;
  if (bias)
    if (int rc = check_buf(dev, bias, channels, UGHIP_F32, "conv_silu_rows bias")) return rc;
  if (int rc = check_buf(dev, ring, n_taps * channels, UGHIP_F32, "conv_silu_rows ring")) return rc;
  if (int rc = check_view(dev, dst, t, channels, UGHIP_F32, "conv_silu_rows dst")) return rc;
  if (t == 0 || channels == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  auto a16 = [](const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; };
  if (n_taps >= 2 && n_taps <= 4 && channels % 4 == 0 && x.stride % 4 == 0 && dst.stride % 4 == 0 && a16(view_ptr<float>(x)) && a16(view_ptr<float>(dst)) && t / ROWS_CONV < 65535) {
    const dim3 g4((unsigned)((channels / 4 + 255) / 256), (unsigned)((t + ROWS_CONV - 1) / ROWS_CONV));
    auto go = [&](auto kernel) {
      kernel<<<g4, 256, 0, dev->stream>>>(view_ptr<float>(x), x.stride, buf_ptr<float>(taps), buf_ptr<float>(bias), buf_ptr<float>(ring), (long long)pos, (int)t, (int)channels,
                                          view_ptr<float>(dst), dst.stride);
    };
    n_taps == 4 ? go(conv_silu_rows4_kernel<4>) : n_taps == 3 ? go(conv_silu_rows4_kernel<3>) : go(conv_silu_rows4_kernel<2>);
    UGHIP_HIPCHK(hipGetLastError());
    return UGHIP_OK;
  }
  const dim3 grid((unsigned)((channels + 255) / 256), (unsigned)(t < 16384 ? t : 16384));
  conv_silu_rows_kernel<<<grid, 256, 0, dev->stream>>>(view_ptr<float>(x), x.stride, buf_ptr<float>(taps), buf_ptr<float>(bias), (int)n_taps, buf_ptr<float>(ring),
                                                       (long long)pos, (int)t, (int)channels, view_ptr<float>(dst), dst.stride);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_conv_ring_store(ughip_device* dev, ughip_view x, size_t n_taps, ughip_slice* ring, size_t pos, size_t t, size_t channels) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "conv_ring_store: null device");
  if (n_taps == 0 || n_taps > 1024) return set_error(UGHIP_ERR_INVALID, "conv_ring_store: %zu taps", n_taps);
  if (int rc = check_view(dev, x, t, channels, UGHIP_F32, "conv_ring_store x")) return rc;
  if (int rc = check_buf(dev, ring, n_taps * channels, UGHIP_F32, "conv_ring_store ring")) return rc;
  if (t == 0 || channels == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  const dim3 grid((unsigned)((channels + 255) / 256), (unsigned)(t < n_taps ? t : n_taps));
  conv_ring_store_kernel<<<grid, 256, 0, dev->stream>>>(view_ptr<float>(x), x.stride, (int)n_taps, static_cast<float*>(ring->ptr), (long long)pos, (int)t, (int)channels);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_ssm_rows(ughip_device* dev, ughip_view xbc, ughip_view dt, const ughip_slice* dt_bias, const ughip_slice* a_log, const ughip_slice* skip, ughip_slice* s,
                              size_t pos, size_t t, size_t heads, size_t vdim, size_t groups, size_t state, ughip_view dst) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "ssm_rows: null device");
  if (heads == 0 || vdim == 0 || groups == 0 || state == 0 || heads % groups != 0 || heads > 65535 || vdim > 65535 || state > 65535)
    return set_error(UGHIP_ERR_INVALID, "ssm_rows: heads %zu, vdim %zu, groups %zu, state %zu", heads, vdim, groups, state);
  if (int rc = check_view(dev, xbc, t, heads * vdim + 2 * groups * state, UGHIP_F32, "ssm_rows xbc")) return rc;
  if (int rc = check_view(dev, dt, t, heads, UGHIP_F32, "ssm_rows dt")) return rc;
  for (const ughip_slice* v : {dt_bias, a_log, skip})
    if (int rc = check_buf(dev, v, heads, UGHIP_F32, "ssm_rows per-head vector")) return rc;
  if (int rc = check_buf(dev, s, heads * state * vdim, UGHIP_F32, "ssm_rows state")) return rc;
  if (int rc = check_view(dev, dst, t, heads * vdim, UGHIP_F32, "ssm_rows dst")) return rc;
  if (t == 0) return UGHIP_OK;
  int q = 64;
  while (q > 16 && (out_lds_bytes(q, (int)state) > 160 * 1024 || (size_t)(q / 2) >= t)) q /= 2;
  if (out_lds_bytes(q, (int)state) > 160 * 1024 || state_lds_bytes(q, (int)state) > 160 * 1024) return set_error(UGHIP_ERR_UNSUPPORTED, "ssm_rows: a state of %zu rows does not fit LDS", state);
  if (int rc = device_activate(dev)) return rc;
  const size_t chunks = (t + q - 1) / q, elems = state * vdim, n_decay = chunks * heads * 64;
  void* ws = nullptr;
  if (int rc = rows_scratch(dev, (2 * n_decay + chunks * heads * elems) * sizeof(float), &ws)) return rc;
  SsmArgs a{view_ptr<float>(xbc), view_ptr<float>(dt), buf_ptr<float>(dt_bias), buf_ptr<float>(a_log), buf_ptr<float>(skip), static_cast<float*>(s->ptr),
            static_cast<float*>(ws) + 2 * n_decay, static_cast<float*>(ws), static_cast<float*>(ws) + n_decay, view_ptr<float>(dst), xbc.stride, dt.stride, dst.stride,
            (int)t, (int)heads, (int)vdim, (int)groups, (int)state, q, (int)chunks, pos == 0};
  // a group's heads share a workgroup unless the chip would stay empty
  const size_t per = heads / groups;
  size_t share = (512 + chunks * groups - 1) / (chunks * groups);
  if (share > per) share = per;
  const dim3 grid((unsigned)chunks, (unsigned)groups, (unsigned)share);
  const bool vec = vdim % 4 == 0 && state % 4 == 0 && xbc.stride % 4 == 0 && (reinterpret_cast<uintptr_t>(a.xbc) & 15) == 0;
  static const hipError_t attr = [] {
    hipError_t e = hipSuccess;
    for (const void* f : {reinterpret_cast<const void*>(ssm_chunk_state_kernel<true>), reinterpret_cast<const void*>(ssm_chunk_state_kernel<false>),
                          reinterpret_cast<const void*>(ssm_chunk_out_kernel<true>), reinterpret_cast<const void*>(ssm_chunk_out_kernel<false>)})
      if (e == hipSuccess) e = hipFuncSetAttribute(f, hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    return e;
  }();
  UGHIP_HIPCHK(attr);
  const size_t lds_s = state_lds_bytes(q, (int)state), lds_o = out_lds_bytes(q, (int)state);
  ssm_chunk_decays_kernel<<<dim3((unsigned)chunks, (unsigned)((heads + 3) / 4)), 256, 0, dev->stream>>>(a);
  if (vec) ssm_chunk_state_kernel<true><<<grid, 256, lds_s, dev->stream>>>(a);
  else ssm_chunk_state_kernel<false><<<grid, 256, lds_s, dev->stream>>>(a);
  ssm_chunk_scan_kernel<<<dim3((unsigned)((elems + 255) / 256), (unsigned)heads), 256, 0, dev->stream>>>(a);
  if (vec) ssm_chunk_out_kernel<true><<<grid, 256, lds_o, dev->stream>>>(a);
  else ssm_chunk_out_kernel<false><<<grid, 256, lds_o, dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_ssm_step(ughip_device* dev, const ughip_slice* p, size_t xbc_offset, size_t dt_offset, const ughip_slice* taps, const ughip_slice* conv_bias,
                              size_t n_taps, ughip_slice* ring, const ughip_slice* dt_bias, const ughip_slice* a_log, const ughip_slice* skip, ughip_slice* s, size_t pos,
                              size_t heads, size_t vdim, size_t groups, size_t state, ughip_view dst) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "ssm_step: null device");
  if (heads == 0 || vdim == 0 || groups == 0 || state == 0 || heads % groups != 0 || heads > 65535 || vdim > 65535 || state > 4096)
    return set_error(UGHIP_ERR_INVALID, "ssm_step: heads %zu, vdim %zu, groups %zu, state %zu", heads, vdim, groups, state);
  if (n_taps == 0 || n_taps > 1024) return set_error(UGHIP_ERR_INVALID, "ssm_step: %zu taps", n_taps);
  const size_t ch = heads * vdim + 2 * groups * state;
  ughip_view in{const_cast<ughip_slice*>(p), xbc_offset, ch}, dt{const_cast<ughip_slice*>(p), dt_offset, heads};
  if (int rc = check_view(dev, in, 1, ch, UGHIP_F32, "ssm_step p")) return rc;
  if (int rc = check_view(dev, dt, 1, heads, UGHIP_F32, "ssm_step p")) return rc;
  if (int rc = check_buf(dev, taps, ch * n_taps, UGHIP_F32, "ssm_step taps")) return rc;
  if (conv_bias)
    if (int rc = check_buf(dev, conv_bias, ch, UGHIP_F32, "ssm_step conv bias")) return rc;
  if (int rc = check_buf(dev, ring, n_taps * ch, UGHIP_F32, "ssm_step ring")) return rc;
  for (const ughip_slice* v : {dt_bias, a_log, skip})
    if (int rc = check_buf(dev, v, heads, UGHIP_F32, "ssm_step per-head vector")) return rc;
  if (int rc = check_buf(dev, s, heads * state * vdim, UGHIP_F32, "ssm_step state")) return rc;
  if (int rc = check_view(dev, dst, 1, heads * vdim, UGHIP_F32, "ssm_step dst")) return rc;
  if (int rc = device_activate(dev)) return rc;
  SsmStepArgs a{view_ptr<float>(in), view_ptr<float>(dt), buf_ptr<float>(taps), buf_ptr<float>(conv_bias), static_cast<float*>(ring->ptr), buf_ptr<float>(dt_bias),
                buf_ptr<float>(a_log), buf_ptr<float>(skip), static_cast<float*>(s->ptr), view_ptr<float>(dst), (long long)pos, (int)n_taps, (int)heads, (int)vdim,
                (int)groups, (int)state, (int)ch};
  ssm_step_kernel<<<dim3((unsigned)heads, (unsigned)((vdim + STEP_COLS - 1) / STEP_COLS)), 256, 2 * state * sizeof(float), dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
