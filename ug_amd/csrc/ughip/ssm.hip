// A state-space recurrence (Mamba-2's) behind a causal convolution (ughip_layers.h).
//
//   S_t = exp(a_t) S_{t-1} + d_t B_t x_t^T,   y_t = S_t^T C_t + skip x_t,   a_t = -exp(a_log) d_t, d_t = softplus(dt_t + bias)
//
// Several positions run in chunks of Q.  With A_i = a_1 + .. + a_i inside a chunk:
//   ssm_chunk_state   what a chunk adds to the state: sum_j exp(A_Q - A_j) d_j B_j x_j^T              (one workgroup per chunk and head)
//   ssm_chunk_scan    the state in front of every chunk, S <- exp(A_Q) S + that, in place              (elementwise, chunks in order)
//   ssm_chunk_out     y_i = sum_{j <= i} exp(A_i - A_j) d_j (C_i . B_j) x_j + exp(A_i) S^T C_i + skip x_i
// Every exponent is <= 0.  The products are v_mfma_f32_16x16x4_f32 on f32 tiles in LDS (lane l: row or column l % 16, k = l / 16;
// result element e: row 4 (l / 16) + e, column l % 16).
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
  float* decay;    // [chunks, heads]: exp(A_Q)
  float* dst;
  size_t xbc_stride, dt_stride, dst_stride;
  int t, heads, vdim, groups, state, q, chunks;
  bool fresh;
};

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

// cum[i] = A_i and d[i] for the chunk's rows, rows past the end with d = 0 and the last A.  The first wave scans (q <= 64).
__device__ __forceinline__ void chunk_decays(const SsmArgs& a, int h, int row0, float* cum, float* d) {
  if (threadIdx.x < 64) {
    const int i = threadIdx.x;
    float dv = 0.f;
    if (i < a.q && row0 + i < a.t) dv = softplus_f(a.dt[(size_t)(row0 + i) * a.dt_stride + h] + a.dt_bias[h]);
    float s = -expf(a.a_log[h]) * dv;
    for (int k = 1; k < 64; k <<= 1) {
      const float o = __shfl_up(s, k, 64);
      if (i >= k) s += o;
    }
    if (i < a.q) cum[i] = s, d[i] = dv;
  }
  __syncthreads();
}

__device__ __forceinline__ f32x4_t mfma16(float x, float y, f32x4_t acc) { return __builtin_amdgcn_mfma_f32_16x16x4f32(x, y, acc, 0, 0, 0); }

constexpr int PB = 64;  // columns of vdim per workgroup

__device__ __host__ inline int pad16(int v) { return (v + 15) & ~15; }
// row strides of LDS tiles: 4 mod 64 or a multiple of 16 plus 4, so that 16 rows x 4 neighbours spread over the banks
__device__ __host__ inline int row_n(int state) { return pad16(state) + 4; }

__global__ void __launch_bounds__(256) ssm_chunk_state_kernel(SsmArgs a) {
  extern __shared__ float lds[];
  const int q = a.q, chunk = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * PB, row0 = chunk * q;
  const int pw = min(PB, a.vdim - p0), N = a.state, ns = row_n(N), ps = PB + 4, inner = a.heads * a.vdim, g = h / (a.heads / a.groups);
  float* cum = lds;
  float* d = lds + 64;
  float* Bs = lds + 128;      // [q][ns]
  float* Xs = Bs + q * ns;    // [q][ps]
  chunk_decays(a, h, row0, cum, d);
  const float end = cum[q - 1];
  const int np = pad16(N);
  for (int e = threadIdx.x; e < q * np; e += 256) {
    const int i = e / np, n = e % np;
    float v = 0.f;
    if (row0 + i < a.t && n < N) v = a.xbc[(size_t)(row0 + i) * a.xbc_stride + inner + (size_t)g * N + n] * (d[i] * expf(end - cum[i]));
    Bs[i * ns + n] = v;
  }
  for (int e = threadIdx.x; e < q * PB; e += 256) {
    const int i = e / PB, p = e % PB;
    Xs[i * ps + p] = row0 + i < a.t && p < pw ? a.xbc[(size_t)(row0 + i) * a.xbc_stride + (size_t)h * a.vdim + p0 + p] : 0.f;
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, kg = lane >> 4;
  const int tn = np / 16, tp = pad16(pw) / 16;
  float* out = a.chunk_s + ((size_t)chunk * a.heads + h) * N * a.vdim;
  for (int tile = wave; tile < tn * tp; tile += 4) {
    const int n0 = (tile / tp) * 16, c0 = (tile % tp) * 16;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    for (int k = kg; k < q; k += 4) acc = mfma16(Bs[k * ns + n0 + j], Xs[k * ps + c0 + j], acc);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int n = n0 + 4 * kg + e;
      if (n < N && c0 + j < pw) out[(size_t)n * a.vdim + p0 + c0 + j] = acc[e];
    }
  }
  if (blockIdx.z == 0 && threadIdx.x == 0) a.decay[(size_t)chunk * a.heads + h] = expf(end);
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
    s = a.decay[(size_t)c * a.heads + h] * s + add;
  }
  a.s[h * per + e] = s;
}

__global__ void __launch_bounds__(256) ssm_chunk_out_kernel(SsmArgs a) {
  extern __shared__ float lds[];
  const int q = a.q, chunk = blockIdx.x, h = blockIdx.y, p0 = blockIdx.z * PB, row0 = chunk * q;
  const int pw = min(PB, a.vdim - p0), N = a.state, ns = row_n(N), ps = PB + 4, ms = q + 4, inner = a.heads * a.vdim, g = h / (a.heads / a.groups);
  float* cum = lds;
  float* d = lds + 64;
  float* Bs = lds + 128;      // [q][ns]
  float* Cs = Bs + q * ns;    // [q][ns]
  float* Xs = Cs + q * ns;    // [q][ps]
  float* Ms = Xs + q * ps;    // [q][ms]
  chunk_decays(a, h, row0, cum, d);
  const int np = pad16(N);
  for (int e = threadIdx.x; e < q * np; e += 256) {
    const int i = e / np, n = e % np;
    float b = 0.f, c = 0.f;
    if (row0 + i < a.t && n < N) {
      const float* row = a.xbc + (size_t)(row0 + i) * a.xbc_stride + inner + (size_t)g * N + n;
      b = row[0];
      c = row[(size_t)a.groups * N];
    }
    Bs[i * ns + n] = b;
    Cs[i * ns + n] = c;
  }
  for (int e = threadIdx.x; e < q * PB; e += 256) {
    const int i = e / PB, p = e % PB;
    Xs[i * ps + p] = row0 + i < a.t && p < pw ? a.xbc[(size_t)(row0 + i) * a.xbc_stride + (size_t)h * a.vdim + p0 + p] : 0.f;
  }
  __syncthreads();
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, kg = lane >> 4, tq = q / 16;
  for (int tile = wave; tile < tq * tq; tile += 4) {
    const int i0 = (tile / tq) * 16, j0 = (tile % tq) * 16;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f};
    if (j0 <= i0)
      for (int k = kg; k < np; k += 4) acc = mfma16(Cs[(i0 + j) * ns + k], Bs[(j0 + j) * ns + k], acc);
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = i0 + 4 * kg + e, jj = j0 + j;
      Ms[i * ms + jj] = jj <= i ? acc[e] * expf(cum[i] - cum[jj]) * d[jj] : 0.f;
    }
  }
  __syncthreads();
  const int tp = pad16(pw) / 16;
  const float* S = a.chunk_s + ((size_t)chunk * a.heads + h) * N * a.vdim + p0;
  for (int tile = wave; tile < tq * tp; tile += 4) {
    const int i0 = (tile / tp) * 16, c0 = (tile % tp) * 16;
    f32x4_t acc = {0.f, 0.f, 0.f, 0.f}, from_s = {0.f, 0.f, 0.f, 0.f};
    for (int k = kg; k < i0 + 16; k += 4) acc = mfma16(Ms[(i0 + j) * ms + k], Xs[k * ps + c0 + j], acc);
    const bool col_ok = c0 + j < pw;
    for (int k = kg; k < np; k += 4) from_s = mfma16(Cs[(i0 + j) * ns + k], col_ok && k < N ? S[(size_t)k * a.vdim + c0 + j] : 0.f, from_s);
    if (!col_ok) continue;
#pragma unroll
    for (int e = 0; e < 4; ++e) {
      const int i = i0 + 4 * kg + e;
      if (row0 + i < a.t)
        a.dst[(size_t)(row0 + i) * a.dst_stride + (size_t)h * a.vdim + p0 + c0 + j] = acc[e] + expf(cum[i]) * from_s[e] + a.skip[h] * Xs[i * ps + c0 + j];
    }
  }
}

// One position in one launch.  A workgroup takes a head and 16 of its columns: it convolves those columns and the head's B and
// C rows (again in every workgroup: a few hundred channels), then 16 threads per column walk the state.  The ring's slot of this
// position is one no tap of this position reads, so the rows go in while other workgroups still convolve.
constexpr int STEP_COLS = 16;
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
  const int col = threadIdx.x & 15, ng = threadIdx.x >> 4, p = p0 + col;
  const float d = softplus_f(a.dt[h] + a.dt_bias[h]), keep = expf(-expf(a.a_log[h]) * d);
  float y = 0.f;
  if (p < a.vdim) {
    const float dx = d * xs[col];
    float* S = a.s + (size_t)h * N * a.vdim + p;
    for (int n = ng; n < N; n += 16) {
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

size_t chunk_lds_bytes(int q, int state) { return (size_t)(128 + 2 * q * row_n(state) + q * (PB + 4) + q * (q + 4)) * sizeof(float); }

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
  while (q > 16 && (chunk_lds_bytes(q, (int)state) > 160 * 1024 || (size_t)(q / 2) >= t)) q /= 2;
  const size_t lds = chunk_lds_bytes(q, (int)state);
  if (lds > 160 * 1024) return set_error(UGHIP_ERR_UNSUPPORTED, "ssm_rows: a state of %zu rows does not fit LDS", state);
  if (int rc = device_activate(dev)) return rc;
  const size_t chunks = (t + q - 1) / q, per = state * vdim, decay_bytes = (chunks * heads * sizeof(float) + 255) & ~(size_t)255;
  void* ws = nullptr;
  if (int rc = rows_scratch(dev, decay_bytes + chunks * heads * per * sizeof(float), &ws)) return rc;
  SsmArgs a{view_ptr<float>(xbc), view_ptr<float>(dt), buf_ptr<float>(dt_bias), buf_ptr<float>(a_log), buf_ptr<float>(skip), static_cast<float*>(s->ptr),
            reinterpret_cast<float*>(static_cast<char*>(ws) + decay_bytes), static_cast<float*>(ws), view_ptr<float>(dst), xbc.stride, dt.stride, dst.stride,
            (int)t, (int)heads, (int)vdim, (int)groups, (int)state, q, (int)chunks, pos == 0};
  const dim3 grid((unsigned)chunks, (unsigned)heads, (unsigned)((vdim + PB - 1) / PB));
  static const hipError_t attr = [] {
    hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(ssm_chunk_state_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
    return e != hipSuccess ? e : hipFuncSetAttribute(reinterpret_cast<const void*>(ssm_chunk_out_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, 160 * 1024);
  }();
  UGHIP_HIPCHK(attr);
  ssm_chunk_state_kernel<<<grid, 256, lds, dev->stream>>>(a);
  ssm_chunk_scan_kernel<<<dim3((unsigned)((per + 255) / 256), (unsigned)heads), 256, 0, dev->stream>>>(a);
  ssm_chunk_out_kernel<<<grid, 256, lds, dev->stream>>>(a);
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
