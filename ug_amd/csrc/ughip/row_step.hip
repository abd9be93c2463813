// Products of one row with their neighbours folded in (ughip_product_row): a decode step of the layers in ughip_layers.h.
//
// A workgroup of four waves takes 4 R columns, R per wave.  It asks for everything the input row is made of (PV 16-byte pieces per
// thread and vector), then every wave for the first NB batches of four runs of 512 elements of its matrix rows (eight elements per
// lane and run);
// the row -- residual add with the norm of the sublayer in front, gate, norm -- is made in LDS in the shadow of the matrix, and
// every wave multiplies, asking for batch b + NB where batch b was.  The input row costs a few cache reads per workgroup and spares the launches that would make it; the
// first workgroup stores the new residual.  PLAIN: the row is x as it is (or, routed, times the experts' weights).  PV = 0: rows of any
// length and alignment, element by element.
#include <hip/hip_runtime.h>

#include "layers.h"
#include "route.h"

using namespace ughip;

namespace {

struct RowArgs {
  const float* x;
  const float* y;
  const float* y_norm;
  const float* gate;
  const float* norm;
  float* x_out;  // null: not kept
  float* dst;
  const void* w;
  const float* bias;
  const void* table;
  const int* ids;
  size_t table_stride, table_col, w_group;
  const float* extra;  // joins x too
  GluForm glu;
  float eps, inv_k;
  int n, k, cols, norm_groups, table_rows, segs;
  bool table_bf16, gate_after;
  const float* logits;
  RouteArgs route;
  int* route_ids;
  float* route_weights;
};

constexpr int RUN = 512, PRE = 4;

template <typename WT>
struct Eight;
template <>
struct Eight<uint16_t> {
  u32x4_t v;
  __device__ void clear() { v = u32x4_t{0, 0, 0, 0}; }
  __device__ void load(const uint16_t* p) { v = __builtin_nontemporal_load(reinterpret_cast<const u32x4_t*>(p)); }
  __device__ void load_some(const uint16_t* p, int left) {
    uint32_t e[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) e[i] = i < left ? p[i] : 0;
    v = u32x4_t{e[0] | e[1] << 16, e[2] | e[3] << 16, e[4] | e[5] << 16, e[6] | e[7] << 16};
  }
  __device__ float dot(const f32x4_t& a, const f32x4_t& b, float s) const {
    s += __uint_as_float(v.x << 16) * a.x;
    s += __uint_as_float(v.x & 0xffff0000u) * a.y;
    s += __uint_as_float(v.y << 16) * a.z;
    s += __uint_as_float(v.y & 0xffff0000u) * a.w;
    s += __uint_as_float(v.z << 16) * b.x;
    s += __uint_as_float(v.z & 0xffff0000u) * b.y;
    s += __uint_as_float(v.w << 16) * b.z;
    s += __uint_as_float(v.w & 0xffff0000u) * b.w;
    return s;
  }
};
template <>
struct Eight<float> {
  f32x4_t u, v;
  __device__ void clear() { u = v = f32x4_t{0.f, 0.f, 0.f, 0.f}; }
  __device__ void load(const float* p) {
    u = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(p));
    v = __builtin_nontemporal_load(reinterpret_cast<const f32x4_t*>(p) + 1);
  }
  __device__ void load_some(const float* p, int left) {
    float e[8];
#pragma unroll
    for (int i = 0; i < 8; ++i) e[i] = i < left ? p[i] : 0.f;
    u = f32x4_t{e[0], e[1], e[2], e[3]}, v = f32x4_t{e[4], e[5], e[6], e[7]};
  }
  __device__ float dot(const f32x4_t& a, const f32x4_t& b, float s) const {
    s += u.x * a.x;
    s += u.y * a.y;
    s += u.z * a.z;
    s += u.w * a.w;
    s += v.x * b.x;
    s += v.y * b.y;
    s += v.z * b.z;
    s += v.w * b.w;
    return s;
  }
};

// R columns of NM matrices per wave; VEC: rows are 16-byte aligned and a multiple of 8 long.  ROUTE as in ughip_row_step: with 2 a
// column's row is the chosen experts' rows one after the other, each from a batch of its own on.
template <typename WT, int R, int NM, int ROUTE, bool VEC, int NB, int PV, bool PLAIN>
__global__ void __launch_bounds__(256) row_step_kernel(RowArgs a) {
  extern __shared__ __attribute__((aligned(16))) float in[];  // the row (segments `padded` apart), then ROUTE 1: logits and work space
  __shared__ float red[4][4];
  __shared__ float part_sum[4 * (PV ? PV : 1)];
  __shared__ int s_ids[64];
  __shared__ float s_wts[64];
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
  const int padded = (a.k + RUN - 1) / RUN * RUN, bps = (padded / RUN + PRE - 1) / PRE, batches = (ROUTE == 2 ? a.segs : 1) * bps;
  const int col0 = (blockIdx.x * 4 + wave) * R;
  constexpr int NP = PV ? PV : 1;
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  const int total = (ROUTE == 2 ? a.segs : 1) * a.k;
  f32x4_t px[NP], py[NP], pyn[NP], pn[NP], pe[NP];  // x, y or the gate, the two norms' weights, and what joins x besides
  if constexpr (PV != 0 && PLAIN) {
#pragma unroll
    for (int u = 0; u < PV; ++u) {
      const int i = (u * 256 + (int)threadIdx.x) * 4;
      px[u] = i < total ? *reinterpret_cast<const f32x4_t*>(a.x + i) : zero;
    }
  } else if constexpr (PV != 0) {
#pragma unroll
    for (int u = 0; u < PV; ++u) {
      const int i = (u * 256 + (int)threadIdx.x) * 4;
      const bool ok = i < a.k;  // a multiple of 4
      px[u] = ok ? *reinterpret_cast<const f32x4_t*>(a.x + i) : zero;
      py[u] = ok && (a.y || a.gate) ? *reinterpret_cast<const f32x4_t*>((a.y ? a.y : a.gate) + i) : zero;
      pyn[u] = ok && a.y ? *reinterpret_cast<const f32x4_t*>(a.y_norm + i) : zero;
      pn[u] = ok && a.norm ? *reinterpret_cast<const f32x4_t*>(a.norm + i) : zero;
      pe[u] = ok && a.extra ? *reinterpret_cast<const f32x4_t*>(a.extra + i) : zero;
    }
  }
  if constexpr (ROUTE == 1) {  // which experts' matrices: before anything of them can be asked for
    float* lg = in + padded;
    for (int e = threadIdx.x; e < a.route.experts; e += 256) lg[e] = a.logits[e];
    __syncthreads();
    if (wave == 0) {
      float* work = lg + a.route.experts;
      int* ids = reinterpret_cast<int*>(work + route_lds_floats(a.route.experts, a.route.groups));
      float* wts = reinterpret_cast<float*>(ids + a.route.top);
      route_choose(lg, a.route, work, ids, wts);
      if (lane < a.route.top) s_ids[lane] = ids[lane];
      if (blockIdx.x == 0 && lane < a.route.top) a.route_ids[lane] = ids[lane], a.route_weights[lane] = wts[lane];
    }
    __syncthreads();
  }
  if constexpr (ROUTE == 2) {
    if (threadIdx.x < (unsigned)a.segs) {
      const int e = a.route_ids[threadIdx.x];
      s_ids[threadIdx.x] = e >= 0 && e < a.route.experts ? e : 0;
      s_wts[threadIdx.x] = a.route_weights[threadIdx.x];
    }
    __syncthreads();
  }
  // a column's matrix row; ROUTE 1: column j n + c is column c of the j-th chosen expert
  const WT* rows[NM][R];
  bool live[R];
#pragma unroll
  for (int r = 0; r < R; ++r) {
    const int col = col0 + r;
    live[r] = col < a.cols;
    size_t at = (size_t)(live[r] ? col : 0) * a.k;
    if (ROUTE == 1) {
      const int j = live[r] ? col / a.n : 0;
      at = (size_t)s_ids[j] * a.w_group + (size_t)((live[r] ? col : 0) - j * a.n) * a.k;
    }
    rows[0][r] = static_cast<const WT*>(a.w) + at;
    if (NM == 2) rows[NM - 1][r] = static_cast<const WT*>(a.w) + at + (size_t)a.n * a.k;  // gate rows, then up rows
  }
  Eight<WT> held[NB][NM][R][PRE];
  int fj = 0, fc = 0;  // the next batch to ask for: segment and batch inside it
  auto fetch = [&](Eight<WT>(&to)[NM][R][PRE]) {
    if (ROUTE == 2 ? fj >= a.segs : fc >= bps) return;  // the same for the whole workgroup
    const size_t seg = ROUTE == 2 ? (size_t)s_ids[fj] * a.w_group : 0;
#pragma unroll
    for (int c = 0; c < PRE; ++c) {
      const int kk = (fc * PRE + c) * RUN + lane * 8;
#pragma unroll
      for (int r = 0; r < R; ++r)
#pragma unroll
        for (int m = 0; m < NM; ++m) {
          Eight<WT>& e = to[m][r][c];
          // every lane loads (past the row's end: its first elements, which meet zeros): with branches around loads the compiler
          // waits for all of them at once
          if constexpr (VEC) e.load(rows[m][r] + seg + (kk < a.k ? kk : 0));
          else e.load_some(rows[m][r] + seg + kk, live[r] ? a.k - kk : 0);
        }
    }
    if (ROUTE == 2 && fc + 1 == bps) ++fj, fc = 0;
    else ++fc;
  };
#pragma unroll
  for (int b = 0; b < NB; ++b) fetch(held[b]);
  __builtin_amdgcn_sched_barrier(0);

  // the input row
  float ss = 0.f;
  if constexpr (PV != 0 && PLAIN) {
#pragma unroll
    for (int u = 0; u < PV; ++u) {
      const int i = (u * 256 + (int)threadIdx.x) * 4;
      if constexpr (ROUTE == 2) {
        // (i + 1/2) / k is never within a rounding of a whole number
        const int j = (int)(((float)i + 0.5f) * a.inv_k);
        if (i < total) *reinterpret_cast<f32x4_t*>(in + j * padded + (i - j * a.k)) = px[u] * s_wts[j];
      } else {
        if (i < padded) *reinterpret_cast<f32x4_t*>(in + i) = px[u];
      }
    }
    if constexpr (ROUTE == 2)
      for (int j = 0; j < a.segs; ++j)
        for (int i = a.k + (int)threadIdx.x; i < padded; i += 256) in[j * padded + i] = 0.f;
  } else if constexpr (ROUTE == 2) {
    for (int j = 0; j < a.segs; ++j) {
      const float w = s_wts[j];
      for (int i = threadIdx.x; i < padded; i += 256) in[j * padded + i] = i < a.k ? a.x[j * a.k + i] * w : 0.f;
    }
  } else if constexpr (PV != 0) {
    auto square = [](const f32x4_t& v) { return v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; };
    if (a.y) {
#pragma unroll
      for (int u = 0; u < PV; ++u) ss += square(py[u]);
      ss = block_sum<4>(ss, red[0]);
      const float inv = 1.f / sqrtf(ss / (float)a.k + a.eps);
#pragma unroll
      for (int u = 0; u < PV; ++u) {
        px[u] = px[u] + py[u] * inv * pyn[u] + pe[u];
        const int i = (u * 256 + (int)threadIdx.x) * 4;
        if (a.x_out && blockIdx.x == 0 && i < a.k) *reinterpret_cast<f32x4_t*>(a.x_out + i) = px[u];
      }
    } else if (a.gate && !a.gate_after) {
#pragma unroll
      for (int u = 0; u < PV; ++u)
#pragma unroll
        for (int e = 0; e < 4; ++e) px[u][e] *= silu_f(py[u][e]);
    }
    if (a.norm && a.norm_groups == 1) {
      ss = 0.f;
#pragma unroll
      for (int u = 0; u < PV; ++u) ss += square(px[u]);
      ss = block_sum<4>(ss, red[1]);
      const float inv = 1.f / sqrtf(ss / (float)a.k + a.eps);
#pragma unroll
      for (int u = 0; u < PV; ++u) px[u] = px[u] * inv * pn[u];
    } else if (a.norm && a.k < 256 * a.norm_groups) {
      // parts inside a wave's piece: 4, 8, .. or 128 elements (the host checks)
      const int part = a.k / a.norm_groups;
#pragma unroll
      for (int u = 0; u < PV; ++u) {
        float s = square(px[u]);
        for (int d = part >> 3; d; d >>= 1) s += __shfl_xor(s, d, 64);
        px[u] = px[u] * (1.f / sqrtf(s / (float)part + a.eps)) * pn[u];
      }
    } else if (a.norm) {
      // parts of whole runs of 256 elements (the host checks): one wave's pieces each
      const int runs = a.k / a.norm_groups / 256;
#pragma unroll
      for (int u = 0; u < PV; ++u) {
        const float s = wave_sum(square(px[u]));
        if (lane == 0) part_sum[u * 4 + wave] = s;
      }
      __syncthreads();
#pragma unroll
      for (int u = 0; u < PV; ++u) {
        const int first = (u * 4 + wave) / runs * runs;
        float s = 0.f;
        for (int i = 0; i < runs && first + i < 4 * PV; ++i) s += part_sum[first + i];
        px[u] = px[u] * (1.f / sqrtf(s / (float)(runs * 256) + a.eps)) * pn[u];
      }
    }
    if (a.gate && a.gate_after) {
#pragma unroll
      for (int u = 0; u < PV; ++u)
#pragma unroll
        for (int e = 0; e < 4; ++e) px[u][e] *= sigmoid_f(py[u][e]);
    }
#pragma unroll
    for (int u = 0; u < PV; ++u) {
      const int i = (u * 256 + (int)threadIdx.x) * 4;
      if (i < padded) *reinterpret_cast<f32x4_t*>(in + i) = px[u];
    }
  } else {
    for (int i = threadIdx.x; i < padded; i += 256) {
      float v = 0.f;
      if (i < a.k) {
        v = a.y ? a.y[i] : a.x[i];
        if (a.gate && !a.gate_after) v *= silu_f(a.gate[i]);
      }
      in[i] = v;  // read back by the same thread until the last barrier
      ss += v * v;
    }
    if (a.y) {
      ss = block_sum<4>(ss, red[0]);
      const float inv = 1.f / sqrtf(ss / (float)a.k + a.eps);
      ss = 0.f;
      for (int i = threadIdx.x; i < a.k; i += 256) {
        const float v = a.x[i] + in[i] * inv * a.y_norm[i] + (a.extra ? a.extra[i] : 0.f);
        in[i] = v;
        ss += v * v;
        if (a.x_out && blockIdx.x == 0) a.x_out[i] = v;
      }
    }
    if (a.norm && a.norm_groups == 1) {
      ss = block_sum<4>(ss, red[1]);
      const float inv = 1.f / sqrtf(ss / (float)a.k + a.eps);
      for (int i = threadIdx.x; i < a.k; i += 256) in[i] *= inv * a.norm[i];
    } else if (a.norm) {
      const int part = a.k / a.norm_groups;
      __syncthreads();  // a part is summed by one wave
      for (int g = wave; g < a.norm_groups; g += 4) {
        float s = 0.f;
        for (int i = lane; i < part; i += 64) s += in[g * part + i] * in[g * part + i];
        s = wave_sum(s);
        const float inv = 1.f / sqrtf(s / (float)part + a.eps);
        for (int i = lane; i < part; i += 64) in[g * part + i] *= inv * a.norm[g * part + i];
      }
    }
    if (a.gate && a.gate_after) {
      __syncthreads();
      for (int i = threadIdx.x; i < a.k; i += 256) in[i] *= sigmoid_f(a.gate[i]);
    }
  }
  __syncthreads();

  float acc[NM][R];
#pragma unroll
  for (int m = 0; m < NM; ++m)
#pragma unroll
    for (int r = 0; r < R; ++r) acc[m][r] = 0.f;
  int dj = 0, dc = 0;  // the batch to multiply
  auto multiply = [&](const Eight<WT>(&from)[NM][R][PRE]) {
    const float* row = in + dj * padded + dc * PRE * RUN + lane * 8;
    const int left = padded / RUN - dc * PRE;
#pragma unroll
    for (int c = 0; c < PRE; ++c) {
      if (c < left) {
        const f32x4_t xa = *reinterpret_cast<const f32x4_t*>(row + c * RUN), xb = *reinterpret_cast<const f32x4_t*>(row + c * RUN + 4);
#pragma unroll
        for (int r = 0; r < R; ++r)
#pragma unroll
          for (int m = 0; m < NM; ++m) acc[m][r] = from[m][r][c].dot(xa, xb, acc[m][r]);
      }
    }
    if (ROUTE == 2 && dc + 1 == bps) ++dj, dc = 0;
    else ++dc;
  };
  for (int b0 = 0; b0 < batches; b0 += NB) {
#pragma unroll
    for (int b = 0; b < NB; ++b) {
      if (b0 + b < batches) {
        multiply(held[b]);
        if (b0 + b + NB < batches) fetch(held[b]);
      }
    }
  }
#pragma unroll
  for (int r = 0; r < R; ++r) {
#pragma unroll
    for (int m = 0; m < NM; ++m) acc[m][r] = wave_sum(acc[m][r]);
    if (lane != 0 || !live[r]) continue;
    const int col = col0 + r;
    float v = acc[0][r];
    if (a.bias) v += a.bias[col];
    if (NM == 2) {
      float u = acc[NM - 1][r];
      if (a.bias) u += a.bias[a.n + col];
      v = glu_f(v, u, a.glu);
    } else if (a.table) {
      const int id = a.ids[0];
      float t = __uint_as_float(0x7fc00000u);
      if (id >= 0 && id < a.table_rows) {
        const size_t at = (size_t)id * a.table_stride + a.table_col + col;
        t = a.table_bf16 ? bf16_to_f32(static_cast<const uint16_t*>(a.table)[at]) : static_cast<const float*>(a.table)[at];
      }
      v = gelu_tanh_f(v) * t;
    }
    a.dst[col] = v;
  }
}

template <typename WT, int R, int NM, int ROUTE, bool VEC, int NB, int PV, bool PLAIN>
hipError_t launch_one(hipStream_t st, const RowArgs& a, size_t lds) {
  const unsigned grid = (unsigned)((a.cols + 4 * R - 1) / (4 * R));
  auto kernel = row_step_kernel<WT, R, NM, ROUTE, VEC, NB, PV, PLAIN>;
  if (lds > 60 * 1024)
    if (hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); e != hipSuccess) return e;
  kernel<<<grid, 256, lds, st>>>(a);
  return hipGetLastError();
}

// pieces: the input row is read 16 bytes at a time
template <typename WT, int R, int NM, int ROUTE>
hipError_t launch_vec(hipStream_t st, const RowArgs& a, size_t lds, bool vec, bool pieces) {
  if (!vec) return launch_one<WT, R, NM, ROUTE, false, 1, 0, false>(st, a, lds);
  const int total = (ROUTE == 2 ? a.segs : 1) * a.k;
  if (pieces && !a.y && !a.gate && !a.norm && total <= 8192) {
    if constexpr (ROUTE != 2)
      if (total <= 2048) return launch_one<WT, R, NM, ROUTE, true, 1, 2, true>(st, a, lds);
    return launch_one<WT, R, NM, ROUTE, true, 2, 8, true>(st, a, lds);
  }
  if constexpr (ROUTE != 2) {
    if (pieces && a.k <= 2048) return launch_one<WT, R, NM, ROUTE, true, 1, 2, false>(st, a, lds);
    if (pieces && a.k <= 4096) return launch_one<WT, R, NM, ROUTE, true, 2, 4, false>(st, a, lds);
  }
  return launch_one<WT, R, NM, ROUTE, true, 2, 0, false>(st, a, lds);
}

template <typename WT, int NM, int ROUTE>
hipError_t launch_rows(hipStream_t st, const RowArgs& a, size_t lds, bool vec, bool pieces) {
  // enough workgroups for the chip first, then more columns for each of them to share the input row
  const int r = a.cols >= 8192 && NM == 1 ? 4 : a.cols >= 2048 ? 2 : 1;
  if constexpr (NM == 1)
    if (r == 4) return launch_vec<WT, 4, NM, ROUTE>(st, a, lds, vec, pieces);
  return r >= 2 ? launch_vec<WT, 2, NM, ROUTE>(st, a, lds, vec, pieces) : launch_vec<WT, 1, NM, ROUTE>(st, a, lds, vec, pieces);
}

template <typename WT>
hipError_t launch_any(hipStream_t st, const RowArgs& a, int route, bool up, size_t lds, bool vec, bool pieces) {
  if (route == 1) return up ? launch_rows<WT, 2, 1>(st, a, lds, vec, pieces) : hipErrorInvalidValue;
  if (route == 2) return launch_rows<WT, 1, 2>(st, a, lds, vec, pieces);
  return up ? launch_rows<WT, 2, 0>(st, a, lds, vec, pieces) : launch_rows<WT, 1, 0>(st, a, lds, vec, pieces);
}

constexpr size_t ROW_MAX = 16000;

}  // namespace

extern "C" int ughip_product_row(ughip_device* dev, const ughip_row_step* p) {
  const char* what = "product_row";
  if (!dev || !p || !p->w || !p->x || !p->dst) return set_error(UGHIP_ERR_INVALID, "%s: null argument", what);
  if (p->act < UGHIP_ACT_NONE || p->act > UGHIP_ACT_GLU || p->route < 0 || p->route > 2) return set_error(UGHIP_ERR_INVALID, "%s: act %d, route %d", what, p->act, p->route);
  if (p->n == 0) return UGHIP_OK;
  const size_t segs = p->route == 2 ? p->top : 1, total = segs * p->k;
  if (p->k == 0 || p->k > ROW_MAX || segs == 0 || segs > 64 || segs * ((p->k + RUN - 1) / RUN * RUN) > 32 * RUN) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: %zu rows of %zu elements, up to %zu in all (in runs of %d) are supported", what, segs, p->k, (size_t)32 * RUN, RUN);
  if (p->n > 0x7fffffffull / 128) return set_error(UGHIP_ERR_INVALID, "%s: shape too large", what);
  if (p->w->dtype != UGHIP_F32 && p->w->dtype != UGHIP_BF16) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: matrices are F32 or BF16", what);
  const bool glu = p->act == UGHIP_ACT_SWIGLU || p->act == UGHIP_ACT_GLU;  // gate and up rows
  const size_t mats = p->route ? p->experts : 1, w_rows = glu ? 2 * p->n : p->n;
  if (p->route) {
    if (int rc = route_check(p->experts, p->groups, p->keep, p->top, what)) return rc;
    if (p->top > 64) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: up to 64 experts per row", what);
    if (p->bias || (p->route == 1 && !glu) || (p->route == 2 && p->act != UGHIP_ACT_NONE) || p->y || p->norm || p->gate)
      return set_error(UGHIP_ERR_UNSUPPORTED, "%s: routed products are SwiGLU (1) or plain (2), on x as it is", what);
    if (int rc = check_buf(dev, p->route_ids, p->top, UGHIP_I32, "product_row ids")) return rc;
    if (int rc = check_buf(dev, p->route_weights, p->top, UGHIP_F32, "product_row weights")) return rc;
  }
  auto row = [&](const ughip_slice* s, size_t off, size_t n, int dtype) { return check_view(dev, ughip_view{const_cast<ughip_slice*>(s), off, n}, 1, n, dtype, what); };
  if (int rc = row(p->x, p->x_offset, total, UGHIP_F32)) return rc;
  if (p->y) {
    if (int rc = row(p->y, p->y_offset, p->k, UGHIP_F32)) return rc;
    if (int rc = row(p->y_norm, 0, p->k, UGHIP_F32)) return rc;
  }
  if (p->extra) {
    if (!p->y) return set_error(UGHIP_ERR_INVALID, "%s: extra rows come with y", what);
    if (int rc = row(p->extra, p->extra_offset, p->k, UGHIP_F32)) return rc;
  }
  if (p->gate_after && !p->gate) return set_error(UGHIP_ERR_INVALID, "%s: gate_after without a gate", what);
  if (p->gate)
    if (int rc = row(p->gate, p->gate_offset, p->k, UGHIP_F32)) return rc;
  if (p->gate && p->y) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: a gate or a residual, not both", what);
  const size_t norm_groups = p->norm_groups ? p->norm_groups : 1;
  if (p->norm) {
    if (p->k % norm_groups) return set_error(UGHIP_ERR_INVALID, "%s: %zu elements in %zu groups", what, p->k, norm_groups);
    if (int rc = row(p->norm, 0, p->k, UGHIP_F32)) return rc;
  }
  if (int rc = row(p->w, 0, mats * w_rows * p->k, -1)) return rc;
  if (p->bias)
    if (int rc = row(p->bias, 0, w_rows, UGHIP_F32)) return rc;
  const size_t cols = p->route == 1 ? p->top * p->n : p->n;
  if (int rc = row(p->dst, p->dst_offset, cols, UGHIP_F32)) return rc;
  if (p->keep_x) {
    if (!p->y) return set_error(UGHIP_ERR_INVALID, "%s: nothing joins x", what);
    if (int rc = row(p->dst, p->x_out, p->k, UGHIP_F32)) return rc;
  }
  if (p->dst == p->x || p->dst == p->y || p->dst == p->gate || (p->extra && p->dst == p->extra)) return set_error(UGHIP_ERR_INVALID, "%s: dst aliases an input", what);
  if (p->act == UGHIP_ACT_GELU_MUL) {
    if (!p->table || (p->table->dtype != UGHIP_F32 && p->table->dtype != UGHIP_BF16)) return set_error(UGHIP_ERR_INVALID, "%s: a gate's table is F32 or BF16", what);
    if (int rc = row(p->table, 0, p->table_rows * p->table_stride, -1)) return rc;
    if (p->table_col > p->table_stride || p->n > p->table_stride - p->table_col) return set_error(UGHIP_ERR_BOUNDS, "%s: table columns %zu + %zu of %zu", what, p->table_col, p->n, p->table_stride);
    if (int rc = row(p->ids, 0, 1, UGHIP_I32)) return rc;
  }
  if (p->route == 1) {
    if (int rc = row(p->logits, p->logits_offset, p->experts, UGHIP_F32)) return rc;
    if (p->correction)
      if (int rc = row(p->correction, 0, p->experts, UGHIP_F32)) return rc;
  }
  if (int rc = device_activate(dev)) return rc;
  RowArgs a{};
  a.x = buf_ptr<float>(p->x) + p->x_offset;
  if (p->y) a.y = buf_ptr<float>(p->y) + p->y_offset, a.y_norm = buf_ptr<float>(p->y_norm);
  if (p->gate) a.gate = buf_ptr<float>(p->gate) + p->gate_offset, a.gate_after = p->gate_after != 0;
  if (p->extra) a.extra = buf_ptr<float>(p->extra) + p->extra_offset;
  a.glu = glu_form(p->act, p->act_alpha, p->act_shift, p->act_limit);
  a.norm = buf_ptr<float>(p->norm), a.norm_groups = (int)norm_groups;
  float* d = static_cast<float*>(p->dst->ptr);
  a.x_out = p->keep_x ? d + p->x_out : nullptr;
  a.dst = d + p->dst_offset;
  a.w = p->w->ptr;
  a.bias = buf_ptr<float>(p->bias);
  if (p->act == UGHIP_ACT_GELU_MUL) {
    a.table = p->table->ptr, a.table_bf16 = p->table->dtype == UGHIP_BF16, a.table_rows = (int)p->table_rows;
    a.table_stride = p->table_stride, a.table_col = p->table_col, a.ids = buf_ptr<int>(p->ids);
  }
  a.w_group = w_rows * p->k, a.eps = p->eps, a.inv_k = 1.f / (float)p->k, a.n = (int)p->n, a.k = (int)p->k, a.cols = (int)cols, a.segs = (int)segs;
  size_t lds = segs * ((p->k + RUN - 1) / RUN * RUN) * sizeof(float);
  if (p->route) {
    a.route = RouteArgs{buf_ptr<float>(p->correction), (int)p->experts, (int)p->groups, (int)p->keep, (int)p->top};
    a.route_ids = static_cast<int*>(p->route_ids->ptr), a.route_weights = static_cast<float*>(p->route_weights->ptr);
    if (p->route == 1) {
      a.logits = buf_ptr<float>(p->logits) + p->logits_offset;
      lds += (p->experts + (size_t)route_lds_floats(a.route.experts, a.route.groups) + 2 * p->top) * sizeof(float);
    }
  }
  const bool vec = p->k % 8 == 0 && (reinterpret_cast<uintptr_t>(a.w) & 15) == 0;
  auto a16 = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  const size_t part = p->k / norm_groups;
  const bool parts_fit = !p->norm || norm_groups == 1 || part % 256 == 0 || (part >= 4 && part < 256 && (part & (part - 1)) == 0);
  const bool pieces = p->k % 4 == 0 && parts_fit && a16(a.x) && a16(a.y) && a16(a.gate) && a16(a.x_out) && a16(a.extra);
  UGHIP_HIPCHK(p->w->dtype == UGHIP_BF16 ? launch_any<uint16_t>(dev->stream, a, p->route, glu, lds, vec, pieces)
                                         : launch_any<float>(dev->stream, a, p->route, glu, lds, vec, pieces));
  return UGHIP_OK;
}
