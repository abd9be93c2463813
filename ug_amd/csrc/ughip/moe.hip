// Routing of rows to experts (ughip_layers.h): scores on the f32 matrix pipe with the choice in the same kernel, and the
// sort of (row, expert) pairs that the grouped products read.
#include <hip/hip_runtime.h>

#include "layers.h"
#include "route.h"

using namespace ughip;

namespace {

// 16 rows per workgroup.  The eight waves share k: each multiplies every eighth run of 16 elements (v_mfma_f32_16x16x4_f32, k
// taken four elements per lane so that rows are read 16 bytes at a time), AHEAD runs asked for before the first is used; their
// partial logits meet in LDS in wave order; then each wave chooses for two of the rows.
constexpr int ROUTE_WAVES = 8, AHEAD = 4;

template <bool VEC>
__device__ __forceinline__ f32x4_t run4(const float* row, bool ok, int kk, int k) {
  f32x4_t v = {0.f, 0.f, 0.f, 0.f};
  if (VEC) {
    if (ok && kk < k) v = *reinterpret_cast<const f32x4_t*>(row + kk);
  } else {
#pragma unroll
    for (int c = 0; c < 4; ++c)
      if (ok && kk + c < k) v[c] = row[kk + c];
  }
  return v;
}

template <bool VEC, int NT>  // NT tiles of 16 experts at a time
__global__ void __launch_bounds__(64 * ROUTE_WAVES) route_rows_kernel(const float* __restrict__ x, size_t x_stride, const float* __restrict__ router, RouteArgs r, int m, int k,
                                                                      int* __restrict__ ids, float* __restrict__ weights) {
  extern __shared__ float smem[];
  const int E = r.experts, per_wave = route_lds_floats(E, r.groups);
  float* logits = smem;  // [16][E]
  float* work = smem + 16 * E;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, g = lane >> 4;
  const int row0 = blockIdx.x * 16;
  const bool row_ok = row0 + j < m;
  const float* xr = x + (size_t)(row_ok ? row0 + j : row0) * x_stride;
  for (int e0 = 0; e0 < E; e0 += 16 * NT) {
    f32x4_t acc[NT];
    const float* wr[NT];
    bool ok[NT];
#pragma unroll
    for (int i = 0; i < NT; ++i) {
      acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
      const int e = e0 + 16 * i + j;
      ok[i] = e < E;
      wr[i] = router + (size_t)(ok[i] ? e : 0) * k;
    }
    for (int k0 = wave * 16; k0 < k; k0 += 16 * ROUTE_WAVES * AHEAD) {
      f32x4_t xv[AHEAD], wv[AHEAD][NT];
#pragma unroll
      for (int u = 0; u < AHEAD; ++u) {
        const int kk = k0 + 16 * ROUTE_WAVES * u + 4 * g;
        xv[u] = run4<VEC>(xr, row_ok, kk, k);
#pragma unroll
        for (int i = 0; i < NT; ++i) wv[u][i] = run4<VEC>(wr[i], ok[i], kk, k);
      }
#pragma unroll
      for (int u = 0; u < AHEAD; ++u)
#pragma unroll
        for (int i = 0; i < NT; ++i)
#pragma unroll
          for (int c = 0; c < 4; ++c) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(xv[u][c], wv[u][i][c], acc[i], 0, 0, 0);
    }
    for (int wv = 0; wv < ROUTE_WAVES; ++wv) {
      if (wave == wv) {
#pragma unroll
        for (int i = 0; i < NT; ++i) {
          const int e = e0 + 16 * i + j;
          if (e >= E) continue;
#pragma unroll
          for (int q = 0; q < 4; ++q) {  // element q: row 4 g + q, column j
            float* at = logits + (4 * g + q) * E + e;
            *at = wv == 0 ? acc[i][q] : *at + acc[i][q];
          }
        }
      }
      __syncthreads();
    }
  }
  for (int t = 0; t < 16 / ROUTE_WAVES; ++t) {
    const int rr = wave * (16 / ROUTE_WAVES) + t;
    if (row0 + rr >= m) break;  // uniform over the wave
    const size_t at = (size_t)(row0 + rr) * r.top;
    route_choose(logits + rr * E, r, work + wave * per_wave, ids + at, weights + at);
  }
}

// A workgroup per expert: every thread takes a run of the pairs and counts the lower experts' and its expert's own, a scan over the
// threads says where its own go (in row order).
__global__ void __launch_bounds__(256) group_rows_kernel(const int* __restrict__ ids, int pairs, int top, int* __restrict__ row_index, int* __restrict__ slots,
                                                         int* __restrict__ group_end) {
  __shared__ int s_own[256], s_low[4];
  const int e = blockIdx.x, tid = threadIdx.x, lane = tid & 63, per = (pairs + 255) / 256, p0 = min(pairs, tid * per), p1 = min(pairs, p0 + per);
  int lower = 0, own = 0;
#pragma unroll 8
  for (int p = p0; p < p1; ++p) {
    const int id = ids[p];
    lower += id < e;
    own += id == e;
  }
  for (int d = 32; d; d >>= 1) lower += __shfl_xor(lower, d, 64);
  if (lane == 0) s_low[tid >> 6] = lower;
  s_own[tid] = own;
  __syncthreads();
  lower = s_low[0] + s_low[1] + s_low[2] + s_low[3];
  for (int d = 1; d < 256; d <<= 1) {  // inclusive scan
    const int o = tid >= d ? s_own[tid - d] : 0;
    __syncthreads();
    s_own[tid] += o;
    __syncthreads();
  }
  if (tid == 255) group_end[e] = lower + s_own[255];
  int at = lower + s_own[tid] - own;
  if (own == 0) return;
  for (int p = p0; p < p1; ++p)
    if (ids[p] == e) {
      row_index[at] = p / top;
      slots[p] = at++;
    }
}

}  // namespace

extern "C" int ughip_route_rows(ughip_device* dev, ughip_view x, const ughip_slice* router, const ughip_slice* correction, size_t m, size_t k, size_t experts, size_t groups,
                                size_t keep, size_t top, ughip_slice* ids, ughip_slice* weights) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "route_rows: null device");
  if (int rc = route_check(experts, groups, keep, top, "route_rows")) return rc;
  if (k == 0 || k > 0x7fffffffull / experts) return set_error(UGHIP_ERR_INVALID, "route_rows: k %zu", k);
  if (int rc = check_view(dev, x, m, k, UGHIP_F32, "route_rows x")) return rc;
  if (int rc = check_buf(dev, router, experts * k, UGHIP_F32, "route_rows router")) return rc;
  if (correction)
    if (int rc = check_buf(dev, correction, experts, UGHIP_F32, "route_rows correction")) return rc;
  if (int rc = check_buf(dev, ids, m * top, UGHIP_I32, "route_rows ids")) return rc;
  if (int rc = check_buf(dev, weights, m * top, UGHIP_F32, "route_rows weights")) return rc;
  if (m == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  const RouteArgs r{buf_ptr<float>(correction), (int)experts, (int)groups, (int)keep, (int)top};
  const size_t lds = (16 * experts + ROUTE_WAVES * (size_t)route_lds_floats((int)experts, (int)groups)) * sizeof(float);
  const float* xp = view_ptr<float>(x);
  const float* rp = buf_ptr<float>(router);
  const unsigned grid = (unsigned)((m + 15) / 16);
  const bool vec = k % 4 == 0 && x.stride % 4 == 0 && (reinterpret_cast<uintptr_t>(xp) & 15) == 0;
  auto go = [&](auto kernel) {
    if (lds > 64 * 1024)
      if (hipError_t e = hipFuncSetAttribute(reinterpret_cast<const void*>(kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); e != hipSuccess) return e;
    kernel<<<grid, 64 * ROUTE_WAVES, lds, dev->stream>>>(xp, x.stride, rp, r, (int)m, (int)k, static_cast<int*>(ids->ptr), static_cast<float*>(weights->ptr));
    return hipSuccess;
  };
  if (experts <= 16) UGHIP_HIPCHK(vec ? go(route_rows_kernel<true, 1>) : go(route_rows_kernel<false, 1>));
  else UGHIP_HIPCHK(vec ? go(route_rows_kernel<true, 4>) : go(route_rows_kernel<false, 4>));
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_group_rows(ughip_device* dev, const ughip_slice* ids, size_t m, size_t top, size_t experts, ughip_slice* row_index, ughip_slice* slots,
                                ughip_slice* group_end) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "group_rows: null device");
  if (top == 0 || experts == 0 || experts > 16384 || m > 0x7fffffffull / top) return set_error(UGHIP_ERR_INVALID, "group_rows: bad shape");
  if (int rc = check_buf(dev, ids, m * top, UGHIP_I32, "group_rows ids")) return rc;
  if (int rc = check_buf(dev, row_index, m * top, UGHIP_I32, "group_rows row_index")) return rc;
  if (int rc = check_buf(dev, slots, m * top, UGHIP_I32, "group_rows slots")) return rc;
  if (int rc = check_buf(dev, group_end, experts, UGHIP_I32, "group_rows group_end")) return rc;
  if (int rc = device_activate(dev)) return rc;
  group_rows_kernel<<<(unsigned)experts, 256, 0, dev->stream>>>(buf_ptr<int>(ids), (int)(m * top), (int)top, static_cast<int*>(row_index->ptr), static_cast<int*>(slots->ptr),
                                                               static_cast<int*>(group_end->ptr));
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
