// Routing of rows to experts (ughip_layers.h): scores on the f32 matrix pipe with the choice in the same kernel, and the
// sort of (row, expert) pairs that the grouped products read.
#include <hip/hip_runtime.h>

#include "layers.h"
#include "route.h"

using namespace ughip;

namespace {

// 16 rows per workgroup.  The four waves share k: each multiplies every fourth run of 16 elements (v_mfma_f32_16x16x4_f32, k
// taken four elements per lane so that rows are read 16 bytes at a time), their partial logits meet in LDS in wave order;
// then each wave chooses for four of the rows.
template <bool VEC>
__global__ void __launch_bounds__(256) route_rows_kernel(const float* __restrict__ x, size_t x_stride, const float* __restrict__ router, RouteArgs r, int m, int k,
                                                         int* __restrict__ ids, float* __restrict__ weights) {
  extern __shared__ float smem[];
  const int E = r.experts, per_wave = route_lds_floats(E, r.groups);
  float* logits = smem;  // [16][E]
  float* work = smem + 16 * E;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6, j = lane & 15, g = lane >> 4;
  const int row0 = blockIdx.x * 16;
  const bool row_ok = row0 + j < m;
  const float* xr = x + (size_t)(row_ok ? row0 + j : row0) * x_stride;
  for (int e0 = 0; e0 < E; e0 += 64) {
    f32x4_t acc[4];
#pragma unroll
    for (int i = 0; i < 4; ++i) acc[i] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    for (int k0 = wave * 16; k0 < k; k0 += 64) {
      const int kk = k0 + 4 * g;
      float xv[4], wv[4];
      if (VEC) {
        const f32x4_t v = row_ok && kk < k ? *reinterpret_cast<const f32x4_t*>(xr + kk) : f32x4_t{0.f, 0.f, 0.f, 0.f};
        xv[0] = v.x, xv[1] = v.y, xv[2] = v.z, xv[3] = v.w;
      } else {
#pragma unroll
        for (int c = 0; c < 4; ++c) xv[c] = row_ok && kk + c < k ? xr[kk + c] : 0.f;
      }
#pragma unroll
      for (int i = 0; i < 4; ++i) {
        if (e0 + 16 * i >= E) continue;  // uniform over the wave
        const int e = e0 + 16 * i + j;
        const float* wr = router + (size_t)(e < E ? e : 0) * k;
        if (VEC) {
          const f32x4_t v = e < E && kk < k ? *reinterpret_cast<const f32x4_t*>(wr + kk) : f32x4_t{0.f, 0.f, 0.f, 0.f};
          wv[0] = v.x, wv[1] = v.y, wv[2] = v.z, wv[3] = v.w;
        } else {
#pragma unroll
          for (int c = 0; c < 4; ++c) wv[c] = e < E && kk + c < k ? wr[kk + c] : 0.f;
        }
#pragma unroll
        for (int c = 0; c < 4; ++c) acc[i] = __builtin_amdgcn_mfma_f32_16x16x4f32(xv[c], wv[c], acc[i], 0, 0, 0);
      }
    }
    for (int wv = 0; wv < 4; ++wv) {
      if (wave == wv) {
#pragma unroll
        for (int i = 0; i < 4; ++i) {
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
  for (int t = 0; t < 4; ++t) {
    const int rr = wave * 4 + t;
    if (row0 + rr >= m) break;  // uniform over the wave
    const size_t at = (size_t)(row0 + rr) * r.top;
    route_choose(logits + rr * E, r, work + wave * per_wave, ids + at, weights + at);
  }
}

// A workgroup (one wave) per expert: it counts the pairs of lower experts and its own, then writes its own in row order.
__global__ void __launch_bounds__(64) group_rows_kernel(const int* __restrict__ ids, int pairs, int top, int* __restrict__ row_index, int* __restrict__ slots,
                                                        int* __restrict__ group_end) {
  const int e = blockIdx.x, lane = threadIdx.x;
  int lower = 0, own = 0;
  for (int p = lane; p < pairs; p += 64) {
    const int id = ids[p];
    lower += id < e;
    own += id == e;
  }
  for (int d = 32; d; d >>= 1) lower += __shfl_xor(lower, d, 64), own += __shfl_xor(own, d, 64);
  if (lane == 0) group_end[e] = lower + own;
  int at = lower;
  for (int p0 = 0; p0 < pairs; p0 += 64) {
    const int p = p0 + lane;
    const bool mine = p < pairs && ids[p] == e;
    const unsigned long long mask = __ballot(mine);
    if (mine) {
      const int r = at + __popcll(mask & ((1ull << lane) - 1));
      row_index[r] = p / top;
      slots[p] = r;
    }
    at += __popcll(mask);
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
  const size_t lds = (16 * experts + 4 * (size_t)route_lds_floats((int)experts, (int)groups)) * sizeof(float);
  const float* xp = view_ptr<float>(x);
  const float* rp = buf_ptr<float>(router);
  const unsigned grid = (unsigned)((m + 15) / 16);
  const bool vec = k % 4 == 0 && x.stride % 4 == 0 && (reinterpret_cast<uintptr_t>(xp) & 15) == 0;
  if (vec) route_rows_kernel<true><<<grid, 256, lds, dev->stream>>>(xp, x.stride, rp, r, (int)m, (int)k, static_cast<int*>(ids->ptr), static_cast<float*>(weights->ptr));
  else route_rows_kernel<false><<<grid, 256, lds, dev->stream>>>(xp, x.stride, rp, r, (int)m, (int)k, static_cast<int*>(ids->ptr), static_cast<float*>(weights->ptr));
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
  group_rows_kernel<<<(unsigned)experts, 64, 0, dev->stream>>>(buf_ptr<int>(ids), (int)(m * top), (int)top, static_cast<int*>(row_index->ptr), static_cast<int*>(slots->ptr),
                                                               static_cast<int*>(group_end->ptr));
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
