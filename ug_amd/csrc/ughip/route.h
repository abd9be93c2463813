// The choice of experts for one row by one wave: shared by the kernel that routes many rows and the one-row step.
#pragma once
#include "layers.h"

namespace ughip {

struct RouteArgs {
  const float* correction;  // may be null
  int experts, groups, keep, top;
};

// LDS one wave needs: the choice scores, the groups' scores and a flag per group.
__host__ __device__ inline int route_lds_floats(int experts, int groups) { return experts + 2 * groups; }
constexpr size_t ROUTE_EXPERTS_MAX = 512;

inline int route_check(size_t experts, size_t groups, size_t keep, size_t top, const char* what) {
  if (experts == 0 || experts > ROUTE_EXPERTS_MAX) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: %zu experts, up to %zu are supported", what, experts, ROUTE_EXPERTS_MAX);
  if (groups == 0 || experts % groups != 0 || keep == 0 || keep > groups || top == 0 || top > keep * (experts / groups))
    return set_error(UGHIP_ERR_INVALID, "%s: %zu of %zu experts in %zu of %zu groups", what, top, experts, keep, groups);
  return UGHIP_OK;
}

// Index of the largest of v[0 .. n) (the lowest among equal ones), the same in every lane; always within the array.
__device__ __forceinline__ int wave_argmax(const float* v, int n) {
  float best = -INFINITY;
  int at = n;
  for (int i = threadIdx.x & 63; i < n; i += 64)
    if (at == n || v[i] > best) best = v[i], at = i;
  for (int d = 32; d; d >>= 1) {
    const float ob = __shfl_xor(best, d, 64);
    const int oa = __shfl_xor(at, d, 64);
    if (oa < n && (at >= n || ob > best || (ob == best && oa < at))) best = ob, at = oa;
  }
  at = __shfl(at, 0, 64);
  return at < n ? at : 0;
}

// One wave; logits [experts] and work (route_lds_floats) in LDS.  LDS operations of one wave complete in order, and nothing
// here is shared with another wave: only the compiler has to be kept from moving them.
__device__ __forceinline__ void route_fence() {
  __builtin_amdgcn_fence(__ATOMIC_ACQ_REL, "workgroup");
  __builtin_amdgcn_wave_barrier();
}
// Up to 64 experts: one per lane.  An expert's place among the chosen is the number of experts in front of it, which every lane
// counts for its own.
__device__ __forceinline__ void route_choose64(const float* logits, const RouteArgs& r, int* ids, float* weights) {
  const int lane = threadIdx.x & 63, size = r.experts / r.groups, E = r.experts;
  const float s = lane < E ? 1.f / (1.f + expf(-logits[lane])) : 0.f;
  float v = lane < E ? s + (r.correction ? r.correction[lane] : 0.f) : -INFINITY;
  const int g = lane / size;
  float a = -INFINITY, b = -INFINITY;
  for (int i = 0; i < size; ++i) {
    const float c = __shfl(v, min(g * size + i, 63), 64);
    b = fmaxf(b, fminf(a, c));
    a = fmaxf(a, c);
  }
  const float score = size > 1 ? a + b : a;
  int front = 0;
  for (int h = 0; h < r.groups; ++h) {
    const float o = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(score), h * size));
    front += o > score || (o == score && h < g);
  }
  if (front >= r.keep) v = -INFINITY;
  front = 0;
  for (int e = 0; e < E; ++e) {
    const float o = __uint_as_float(__builtin_amdgcn_readlane(__float_as_uint(v), e));
    front += o > v || (o == v && e < lane);
  }
  for (int i = lane; i < r.top; i += 64) ids[i] = i, weights[i] = 0.f;  // (scores that are not numbers leave places empty)
  route_fence();
  if (lane < E && front < r.top) ids[front] = lane, weights[front] = s;
  route_fence();
}

__device__ __forceinline__ void route_choose(const float* logits, const RouteArgs& r, float* work, int* ids, float* weights) {
  if (r.experts <= 64) return route_choose64(logits, r, ids, weights);
  const int lane = threadIdx.x & 63, size = r.experts / r.groups;
  float* choice = work;
  float* score = work + r.experts;
  float* kept = score + r.groups;
  for (int e = lane; e < r.experts; e += 64) choice[e] = 1.f / (1.f + expf(-logits[e])) + (r.correction ? r.correction[e] : 0.f);
  route_fence();
  for (int g = lane; g < r.groups; g += 64) {
    float a = choice[g * size], b = -INFINITY;
    for (int i = 1; i < size; ++i) {
      const float c = choice[g * size + i];
      if (c > a) b = a, a = c;
      else if (c > b) b = c;
    }
    score[g] = size > 1 ? a + b : a;
    kept[g] = 0.f;
  }
  route_fence();
  for (int i = 0; i < r.keep; ++i) {
    const int g = wave_argmax(score, r.groups);
    route_fence();
    if (lane == 0) kept[g] = 1.f, score[g] = -INFINITY;
    route_fence();
  }
  for (int e = lane; e < r.experts; e += 64)
    if (kept[e / size] == 0.f) choice[e] = -INFINITY;
  route_fence();
  for (int i = 0; i < r.top; ++i) {
    const int e = wave_argmax(choice, r.experts);
    route_fence();
    if (lane == 0) {
      ids[i] = e;
      weights[i] = 1.f / (1.f + expf(-logits[e]));
      choice[e] = -INFINITY;
    }
    route_fence();
  }
}

}  // namespace ughip
