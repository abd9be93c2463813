// Shared by the files behind ughip_layers.h: argument checks and small device helpers.
#pragma once
#include <hip/hip_runtime.h>

#include <cstdint>

#include "internal.h"
#include "ughip_layers.h"
#include "wave_ops.h"

namespace ughip {

typedef float f32x4_t __attribute__((ext_vector_type(4)));
typedef unsigned u32x4_t __attribute__((ext_vector_type(4)));

// m rows of n elements of `s`, row i at offset + i * stride; dtype < 0: any.
inline int check_view(const ughip_device* dev, const ughip_view& v, size_t m, size_t n, int dtype, const char* what) {
  if (!v.s) return set_error(UGHIP_ERR_INVALID, "%s: null slice", what);
  if (v.s->dev != dev) return set_error(UGHIP_ERR_INVALID, "%s: slice lives on another device", what);
  if (dtype >= 0 && v.s->dtype != dtype) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: dtype %s, expected %s", what, dtype_name(v.s->dtype), dtype_name(dtype));
  if (m == 0 || n == 0) return UGHIP_OK;
  if (m > 0x7fffffffull || n > 0x7fffffffull || v.stride > 0x7fffffffull) return set_error(UGHIP_ERR_INVALID, "%s: shape too large", what);
  if (m > 1 && v.stride < n) return set_error(UGHIP_ERR_INVALID, "%s: rows of %zu elements %zu apart overlap", what, n, v.stride);
  if (v.offset > v.s->len || (m - 1) * v.stride + n > v.s->len - v.offset)
    return set_error(UGHIP_ERR_BOUNDS, "%s: slice has %zu elements, rows reach %zu", what, v.s->len, v.offset + (m - 1) * v.stride + n);
  return UGHIP_OK;
}
inline int check_buf(const ughip_device* dev, const ughip_slice* s, size_t n, int dtype, const char* what) {
  ughip_view v{const_cast<ughip_slice*>(s), 0, n};
  return check_view(dev, v, 1, n, dtype, what);
}
template <typename T>
inline T* view_ptr(const ughip_view& v) {
  return v.s ? static_cast<T*>(v.s->ptr) + v.offset : nullptr;
}
template <typename T>
inline const T* buf_ptr(const ughip_slice* s) {
  return s ? static_cast<const T*>(s->ptr) : nullptr;
}

__device__ __forceinline__ float bf16_to_f32(uint16_t v) { return __uint_as_float((uint32_t)v << 16); }
// z / (1 + exp(-z)) with the exponential as a power of two and a reciprocal: a few units of the last place
__device__ __forceinline__ float silu_f(float z) { return z * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }
__device__ __forceinline__ float softplus_f(float z) { return z > 20.f ? z + log1pf(expf(-z)) : log1pf(expf(z)); }
__device__ __forceinline__ float gelu_tanh_f(float z) {
  return 0.5f * z * (1.f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z)));
}

// A gated linear unit: gate * sigmoid(alpha gate) * (up + shift), the gate cut off above `limit`, up on both sides (limit <= 0:
// neither).  alpha = 1, shift = 0 without a limit is SwiGLU.
struct GluForm {
  float alpha = 1.f, shift = 0.f, limit = 0.f;
};
__device__ __forceinline__ float glu_f(float gate, float up, const GluForm& f) {
  if (f.limit > 0.f) {  // the same for every thread of a launch
    gate = gate > f.limit ? f.limit : gate;  // (a NaN stays one)
    up = up > f.limit ? f.limit : up < -f.limit ? -f.limit : up;
  }
  return gate * __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * f.alpha * gate)) * (up + f.shift);
}
// What ughip_product and ughip_row_step say of it.
inline GluForm glu_form(int act, float alpha, float shift, float limit) {
  GluForm f;
  if (act == UGHIP_ACT_GLU) f.alpha = alpha, f.shift = shift, f.limit = limit;
  return f;
}
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.f + __builtin_amdgcn_exp2f(-1.4426950408889634f * z)); }

// The sum over a workgroup of 64 * WAVES threads, the same value in every thread; `red` holds WAVES floats and is free to
// be used again after the next barrier of the caller.
template <int WAVES>
__device__ __forceinline__ float block_sum(float v, float* red) {
  v = wave_sum(v);
  if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
  __syncthreads();
  float s = 0.f;
#pragma unroll
  for (int i = 0; i < WAVES; ++i) s += red[i];
  return s;
}

}  // namespace ughip
