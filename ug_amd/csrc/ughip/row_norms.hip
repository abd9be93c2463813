// Lookups and RMS norms over rows (ughip_layers.h): a workgroup per row (or per part of a row), the row in LDS between the
// pass that sums its squares and the pass that scales it.
#include <hip/hip_runtime.h>

#include "bf16_split.h"
#include "layers.h"

using namespace ughip;

namespace {

// An element of a result that is F32 or BF16.
__device__ __forceinline__ void put(void* dst, bool bf16, size_t at, float v) {
  if (bf16) static_cast<uint16_t*>(dst)[at] = bf16_rne(v);
  else static_cast<float*>(dst)[at] = v;
}

template <typename T>
__global__ void __launch_bounds__(256) gather_rows_kernel(const T* __restrict__ table, int table_rows, size_t stride, size_t col, int cols, const int* __restrict__ ids,
                                                          void* __restrict__ dst, size_t dst_stride, bool dst_bf16) {
  const int row = blockIdx.y, id = ids[row];
  const int c = blockIdx.x * 256 + threadIdx.x;
  if (c >= cols) return;
  float v = __uint_as_float(0x7fc00000u);
  if (id >= 0 && id < table_rows) {
    const T e = table[(size_t)id * stride + col + c];
    if constexpr (sizeof(T) == 2) v = bf16_to_f32(e);
    else v = e;
  }
  put(dst, dst_bf16, (size_t)row * dst_stride + c, v);
}

struct AddNormArgs {
  const float* x;
  const float* y;
  const float* w;
  void* dst;
  void* copy;
  const float* extra;
  const float* next;
  size_t x_stride, y_stride, dst_stride, extra_stride;
  const int* slots;
  const float* weights;
  int top, y_rows, n;
  float eps;
  bool dst_bf16, copy_bf16;
};

__global__ void __launch_bounds__(256) add_rms_norm_kernel(AddNormArgs a) {
  extern __shared__ float row[];
  __shared__ float red[2][4];
  const size_t i = blockIdx.x;
  float ss = 0.f;
  if (!a.y) {
    for (int c = threadIdx.x; c < a.n; c += 256) row[c] = 0.f;
  } else if (a.slots) {
    for (int c = threadIdx.x; c < a.n; c += 256) {
      float v = 0.f;
      for (int j = 0; j < a.top; ++j) {
        const int r = a.slots[i * a.top + j];
        if (r >= 0 && r < a.y_rows) v += a.weights[i * a.top + j] * a.y[(size_t)r * a.y_stride + c];
      }
      row[c] = v;
      ss += v * v;
    }
  } else {
    for (int c = threadIdx.x; c < a.n; c += 256) {
      const float v = a.y[i * a.y_stride + c];
      row[c] = v;
      ss += v * v;
    }
  }
  ss = block_sum<4>(ss, red[0]);
  const float inv = 1.f / sqrtf(ss / (float)a.n + a.eps);
  ss = 0.f;
  for (int c = threadIdx.x; c < a.n; c += 256) {
    float v = a.y ? row[c] * inv * a.w[c] : 0.f;  // every thread reads back its own elements
    if (a.x) v += a.x[i * a.x_stride + c];
    if (a.extra) v += a.extra[i * a.extra_stride + c];
    put(a.dst, a.dst_bf16, i * a.dst_stride + c, v);
    if (a.next) row[c] = v, ss += v * v;
    else if (a.copy) put(a.copy, a.copy_bf16, i * a.n + c, v);
  }
  if (!a.next) return;
  ss = block_sum<4>(ss, red[1]);
  const float inv2 = 1.f / sqrtf(ss / (float)a.n + a.eps);
  for (int c = threadIdx.x; c < a.n; c += 256) put(a.copy, a.copy_bf16, i * a.n + c, row[c] * inv2 * a.next[c]);
}

// The same without routed rows for up to 4096 elements, a multiple of 4, held in registers.
__global__ void __launch_bounds__(256) add_rms_norm4_kernel(AddNormArgs a) {
  __shared__ float red[2][4];
  const size_t i = blockIdx.x;
  f32x4_t v[4], x[4], e[4];
  const f32x4_t zero = {0.f, 0.f, 0.f, 0.f};
  float ss = 0.f;
  auto square = [](const f32x4_t& q) { return q.x * q.x + q.y * q.y + q.z * q.z + q.w * q.w; };
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int c = (u * 256 + (int)threadIdx.x) * 4;
    const bool ok = c < a.n;
    v[u] = ok && a.y ? *reinterpret_cast<const f32x4_t*>(a.y + i * a.y_stride + c) : zero;
    x[u] = ok && a.x ? *reinterpret_cast<const f32x4_t*>(a.x + i * a.x_stride + c) : zero;
    e[u] = ok && a.extra ? *reinterpret_cast<const f32x4_t*>(a.extra + i * a.extra_stride + c) : zero;
  }
#pragma unroll
  for (int u = 0; u < 4; ++u) ss += square(v[u]);
  ss = block_sum<4>(ss, red[0]);
  const float inv = 1.f / sqrtf(ss / (float)a.n + a.eps);
  auto put4 = [](void* dst, bool bf16, size_t at, const f32x4_t& q) {
    if (bf16) *reinterpret_cast<ushort4*>(static_cast<uint16_t*>(dst) + at) = make_ushort4(bf16_rne(q.x), bf16_rne(q.y), bf16_rne(q.z), bf16_rne(q.w));
    else *reinterpret_cast<f32x4_t*>(static_cast<float*>(dst) + at) = q;
  };
  ss = 0.f;
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int c = (u * 256 + (int)threadIdx.x) * 4;
    if (c >= a.n) continue;
    if (a.y) v[u] = v[u] * inv * *reinterpret_cast<const f32x4_t*>(a.w + c) + x[u] + e[u];
    else v[u] = x[u] + e[u];
    put4(a.dst, a.dst_bf16, i * a.dst_stride + c, v[u]);
    if (a.copy && !a.next) put4(a.copy, a.copy_bf16, i * a.n + c, v[u]);
    ss += square(v[u]);
  }
  if (!a.next) return;
  ss = block_sum<4>(ss, red[1]);
  const float inv2 = 1.f / sqrtf(ss / (float)a.n + a.eps);
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int c = (u * 256 + (int)threadIdx.x) * 4;
    if (c < a.n) put4(a.copy, a.copy_bf16, i * a.n + c, v[u] * inv2 * *reinterpret_cast<const f32x4_t*>(a.next + c));
  }
}

__global__ void __launch_bounds__(256) gated_rms_norm_kernel(const float* __restrict__ y, size_t y_stride, const float* __restrict__ z, size_t z_stride,
                                                             const float* __restrict__ w, float eps, void* __restrict__ dst, size_t dst_stride, bool dst_bf16, int part) {
  extern __shared__ float row[];
  __shared__ float red[4];
  const size_t i = blockIdx.x, c0 = (size_t)blockIdx.y * part;
  float ss = 0.f;
  for (int c = threadIdx.x; c < part; c += 256) {
    float g = y[i * y_stride + c0 + c];
    if (z) g *= silu_f(z[i * z_stride + c0 + c]);
    row[c] = g;
    ss += g * g;
  }
  ss = block_sum<4>(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
  for (int c = threadIdx.x; c < part; c += 256) put(dst, dst_bf16, i * dst_stride + c0 + c, row[c] * inv * w[c0 + c]);
}

// Checks a result that may be F32 or BF16; *at: its first element.
int check_result(const ughip_device* dev, const ughip_view& v, size_t m, size_t n, const char* what, void** at, bool* bf16) {
  if (int rc = check_view(dev, v, m, n, -1, what)) return rc;
  if (v.s->dtype != UGHIP_F32 && v.s->dtype != UGHIP_BF16) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: dtype %s, F32 or BF16 expected", what, dtype_name(v.s->dtype));
  *bf16 = v.s->dtype == UGHIP_BF16;
  *at = static_cast<char*>(v.s->ptr) + v.offset * (*bf16 ? 2 : 4);
  return UGHIP_OK;
}

// The same for parts of up to 4096 elements, a multiple of 4, held in registers.
__global__ void __launch_bounds__(256) gated_rms_norm4_kernel(const float* __restrict__ y, size_t y_stride, const float* __restrict__ z, size_t z_stride,
                                                              const float* __restrict__ w, float eps, void* __restrict__ dst, size_t dst_stride, bool dst_bf16, int part) {
  __shared__ float red[4];
  const size_t i = blockIdx.x, c0 = (size_t)blockIdx.y * part;
  f32x4_t g[4];
  float ss = 0.f;
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int c = (u * 256 + (int)threadIdx.x) * 4;
    g[u] = f32x4_t{0.f, 0.f, 0.f, 0.f};
    if (c >= part) continue;
    g[u] = *reinterpret_cast<const f32x4_t*>(y + i * y_stride + c0 + c);
    if (z) {
      const f32x4_t q = *reinterpret_cast<const f32x4_t*>(z + i * z_stride + c0 + c);
#pragma unroll
      for (int e = 0; e < 4; ++e) g[u][e] *= silu_f(q[e]);
    }
    ss += g[u].x * g[u].x + g[u].y * g[u].y + g[u].z * g[u].z + g[u].w * g[u].w;
  }
  ss = block_sum<4>(ss, red);
  const float inv = 1.f / sqrtf(ss / (float)part + eps);
#pragma unroll
  for (int u = 0; u < 4; ++u) {
    const int c = (u * 256 + (int)threadIdx.x) * 4;
    if (c >= part) continue;
    const f32x4_t v = g[u] * inv * *reinterpret_cast<const f32x4_t*>(w + c0 + c);
    const size_t at = i * dst_stride + c0 + c;
    if (dst_bf16) *reinterpret_cast<ushort4*>(static_cast<uint16_t*>(dst) + at) = make_ushort4(bf16_rne(v.x), bf16_rne(v.y), bf16_rne(v.z), bf16_rne(v.w));
    else *reinterpret_cast<f32x4_t*>(static_cast<float*>(dst) + at) = v;
  }
}

constexpr size_t ROW_MAX = 16000;  // the row and the reduction fit the 64 KiB a launch gets without asking

}  // namespace

extern "C" int ughip_gather_rows(ughip_device* dev, const ughip_slice* table, size_t table_rows, size_t stride, size_t col, size_t cols, const ughip_slice* ids, size_t m,
                                 ughip_view dst) {
  if (!dev || !table) return set_error(UGHIP_ERR_INVALID, "gather_rows: null argument");
  if (table->dtype != UGHIP_F32 && table->dtype != UGHIP_BF16) return set_error(UGHIP_ERR_UNSUPPORTED, "gather_rows: a table is F32 or BF16");
  if (int rc = check_view(dev, ughip_view{const_cast<ughip_slice*>(table), 0, stride}, table_rows, stride, -1, "gather_rows table")) return rc;
  if (col > stride || cols > stride - col) return set_error(UGHIP_ERR_BOUNDS, "gather_rows: columns %zu + %zu of rows of %zu", col, cols, stride);
  if (int rc = check_buf(dev, ids, m, UGHIP_I32, "gather_rows ids")) return rc;
  void* d;
  bool bf16;
  if (int rc = check_result(dev, dst, m, cols, "gather_rows dst", &d, &bf16)) return rc;
  if (m == 0 || cols == 0) return UGHIP_OK;
  if (m > 65535) return set_error(UGHIP_ERR_UNSUPPORTED, "gather_rows: up to 65535 rows");
  if (int rc = device_activate(dev)) return rc;
  const dim3 grid((unsigned)((cols + 255) / 256), (unsigned)m);
  if (table->dtype == UGHIP_F32)
    gather_rows_kernel<float><<<grid, 256, 0, dev->stream>>>(buf_ptr<float>(table), (int)table_rows, stride, col, (int)cols, buf_ptr<int>(ids), d, dst.stride, bf16);
  else
    gather_rows_kernel<uint16_t><<<grid, 256, 0, dev->stream>>>(buf_ptr<uint16_t>(table), (int)table_rows, stride, col, (int)cols, buf_ptr<int>(ids), d, dst.stride, bf16);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_add_rms_norm_rows(ughip_device* dev, ughip_view x, ughip_view y, const ughip_slice* slots, const ughip_slice* weights, size_t top, size_t y_rows,
                                       const ughip_slice* w, float eps, ughip_view extra, ughip_view dst, const ughip_slice* next, ughip_slice* copy, size_t m, size_t n) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "add_rms_norm_rows: null device");
  if (n > ROW_MAX) return set_error(UGHIP_ERR_UNSUPPORTED, "add_rms_norm_rows: rows of %zu elements, up to %zu are supported", n, ROW_MAX);
  if (x.s)
    if (int rc = check_view(dev, x, m, n, UGHIP_F32, "add_rms_norm_rows x")) return rc;
  if (y.s)
    if (int rc = check_view(dev, y, slots ? y_rows : m, n, UGHIP_F32, "add_rms_norm_rows y")) return rc;
  if (extra.s)
    if (int rc = check_view(dev, extra, m, n, UGHIP_F32, "add_rms_norm_rows extra")) return rc;
  if (!y.s && (!x.s || slots)) return set_error(UGHIP_ERR_INVALID, "add_rms_norm_rows: neither rows to norm nor rows to add to");
  if (slots) {
    if (top == 0 || top > 4096) return set_error(UGHIP_ERR_INVALID, "add_rms_norm_rows: top %zu", top);
    if (int rc = check_buf(dev, slots, m * top, UGHIP_I32, "add_rms_norm_rows slots")) return rc;
    if (int rc = check_buf(dev, weights, m * top, UGHIP_F32, "add_rms_norm_rows weights")) return rc;
  }
  if (y.s)
    if (int rc = check_buf(dev, w, n, UGHIP_F32, "add_rms_norm_rows w")) return rc;
  if (next) {
    if (!copy) return set_error(UGHIP_ERR_INVALID, "add_rms_norm_rows: a second norm without a place for it");
    if (int rc = check_buf(dev, next, n, UGHIP_F32, "add_rms_norm_rows next")) return rc;
  }
  void* d;
  bool bf16;
  if (int rc = check_result(dev, dst, m, n, "add_rms_norm_rows dst", &d, &bf16)) return rc;
  void* copy_at = nullptr;
  bool copy_bf16 = false;
  if (copy)
    if (int rc = check_result(dev, ughip_view{copy, 0, n}, m, n, "add_rms_norm_rows copy", &copy_at, &copy_bf16)) return rc;
  if (m == 0 || n == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  AddNormArgs a{view_ptr<float>(x), view_ptr<float>(y), buf_ptr<float>(w), d, copy_at, view_ptr<float>(extra), buf_ptr<float>(next), x.stride, y.stride, dst.stride, extra.stride,
                buf_ptr<int>(slots), buf_ptr<float>(weights), (int)top, (int)y_rows, (int)n, eps, bf16, copy_bf16};
  auto rows4 = [](const void* q, size_t stride) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0 && (!q || stride % 4 == 0); };
  if (!slots && n % 4 == 0 && n <= 4096 && rows4(a.x, a.x_stride) && rows4(a.y, a.y_stride) && rows4(a.extra, a.extra_stride) && rows4(d, a.dst_stride)) {
    add_rms_norm4_kernel<<<(unsigned)m, 256, 0, dev->stream>>>(a);
    UGHIP_HIPCHK(hipGetLastError());
    return UGHIP_OK;
  }
  add_rms_norm_kernel<<<(unsigned)m, 256, n * sizeof(float), dev->stream>>>(a);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}

extern "C" int ughip_gated_rms_norm_rows(ughip_device* dev, ughip_view y, ughip_view z, const ughip_slice* w, float eps, size_t groups, ughip_view dst, size_t m, size_t n) {
  if (!dev) return set_error(UGHIP_ERR_INVALID, "gated_rms_norm_rows: null device");
  if (groups == 0 || n % groups != 0 || groups > 65535) return set_error(UGHIP_ERR_INVALID, "gated_rms_norm_rows: %zu elements in %zu groups", n, groups);
  if (n / groups > ROW_MAX) return set_error(UGHIP_ERR_UNSUPPORTED, "gated_rms_norm_rows: groups of up to %zu elements", ROW_MAX);
  if (int rc = check_view(dev, y, m, n, UGHIP_F32, "gated_rms_norm_rows y")) return rc;
  if (z.s)
    if (int rc = check_view(dev, z, m, n, UGHIP_F32, "gated_rms_norm_rows z")) return rc;
  if (int rc = check_buf(dev, w, n, UGHIP_F32, "gated_rms_norm_rows w")) return rc;
  void* d;
  bool bf16;
  if (int rc = check_result(dev, dst, m, n, "gated_rms_norm_rows dst", &d, &bf16)) return rc;
  if (m == 0 || n == 0) return UGHIP_OK;
  if (int rc = device_activate(dev)) return rc;
  const size_t part = n / groups;
  auto a16 = [](const void* q) { return (reinterpret_cast<uintptr_t>(q) & 15) == 0; };
  if (part % 4 == 0 && part <= 4096 && y.stride % 4 == 0 && (!z.s || z.stride % 4 == 0) && dst.stride % 4 == 0 && a16(view_ptr<float>(y)) && a16(view_ptr<float>(z)) && a16(d)) {
    gated_rms_norm4_kernel<<<dim3((unsigned)m, (unsigned)groups), 256, 0, dev->stream>>>(view_ptr<float>(y), y.stride, view_ptr<float>(z), z.stride, buf_ptr<float>(w), eps, d,
                                                                                         dst.stride, bf16, (int)part);
    UGHIP_HIPCHK(hipGetLastError());
    return UGHIP_OK;
  }
  gated_rms_norm_kernel<<<dim3((unsigned)m, (unsigned)groups), 256, part * sizeof(float), dev->stream>>>(view_ptr<float>(y), y.stride, view_ptr<float>(z), z.stride,
                                                                                                        buf_ptr<float>(w), eps, d, dst.stride, bf16, (int)part);
  UGHIP_HIPCHK(hipGetLastError());
  return UGHIP_OK;
}
