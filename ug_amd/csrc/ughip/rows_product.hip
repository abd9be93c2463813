// Products of rows of any size with their neighbours folded in (ughip_product_rows): y = x w^T for m >= 1 rows, any n and k,
// x / w / result as F32 or BF16, bias, SwiGLU or gated-lookup epilogues, and the grouped form (rows sorted by expert, a
// matrix per group, rows of x gathered on their way in).
//
// A workgroup of four waves (2 x 2) takes a 64 MI x 64 NI tile.  A K step is 128 bytes of every row in LDS (256 for the smallest
// tile), in 16-byte chunks; rows are 16 bytes further apart than they are long, which spreads the 16-byte reads of consecutive
// rows over all banks.  Two LDS buffers: while one step is multiplied the next ones' elements are in flight to registers.  Whatever type
// the operands are stored in, they are converted between registers and LDS; the products are v_mfma_f32_32x32x16_bf16 or, for
// F32, four v_mfma_f32_32x32x2_f32 per chunk (k taken chunk by chunk: lanes 0-31 the even, lanes 32-63 the odd one).
#include <hip/hip_runtime.h>

#include "bf16_split.h"
#include "gemm.h"
#include "layers.h"

using namespace ughip;

namespace {

typedef float f32x16 __attribute__((ext_vector_type(16)));
typedef float f32x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x8 __attribute__((ext_vector_type(8)));
typedef __bf16 bf16x4 __attribute__((ext_vector_type(4)));

struct ProductArgs {
  const void* x;
  const void* w;
  const float* bias;
  void* dst;
  size_t x_stride, w_stride, dst_stride, w_group;  // elements; w_group: from one group's matrix to the next
  int m, n, k;
  bool dst_bf16;
  const void* table;
  const int* ids;
  size_t table_stride, table_col;
  int table_rows;
  bool table_bf16;
  const int* row_index;
  const int* group_end;
  int groups, x_rows;
  GluForm glu;
};

// One 16-byte LDS chunk's worth of a row, as it is stored: 8 elements for bf16 products, 4 for f32 ones.
template <typename CT, typename ST>
struct Raw;
template <>
struct Raw<__bf16, float> {
  f32x4_t a, b;
  bool ok;
  __device__ u32x4_t pack() const {
    if (!ok) return u32x4_t{0, 0, 0, 0};
    const f32x8 v = {a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w};
    return __builtin_bit_cast(u32x4_t, __builtin_convertvector(v, bf16x8));
  }
};
template <>
struct Raw<__bf16, uint16_t> {
  u32x4_t a;
  bool ok;
  __device__ u32x4_t pack() const { return ok ? a : u32x4_t{0, 0, 0, 0}; }
};
template <>
struct Raw<float, float> {
  f32x4_t a;
  bool ok;
  __device__ u32x4_t pack() const { return ok ? __builtin_bit_cast(u32x4_t, a) : u32x4_t{0, 0, 0, 0}; }
};

template <typename CT, typename ST, bool VEC>
__device__ __forceinline__ Raw<CT, ST> load_chunk(const ST* row, int k0, int k, bool ok) {
  constexpr int E = sizeof(CT) == 2 ? 8 : 4;
  Raw<CT, ST> r;
  if constexpr (VEC) {
    // k is a multiple of 8 and rows are 16-byte aligned: a chunk is inside or outside as a whole.  Every lane loads (its row's
    // first elements where there is nothing of its own; pack() makes that zeros): with branches around loads the compiler waits for
    // all of them at once.
    r.ok = ok && k0 < k;
    const ST* p = row + (k0 < k ? k0 : 0);
    if constexpr (sizeof(ST) == 4) {
      r.a = *reinterpret_cast<const f32x4_t*>(p);
      if constexpr (sizeof(CT) == 2) r.b = *reinterpret_cast<const f32x4_t*>(p + 4);
    } else {
      r.a = *reinterpret_cast<const u32x4_t*>(p);
    }
  } else {
    ST v[E];
    r.ok = true;
#pragma unroll
    for (int i = 0; i < E; ++i) v[i] = ok && k0 + i < k ? row[k0 + i] : ST(0);
    if constexpr (sizeof(CT) == 2 && sizeof(ST) == 4) {
      r.a = f32x4_t{v[0], v[1], v[2], v[3]};
      r.b = f32x4_t{v[4], v[5], v[6], v[7]};
    } else if constexpr (sizeof(ST) == 4) {
      r.a = f32x4_t{v[0], v[1], v[2], v[3]};
    } else {
      r.a = u32x4_t{v[0] | (uint32_t)v[1] << 16, v[2] | (uint32_t)v[3] << 16, v[4] | (uint32_t)v[5] << 16, v[6] | (uint32_t)v[7] << 16};
    }
  }
  return r;
}

template <typename CT>
__device__ __forceinline__ void mfma_chunk(const u32x4_t& a, const u32x4_t& b, f32x16& acc) {
  if constexpr (sizeof(CT) == 2) {
    acc = __builtin_amdgcn_mfma_f32_32x32x16_bf16(__builtin_bit_cast(bf16x8, a), __builtin_bit_cast(bf16x8, b), acc, 0, 0, 0);
  } else {
    const f32x4_t fa = __builtin_bit_cast(f32x4_t, a), fb = __builtin_bit_cast(f32x4_t, b);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(fa.x, fb.x, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(fa.y, fb.y, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(fa.z, fb.z, acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_32x32x2f32(fa.w, fb.w, acc, 0, 0, 0);
  }
}

template <typename CT, typename XT, typename WT, int MI, int NI, int ACT, bool VEC>
__global__ void __launch_bounds__(256) rows_product_kernel(ProductArgs a) {
  constexpr int BM = 64 * MI, BN = 64 * NI;
  // 16-byte chunks of a row per K step (the small tile's steps are twice as long: it has little to do between two barriers), rows in
  // LDS 16 bytes further apart than they are long, rows a pass of the workgroup covers
  constexpr int CHUNKS = MI * NI == 1 ? 16 : 8, ROW_BYTES = CHUNKS * 16 + 16, CSH = CHUNKS == 16 ? 4 : 3, RP = 256 / CHUNKS;
  constexpr int XC = BM / RP, WC = BN / RP, CE = sizeof(CT) == 2 ? 8 : 4, KE = CHUNKS * CE;
  constexpr int COLS = ACT == UGHIP_ACT_SWIGLU ? BN / 2 : BN;  // result columns of a tile
  __shared__ __attribute__((aligned(16))) char lds[2][(BM + BN) * ROW_BYTES];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, wm = wave >> 1, wn = wave & 1;
  const int n0 = blockIdx.x * COLS;
  int m0 = blockIdx.y * BM, m_end = a.m, group = 0;
  if (a.groups) {
    // which group this tile of rows belongs to: groups take ceil(rows / BM) tiles each, in order
    int tile = blockIdx.y, begin = 0;
    bool found = false;
    for (int g = 0; g < a.groups; ++g) {
      int end = a.group_end[g];
      end = end < begin ? begin : end > a.m ? a.m : end;
      const int tiles = (end - begin + BM - 1) / BM;
      if (tile < tiles) {
        group = g, m0 = begin + tile * BM, m_end = end, found = true;
        break;
      }
      tile -= tiles;
      begin = end;
    }
    if (!found) return;  // the same for the whole workgroup
  }
  const XT* xrow[XC];
  bool xok[XC];
  const WT* wrow[WC];
  bool wok[WC];
#pragma unroll
  for (int i = 0; i < XC; ++i) {
    const int r = m0 + (tid >> CSH) + RP * i;
    xok[i] = r < m_end;
    int src = xok[i] ? r : 0;
    if (a.row_index && xok[i]) {
      src = a.row_index[r];
      xok[i] = src >= 0 && src < a.x_rows;
      if (!xok[i]) src = 0;
    }
    xrow[i] = static_cast<const XT*>(a.x) + (size_t)src * a.x_stride;
  }
#pragma unroll
  for (int i = 0; i < WC; ++i) {
    const int rb = (tid >> CSH) + RP * i;
    int col, up = 0;
    if (ACT == UGHIP_ACT_SWIGLU) {  // LDS rows: 32 gate columns, the same 32 of up, the next 32 gate columns, ...
      col = n0 + (rb >> 6) * 32 + (rb & 31);
      up = rb & 32 ? a.n : 0;
    } else {
      col = n0 + rb;
    }
    wok[i] = col < a.n;
    wrow[i] = static_cast<const WT*>(a.w) + (size_t)group * a.w_group + (size_t)(wok[i] ? up + col : 0) * a.w_stride;
  }
  f32x16 acc[MI][NI];
#pragma unroll
  for (int i = 0; i < MI; ++i)
#pragma unroll
    for (int j = 0; j < NI; ++j)
#pragma unroll
      for (int e = 0; e < 16; ++e) acc[i][j][e] = 0.f;

  // steps on their way in registers: the small tile's are short, one would not cover the way from memory
  constexpr int DEPTH = MI * NI == 1 ? 2 : 1;
  Raw<CT, XT> xr[DEPTH][XC];
  Raw<CT, WT> wr[DEPTH][WC];
  const int ck = (tid & (CHUNKS - 1)) * CE;
  auto fetch = [&](int d, int k0) {
#pragma unroll
    for (int i = 0; i < XC; ++i) xr[d][i] = load_chunk<CT, XT, VEC>(xrow[i], k0 + ck, a.k, xok[i]);
#pragma unroll
    for (int i = 0; i < WC; ++i) wr[d][i] = load_chunk<CT, WT, VEC>(wrow[i], k0 + ck, a.k, wok[i]);
  };
  const int steps = (a.k + KE - 1) / KE;
  // element e of an accumulator: row 8 (e / 4) + 4 (lane / 32) + e % 4, column lane % 32
  auto row_of = [&](int i, int e) { return m0 + wm * 32 * MI + i * 32 + 8 * (e >> 2) + 4 * (lane >> 5) + (e & 3); };
  // what the gates of the rows multiply, asked for here so that the way to the table's scattered rows is over by the end: the rows'
  // tokens first, then all of their table elements
  constexpr bool GATE = ACT == UGHIP_ACT_GELU_MUL;
  int id[GATE ? MI : 1][16];
  uint32_t factor[GATE ? MI : 1][16][NI];  // bits
  bool there[GATE ? MI : 1][16];
  if constexpr (GATE) {
#pragma unroll
    for (int i = 0; i < MI; ++i)
#pragma unroll
      for (int e = 0; e < 16; ++e) id[i][e] = a.ids[min(row_of(i, e), a.m - 1)];
  }
#pragma unroll
  for (int d = 0; d < DEPTH; ++d) fetch(d, d * KE);  // (past the end: zeros)
  if constexpr (GATE) {
    auto ask = [&](auto* table) {  // (one branch on the table's type around all of the loads)
#pragma unroll
      for (int i = 0; i < MI; ++i)
#pragma unroll
        for (int e = 0; e < 16; ++e)
#pragma unroll
          for (int j = 0; j < NI; ++j) {
            there[i][e] = id[i][e] >= 0 && id[i][e] < a.table_rows;
            const size_t at = (size_t)(there[i][e] ? id[i][e] : 0) * a.table_stride + a.table_col + min(n0 + wn * 32 * NI + j * 32 + (lane & 31), a.n - 1);
            factor[i][e][j] = table[at];
          }
    };
    if (a.table_bf16) ask(static_cast<const uint16_t*>(a.table));
    else ask(static_cast<const uint32_t*>(a.table));
  }
  for (int s0 = 0; s0 < steps; s0 += DEPTH)
#pragma unroll
   for (int d = 0; d < DEPTH; ++d) {
    const int s = s0 + d;
    if (s >= steps) break;
    char* buf = lds[s & 1];
#pragma unroll
    for (int i = 0; i < XC; ++i) *reinterpret_cast<u32x4_t*>(buf + ((tid >> CSH) + RP * i) * ROW_BYTES + (tid & (CHUNKS - 1)) * 16) = xr[d][i].pack();
#pragma unroll
    for (int i = 0; i < WC; ++i) *reinterpret_cast<u32x4_t*>(buf + (BM + (tid >> CSH) + RP * i) * ROW_BYTES + (tid & (CHUNKS - 1)) * 16) = wr[d][i].pack();
    if (DEPTH > 1 || s + 1 < steps) fetch(d, (s + DEPTH) * KE);  // (without a branch, so that the next step's loads can be waited for alone)
    __syncthreads();  // (one barrier a step: the buffer written two steps from now is read before the next barrier)
    const char* xa = buf + (wm * 32 * MI + (lane & 31)) * ROW_BYTES + (lane >> 5) * 16;
    const char* wa = buf + (BM + wn * 32 * NI + (lane & 31)) * ROW_BYTES + (lane >> 5) * 16;
    // fragments of BATCH pairs of chunks at once: a small tile's products do not cover the way from LDS one by one
    constexpr int BATCH = MI * NI == 1 ? CHUNKS / 4 : 1;
#pragma unroll
    for (int c0 = 0; c0 < CHUNKS / 2; c0 += BATCH) {
      u32x4_t fx[BATCH][MI], fw[BATCH][NI];
#pragma unroll
      for (int c = 0; c < BATCH; ++c) {
#pragma unroll
        for (int i = 0; i < MI; ++i) fx[c][i] = *reinterpret_cast<const u32x4_t*>(xa + i * 32 * ROW_BYTES + (c0 + c) * 32);
#pragma unroll
        for (int j = 0; j < NI; ++j) fw[c][j] = *reinterpret_cast<const u32x4_t*>(wa + j * 32 * ROW_BYTES + (c0 + c) * 32);
      }
#pragma unroll
      for (int c = 0; c < BATCH; ++c)
#pragma unroll
        for (int i = 0; i < MI; ++i)
#pragma unroll
          for (int j = 0; j < NI; ++j) mfma_chunk<CT>(fx[c][i], fw[c][j], acc[i][j]);
    }
   }

#pragma unroll
  for (int i = 0; i < MI; ++i) {
#pragma unroll
    for (int e = 0; e < 16; ++e) {
      const int r = row_of(i, e);
      if (r >= m_end) continue;
#pragma unroll
      for (int j = 0; j < (ACT == UGHIP_ACT_SWIGLU ? 1 : NI); ++j) {
        const int col = ACT == UGHIP_ACT_SWIGLU ? n0 + wn * 32 + (lane & 31) : n0 + wn * 32 * NI + j * 32 + (lane & 31);
        if (col >= a.n) continue;
        float v = acc[i][j][e];
        if (a.bias) v += a.bias[col];
        if constexpr (ACT == UGHIP_ACT_SWIGLU) {
          float u = acc[i][1][e];
          if (a.bias) u += a.bias[a.n + col];
          v = glu_f(v, u, a.glu);
        }
        if constexpr (ACT == UGHIP_ACT_GELU_MUL) v = gelu_tanh_f(v) * __uint_as_float(!there[i][e] ? 0x7fc00000u : a.table_bf16 ? factor[i][e][j] << 16 : factor[i][e][j]);
        const size_t at = (size_t)r * a.dst_stride + col;
        if (a.dst_bf16) static_cast<uint16_t*>(a.dst)[at] = bf16_rne(v);
        else static_cast<float*>(a.dst)[at] = v;
      }
    }
  }
}

template <typename CT, typename XT, typename WT, int MI, int NI, int ACT>
hipError_t launch_tile(hipStream_t st, const ProductArgs& a, bool vec) {
  constexpr int BM = 64 * MI, COLS = ACT == UGHIP_ACT_SWIGLU ? 32 * NI : 64 * NI;
  const dim3 grid((unsigned)((a.n + COLS - 1) / COLS), (unsigned)((a.m + BM - 1) / BM + (a.groups ? a.groups : 0)));
  if (grid.y > 65535) return hipErrorInvalidValue;
  if (vec) rows_product_kernel<CT, XT, WT, MI, NI, ACT, true><<<grid, 256, 0, st>>>(a);
  else rows_product_kernel<CT, XT, WT, MI, NI, ACT, false><<<grid, 256, 0, st>>>(a);
  return hipGetLastError();
}

template <typename CT, typename XT, typename WT, int ACT>
hipError_t launch_act(hipStream_t st, const ProductArgs& a, bool vec) {
  const int rows = a.groups ? (a.m + a.groups - 1) / a.groups : a.m;
  if constexpr (ACT == UGHIP_ACT_SWIGLU) {  // a tile's columns come in gate / up pairs
    return rows > 64 ? launch_tile<CT, XT, WT, 2, 2, ACT>(st, a, vec) : launch_tile<CT, XT, WT, 1, 2, ACT>(st, a, vec);
  } else {
    const long long big = (long long)((a.m + 127) / 128) * ((a.n + 127) / 128);
    if (rows > 64 && big >= 192) return launch_tile<CT, XT, WT, 2, 2, ACT>(st, a, vec);
    return launch_tile<CT, XT, WT, 1, 1, ACT>(st, a, vec);
  }
}

template <typename CT, typename XT, typename WT>
hipError_t launch_types(hipStream_t st, const ProductArgs& a, int act, bool vec) {
  if (act == UGHIP_ACT_SWIGLU) return launch_act<CT, XT, WT, UGHIP_ACT_SWIGLU>(st, a, vec);
  if (act == UGHIP_ACT_GELU_MUL) return launch_act<CT, XT, WT, UGHIP_ACT_GELU_MUL>(st, a, vec);
  return launch_act<CT, XT, WT, UGHIP_ACT_NONE>(st, a, vec);
}

constexpr size_t DMA_ROWS_MIN = 96;  // below that a 128-row tile is mostly padding

bool aligned16(const void* p) { return (reinterpret_cast<uintptr_t>(p) & 15) == 0; }

}  // namespace

extern "C" int ughip_product_rows(ughip_device* dev, const ughip_product* p) {
  const char* what = "product_rows";
  if (!dev || !p || !p->w) return set_error(UGHIP_ERR_INVALID, "%s: null argument", what);
  if (p->product != UGHIP_PRODUCT_F32 && p->product != UGHIP_PRODUCT_BF16) return set_error(UGHIP_ERR_INVALID, "%s: unknown product %d", what, p->product);
  if (p->act < UGHIP_ACT_NONE || p->act > UGHIP_ACT_GLU) return set_error(UGHIP_ERR_INVALID, "%s: unknown act %d", what, p->act);
  const bool glu = p->act == UGHIP_ACT_SWIGLU || p->act == UGHIP_ACT_GLU;  // gate and up rows
  const int act = glu ? (int)UGHIP_ACT_SWIGLU : p->act;
  if (p->m == 0 || p->n == 0) return UGHIP_OK;
  if (p->k == 0) return set_error(UGHIP_ERR_INVALID, "%s: k == 0", what);
  const bool f32 = p->product == UGHIP_PRODUCT_F32;
  const size_t mats = p->groups ? p->groups : 1;
  if (p->groups > 16384 || p->n > 0x7fffffffull / p->k) return set_error(UGHIP_ERR_INVALID, "%s: shape too large", what);
  const size_t x_rows = p->row_index ? p->x_rows : p->m;
  if (p->row_index && !p->groups) return set_error(UGHIP_ERR_INVALID, "%s: row_index belongs to the grouped form", what);
  if (x_rows == 0) return set_error(UGHIP_ERR_INVALID, "%s: no rows of x", what);
  if (int rc = check_view(dev, p->x, x_rows, p->k, f32 ? UGHIP_F32 : -1, "product_rows x")) return rc;
  const size_t w_stride = p->w_stride ? p->w_stride : p->k;
  const size_t w_rows = glu ? 2 * p->n : p->n;
  if (w_stride != p->k && p->groups) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: rows of w %zu elements apart belong to the plain form", what, w_stride);
  if (p->groups) {
    if (int rc = check_buf(dev, p->w, mats * w_rows * p->k, f32 ? UGHIP_F32 : -1, "product_rows w")) return rc;
  } else if (int rc = check_view(dev, ughip_view{const_cast<ughip_slice*>(p->w), 0, w_stride}, w_rows, p->k, f32 ? UGHIP_F32 : -1, "product_rows w")) {
    return rc;
  }
  if (int rc = check_view(dev, p->dst, p->m, p->n, f32 ? UGHIP_F32 : -1, "product_rows dst")) return rc;
  auto f_or_b = [](const ughip_slice* s) { return s->dtype == UGHIP_F32 || s->dtype == UGHIP_BF16; };
  if (!f_or_b(p->x.s) || !f_or_b(p->w) || !f_or_b(p->dst.s)) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: operands are F32 or BF16", what);
  if (p->bias && p->groups) return set_error(UGHIP_ERR_UNSUPPORTED, "%s: the grouped form takes no bias", what);
  if (p->bias)
    if (int rc = check_buf(dev, p->bias, w_rows, UGHIP_F32, "product_rows bias")) return rc;
  if (p->act == UGHIP_ACT_GELU_MUL) {
    if (!p->table || !f_or_b(p->table)) return set_error(UGHIP_ERR_INVALID, "%s: a gate's table is F32 or BF16", what);
    if (int rc = check_buf(dev, p->table, p->table_rows * p->table_stride, p->table->dtype, "product_rows table")) return rc;
    if (p->table_col > p->table_stride || p->n > p->table_stride - p->table_col) return set_error(UGHIP_ERR_BOUNDS, "%s: table columns %zu + %zu of %zu", what, p->table_col, p->n, p->table_stride);
    if (int rc = check_buf(dev, p->ids, p->m, UGHIP_I32, "product_rows ids")) return rc;
  }
  if (p->groups) {
    if (int rc = check_buf(dev, p->group_end, p->groups, UGHIP_I32, "product_rows group_end")) return rc;
    if (p->row_index)
      if (int rc = check_buf(dev, p->row_index, p->m, UGHIP_I32, "product_rows row_index")) return rc;
  }
  if (p->dst.s == p->x.s && p->dst.s->ptr && p->act != UGHIP_ACT_NONE) return set_error(UGHIP_ERR_INVALID, "%s: dst aliases x", what);
  if (int rc = device_activate(dev)) return rc;
  ProductArgs a{};
  const size_t xs = p->x.s->dtype == UGHIP_BF16 ? 2 : 4;
  a.x = static_cast<const char*>(p->x.s->ptr) + p->x.offset * xs;
  a.w = p->w->ptr;
  a.bias = buf_ptr<float>(p->bias);
  a.dst_bf16 = p->dst.s->dtype == UGHIP_BF16;
  a.dst = static_cast<char*>(p->dst.s->ptr) + p->dst.offset * (a.dst_bf16 ? 2 : 4);
  a.x_stride = p->x.stride, a.w_stride = w_stride, a.dst_stride = p->dst.stride, a.w_group = w_rows * p->k;
  a.m = (int)p->m, a.n = (int)p->n, a.k = (int)p->k;
  if (p->act == UGHIP_ACT_GELU_MUL) {
    a.table = p->table->ptr, a.table_bf16 = p->table->dtype == UGHIP_BF16, a.table_rows = (int)p->table_rows;
    a.table_stride = p->table_stride, a.table_col = p->table_col, a.ids = buf_ptr<int>(p->ids);
  }
  a.row_index = buf_ptr<int>(p->row_index), a.group_end = buf_ptr<int>(p->group_end), a.groups = (int)p->groups, a.x_rows = (int)x_rows;
  a.glu = glu_form(p->act, p->act_alpha, p->act_shift, p->act_limit);
  const bool vec = p->k % 8 == 0 && (p->x.stride * xs) % 16 == 0 && (w_stride * (p->w->dtype == UGHIP_BF16 ? 2 : 4)) % 16 == 0 && aligned16(a.x) && aligned16(a.w);
  const bool xb = p->x.s->dtype == UGHIP_BF16, wb = p->w->dtype == UGHIP_BF16;
  // few dense rows: products that share their K among workgroups
  if (!f32 && !xb && wb && !a.dst_bf16 && p->act == UGHIP_ACT_NONE && !a.bias && !a.groups && p->x.stride == p->k && p->dst.stride == p->n && w_stride == p->k &&
      few_rows_product_fits(p->w, static_cast<const float*>(a.x), static_cast<const float*>(a.dst), p->m, p->n, p->k))
    return few_rows_product(dev, what, static_cast<const float*>(a.x), p->w, static_cast<float*>(a.dst), p->m, p->n, p->k);
  if (xb && wb && p->act != UGHIP_ACT_GELU_MUL && p->m >= DMA_ROWS_MIN) {
    MMArgs q;
    q.a = a.x, q.b = a.w, q.c = nullptr;
    q.M = a.m, q.N = (int)w_rows, q.K = a.k;
    q.a_rs = (long long)a.x_stride, q.a_cs = 1, q.b_rs = 1, q.b_cs = (long long)a.w_stride;
    q.a_bs = q.b_bs = q.c_bs = 0;
    DmaRows r;
    r.row_index = a.row_index, r.group_end = a.group_end, r.bias = a.bias, r.dst = a.dst, r.w_group = (long long)a.w_group, r.dst_stride = (long long)a.dst_stride;
    r.groups = a.groups, r.x_rows = a.x_rows, r.n_out = a.n, r.dst_bf16 = a.dst_bf16;
    r.glu_alpha = a.glu.alpha, r.glu_shift = a.glu.shift, r.glu_limit = a.glu.limit;
    if (const int tile = gemm_dma_rows_pick(q, r, glu)) {
      UGHIP_HIPCHK(gemm_dma_launch_rows(dev->stream, q, r, glu, tile));
      return UGHIP_OK;
    }
  }
  hipError_t e;
  if (f32) e = launch_types<float, float, float>(dev->stream, a, act, vec);
  else if (xb && wb) e = launch_types<__bf16, uint16_t, uint16_t>(dev->stream, a, act, vec);
  else if (wb) e = launch_types<__bf16, float, uint16_t>(dev->stream, a, act, vec);
  else if (p->act == UGHIP_ACT_NONE && xb) e = launch_act<__bf16, uint16_t, float, UGHIP_ACT_NONE>(dev->stream, a, vec);
  else if (p->act == UGHIP_ACT_NONE) e = launch_act<__bf16, float, float, UGHIP_ACT_NONE>(dev->stream, a, vec);
  else return set_error(UGHIP_ERR_UNSUPPORTED, "%s: bf16 products with an activation take a BF16 matrix", what);
  UGHIP_HIPCHK(e);
  note_kernel("rows_product<%s,%s%s>", f32 ? "f32" : "bf16", p->act == UGHIP_ACT_SWIGLU ? "swiglu" : p->act == UGHIP_ACT_GLU ? "glu" : p->act == UGHIP_ACT_GELU_MUL ? "gelu_mul" : "none", p->groups ? ",grouped" : "");
  return UGHIP_OK;
}
