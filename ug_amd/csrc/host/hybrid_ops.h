// What the parts of a listed-layers decoder (hybrid.h) are built from: schedule items over this library's entry points, products of the
// stream's rows with their neighbours folded in, and the loader of their weights.
#pragma once
#include <functional>
#include <string>
#include <utility>
#include <vector>

#include "hybrid.h"
#include "ughip_layers.h"

namespace ug_llama {

// A schedule item over `args` (buffers may repeat: each reaches the item once), its result a new buffer of `shape`.  Arguments
// may be written as well (caches, states, scratch): they are stores that only this model's ops touch, in the order the data
// dependences between those ops give.
using HipCall = std::function<int(ughip_device*, const std::vector<ughip_slice*>&, ughip_slice*)>;
LB hip_op(const char* what, const std::vector<LB>& args, const std::vector<size_t>& shape, HipCall call, ug::DType dtype = ug::DType::F32);
LB scratch(ug::DType dtype, size_t n, const ug::DevicePtr& dev);

// From kHalfRows positions on the stream is kept as bf16 rows too, for the products of bf16 matrices; plain products of up to
// kFewRows positions are better off with the f32 rows (they share their K among workgroups).
constexpr size_t kHalfRows = 33, kFewRows = 128;

// The gated unit of UGHIP_ACT_GLU.
struct Glu {
  float alpha = 1.f, shift = 0.f, limit = 0.f;
};

struct Product {
  LB w, bias;  // a gated unit: gate rows then up rows
  size_t n = 0, k = 0;
  int act = UGHIP_ACT_NONE;
  LB table, ids;
  size_t table_rows = 0, table_stride = 0, table_col = 0;
  Glu glu;
  bool gated() const { return act == UGHIP_ACT_SWIGLU || act == UGHIP_ACT_GLU; }
};
inline int product_mode(const LB& w) { return w.dtype() == ug::DType::BF16 ? (int)UGHIP_PRODUCT_BF16 : (int)UGHIP_PRODUCT_F32; }

// `after`: a buffer whose op has to run first (x is scratch that it wrote).
LB product_rows(const Rows& x, size_t m, const Product& p, const LB& after = LB(), ug::DType out_type = ug::DType::F32);
LB norm_rows(const Rows& y, size_t m, size_t n, const LB& w, float eps, ug::DType out_type = ug::DType::F32);
// copy (may be invalid): scratch that receives the rows as bf16
LB gather_rows(const LB& table, size_t rows, size_t stride, size_t col, size_t cols, const LB& ids, size_t m, const LB& copy = LB());

// What is pending joins the residual: s.x is a plain [t, width] buffer afterwards.  With a norm in front of the next sublayer s.h holds
// the normed rows, in the form its first product reads (gated: a gated unit's).
void settle(StepContext& c, Stream& s, bool gated = false);
// A product of the (settled) stream's rows, in the form the step's products read.
LB stream_product(const StepContext& c, const Stream& s, const Product& p, ug::DType out_type = ug::DType::F32);
// What a producer of rows that only a product reads writes.
inline ug::DType half_type(const StepContext& c) { return c.half_rows && c.t > kFewRows ? ug::DType::BF16 : ug::DType::F32; }

// One position: a product of one row with what stands in front of it folded in (ughip_product_row).
struct RowStep {
  Product p;
  LB norm, gate;  // v = x * silu(gate), then normed over `norm_groups` parts; gate_after: normed, then times sigmoid(gate)
  size_t norm_groups = 1, gate_offset = 0;
  float eps = 0;
  bool gate_after = false;
};
constexpr size_t kRowStepMax = 16000;  // elements of the row a folded product meets (an expert's part counts in runs of 512)
// `pending` joins x first; keep_x: the joined row lies in front of the result (which starts at *at).
LB row_step(const Rows& x, const Stream* pending, size_t width, const RowStep& r, size_t* at, bool keep_x = true);
// A product of the stream's row (normed first where the stream says so); what was pending joins the residual on the way, which then
// lies in front of the result.
LB stream_step(StepContext& c, Stream& s, RowStep r, size_t* at);

struct Loader {
  WeightSource& w;
  Precision precision;
  const ug::DevicePtr& dev;
  // (v + plus) * times, `repeat` times in a row
  LB vec(const std::string& name, size_t n, float plus = 0.f, float times = 1.f, size_t repeat = 1) const;
  LB stacked_vec(const std::vector<std::pair<std::string, size_t>>& parts) const;
  LB f32(const std::string& name, const std::vector<size_t>& shape) const { return w.load(name, shape, dev); }
  // several [rows, k] tensors by rows, in f32
  LB stacked_f32(const std::vector<std::pair<std::string, size_t>>& parts, size_t k) const;
  // a matrix (or several by rows) in the dtype the products of this model read
  LB matrix(const std::string& name, const std::vector<size_t>& shape) const { return stored(w.load(name, shape, dev)); }
  LB stacked(const std::vector<std::pair<std::string, size_t>>& parts, size_t k) const { return stored(stacked_f32(parts, k)); }
  // Rows of a tensor whose size only the weights say (random ones take `fallback`).
  size_t rows_of(const std::string& name, size_t fallback) const;

 private:
  LB stored(const LB& lb) const;
};

}  // namespace ug_llama
