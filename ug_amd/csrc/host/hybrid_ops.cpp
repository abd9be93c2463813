#include "hybrid_ops.h"

#include "hip_device.h"

namespace ug_llama {

using namespace ug;

LB hip_op(const char* what, const std::vector<LB>& args, const std::vector<size_t>& shape, HipCall call, DType dtype) {
  HipDevice* hd = dynamic_cast<HipDevice*>(args[0].device().get());
  if (!hd) bail(std::string(what) + ": this model runs on the hip device only");
  ughip_device* dev = hd->raw();
  std::vector<LB> unique;
  std::vector<size_t> index;
  for (const LB& a : args) {
    size_t i = 0;
    while (i < unique.size() && unique[i].data().get() != a.data().get()) ++i;
    if (i == unique.size()) unique.push_back(a);
    index.push_back(i);
  }
  const std::string name = what;
  auto f = [=, n = unique.size()](const std::vector<Slice*>& vs) {
    if (vs.size() != n + 1) bail(name + ": unexpected number of slices");
    std::vector<ughip_slice*> in;
    in.reserve(index.size());
    for (size_t i : index) in.push_back(hip_raw_slice(*vs[i]));
    if (call(dev, in, hip_raw_slice(*vs[n]))) bail(name + ": " + ughip_last_error());
  };
  return LB::custom(f, unique, Shape(shape), dtype, args[0].device());
}

LB scratch(DType dtype, size_t n, const DevicePtr& dev) {
  LB lb = LB::alloc_uninit(dtype, Shape({n}), dev);
  lb.maybe_allocate_uninit();
  return lb;
}

LB product_rows(const Rows& x, size_t m, const Product& p, const LB& after, DType out_type) {
  std::vector<LB> args = {x.lb, p.w};
  auto add = [&](const LB& lb) {
    if (!lb.valid()) return (size_t)0;
    args.push_back(lb);
    return args.size() - 1;
  };
  const size_t b = add(p.bias), tb = add(p.table), ids = add(p.ids);
  add(after);
  const size_t off = x.offset, stride = x.stride, n = p.n, k = p.k, trows = p.table_rows, tstride = p.table_stride, tcol = p.table_col;
  const int act = p.act, mode = product_mode(p.w);
  const Glu glu = p.glu;
  return hip_op("product_rows", args, {m, n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    ughip_product q{};
    q.x = {in[0], off, stride};
    q.dst = {out, 0, n};
    q.w = in[1];
    if (b) q.bias = in[b];
    if (tb) q.table = in[tb], q.ids = in[ids];
    q.m = m, q.n = n, q.k = k, q.product = mode, q.act = act;
    q.table_rows = trows, q.table_stride = tstride, q.table_col = tcol;
    q.act_alpha = glu.alpha, q.act_shift = glu.shift, q.act_limit = glu.limit;
    return ughip_product_rows(d, &q);
  }, out_type);
}

LB norm_rows(const Rows& y, size_t m, size_t n, const LB& w, float eps, DType out_type) {
  const size_t off = y.offset, stride = y.stride;
  return hip_op("norm_rows", {y.lb, w}, {m, n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    return ughip_add_rms_norm_rows(d, {nullptr, 0, 0}, {in[0], off, stride}, nullptr, nullptr, 0, 0, in[1], eps, {nullptr, 0, 0}, {out, 0, n}, nullptr, nullptr, m, n);
  }, out_type);
}

LB gather_rows(const LB& table, size_t rows, size_t stride, size_t col, size_t cols, const LB& ids, size_t m, const LB& copy) {
  std::vector<LB> args = {table, ids};
  const bool twice = copy.valid();
  if (twice) args.push_back(copy);
  return hip_op("gather_rows", args, {m, cols}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    if (twice)
      if (int rc = ughip_gather_rows(d, in[0], rows, stride, col, cols, in[1], m, {in[2], 0, cols})) return rc;
    return ughip_gather_rows(d, in[0], rows, stride, col, cols, in[1], m, {out, 0, cols});
  });
}

void settle(StepContext& c, Stream& s, bool gated) {
  const bool join = s.norm.valid(), extra = s.extra.lb.valid(), ahead = s.ahead.valid() && !s.h.valid();
  const size_t t = c.t, n = c.width;
  const float eps = c.eps;
  const DType h_type = c.half_rows && (gated || t > kFewRows) ? DType::BF16 : DType::F32;
  if (!join && !extra) {
    if (ahead) s.h = norm_rows(s.x, t, n, s.ahead, eps, h_type), s.h_by = s.h;
    return;
  }
  const Rows x = s.x, y = s.y, e = s.extra;
  const size_t top = s.top, y_rows = s.y_rows;
  std::vector<LB> args = {x.lb};
  auto add = [&](const LB& lb) {
    if (!lb.valid()) return (size_t)0;
    args.push_back(lb);
    return args.size() - 1;
  };
  const size_t iy = join ? add(y.lb) : 0, in_ = join ? add(s.norm) : 0, is = top ? add(s.slots) : 0, iw = top ? add(s.weights) : 0, ie = extra ? add(e.lb) : 0;
  // the rows once more: as bf16, or normed for the next sublayer
  s.x16 = c.half_rows && !c.norm_ahead ? scratch(DType::BF16, t * n, c.dev) : LB();
  if (ahead) s.h = scratch(h_type, t * n, c.dev);
  const size_t copy = ahead ? add(s.h) : add(s.x16), next = ahead ? add(s.ahead) : 0;
  LB out = hip_op("add_norm", args, {t, n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* dst) {
    const ughip_view none{nullptr, 0, 0};
    return ughip_add_rms_norm_rows(d, {in[0], x.offset, x.stride}, iy ? ughip_view{in[iy], y.offset, y.stride} : none, is ? in[is] : nullptr, iw ? in[iw] : nullptr, top, y_rows,
                                   in_ ? in[in_] : nullptr, eps, ie ? ughip_view{in[ie], e.offset, e.stride} : none, {dst, 0, n}, next ? in[next] : nullptr,
                                   copy ? in[copy] : nullptr, t, n);
  });
  if (ahead) s.h_by = out;
  s.x = {out, 0, n};
  s.y = s.extra = Rows();
  s.norm = LB();
  s.slots = s.weights = LB();
  s.top = s.y_rows = 0;
}

LB stream_product(const StepContext& c, const Stream& s, const Product& p, DType out_type) {
  if (s.h.valid()) return product_rows({s.h, 0, c.width}, c.t, p, s.h_by, out_type);
  if (s.x16.valid() && (c.t > kFewRows || p.gated())) return product_rows({s.x16, 0, c.width}, c.t, p, s.x.lb, out_type);
  return product_rows(s.x, c.t, p, LB(), out_type);
}

LB row_step(const Rows& x, const Stream* pending, size_t width, const RowStep& r, size_t* at, bool keep_x) {
  const bool join = pending && pending->norm.valid();
  std::vector<LB> args = {x.lb, r.p.w};
  auto add = [&](const LB& lb) {
    if (!lb.valid()) return (size_t)0;
    args.push_back(lb);
    return args.size() - 1;
  };
  const size_t b = add(r.p.bias), tb = add(r.p.table), ids = add(r.p.ids), nm = add(r.norm), gt = add(r.gate);
  const size_t y = join ? add(pending->y.lb) : 0, yn = join ? add(pending->norm) : 0, y_off = join ? pending->y.offset : 0, off = x.offset;
  const bool extra = join && pending->extra.lb.valid(), after = r.gate_after;
  const size_t ex = extra ? add(pending->extra.lb) : 0, e_off = extra ? pending->extra.offset : 0;
  const Glu glu = r.p.glu;
  const Product pr = r.p;  // (the buffers inside keep their owners alive as the arguments do)
  const size_t ng = r.norm_groups, g_off = r.gate_offset, base = join && keep_x ? width : 0;
  const float eps = r.eps;
  const size_t n = pr.n, k = pr.k, trows = pr.table_rows, tstride = pr.table_stride, tcol = pr.table_col;
  const int act = pr.act;
  *at = base;
  return hip_op("row_step", args, {1, base + n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    ughip_row_step q{};
    q.x = in[0], q.x_offset = off, q.w = in[1];
    if (y) q.y = in[y], q.y_offset = y_off, q.y_norm = in[yn], q.keep_x = base != 0;
    if (b) q.bias = in[b];
    if (tb) q.table = in[tb], q.ids = in[ids];
    if (nm) q.norm = in[nm], q.norm_groups = ng;
    if (gt) q.gate = in[gt], q.gate_offset = g_off, q.gate_after = after;
    if (ex) q.extra = in[ex], q.extra_offset = e_off;
    q.act_alpha = glu.alpha, q.act_shift = glu.shift, q.act_limit = glu.limit;
    q.eps = eps, q.act = act, q.n = n, q.k = k;
    q.table_rows = trows, q.table_stride = tstride, q.table_col = tcol;
    q.dst = out, q.dst_offset = base, q.x_out = 0;
    return ughip_product_row(d, &q);
  });
}

LB stream_step(StepContext& c, Stream& s, RowStep r, size_t* at) {
  if (s.top || (s.extra.lb.valid() && !s.norm.valid())) {
    const LB ahead = s.ahead;
    s.ahead = LB();  // (this product norms its row itself)
    settle(c, s);
    s.ahead = ahead;
  }
  if (s.ahead.valid()) r.norm = s.ahead;
  r.eps = c.eps;
  LB out = row_step(s.x, &s, c.width, r, at);
  if (s.norm.valid()) {
    s.x = {out, 0, c.width};
    s.y = s.extra = Rows();
    s.norm = LB();
  }
  return out;
}

LB Loader::vec(const std::string& name, size_t n, float plus, float times, size_t repeat) const {
  std::vector<float> v = w.get(name, {n}), all;
  for (float& e : v) e = (e + plus) * times;
  for (size_t i = 0; i < repeat; ++i) all.insert(all.end(), v.begin(), v.end());
  return LB::copy(all.data(), DType::F32, all.size(), Shape({all.size()}), dev);
}

LB Loader::stacked_vec(const std::vector<std::pair<std::string, size_t>>& parts) const {
  std::vector<float> all;
  for (const auto& p : parts) {
    std::vector<float> v = w.get(p.first, {p.second});
    all.insert(all.end(), v.begin(), v.end());
  }
  return LB::copy(all.data(), DType::F32, all.size(), Shape({all.size()}), dev);
}

LB Loader::stacked_f32(const std::vector<std::pair<std::string, size_t>>& parts, size_t k) const {
  size_t rows = 0;
  for (const auto& p : parts) rows += p.second;
  std::vector<float> all;
  all.reserve(rows * k);
  for (const auto& p : parts) {
    std::vector<float> v = w.get(p.first, {p.second, k});
    all.insert(all.end(), v.begin(), v.end());
  }
  return LB::copy(all.data(), DType::F32, all.size(), Shape({rows, k}), dev);
}

size_t Loader::rows_of(const std::string& name, size_t fallback) const {
  const std::vector<size_t> shape = w.shape_of(name, {fallback, 1});
  if (shape.size() != 2 || shape[0] == 0) bail("unexpected shape for " + name + ": a matrix was expected");
  return shape[0];
}

LB Loader::stored(const LB& lb) const {
  if (precision == Precision::F32) return lb;
  LB n = lb.cast(DType::BF16);
  n.realize();
  n.detach();
  return n;
}

}  // namespace ug_llama
