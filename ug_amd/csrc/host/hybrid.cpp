#include "hybrid.h"

#include <algorithm>
#include <cmath>
#include <mutex>

#include "hip_device.h"
#include "ughip_layers.h"

namespace ug_llama {

using namespace ug;

namespace {

// ---- ops ------------------------------------------------------------------------------------------------------------------
// A schedule item over `args` (buffers may repeat: each reaches the item once), its result a new buffer of `shape`.  Arguments
// may be written as well (caches, states, scratch): they are stores that only this model's ops touch, in the order the data
// dependences between those ops give.
using HipCall = std::function<int(ughip_device*, const std::vector<ughip_slice*>&, ughip_slice*)>;
LB hip_op(const char* what, const std::vector<LB>& args, const std::vector<size_t>& shape, HipCall call, DType dtype = DType::F32) {
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

// From kHalfRows positions on the stream is kept as bf16 rows too, for the products of bf16 matrices; plain products of up to
// kFewRows positions are better off with the f32 rows (they share their K among workgroups).
constexpr size_t kHalfRows = 33, kFewRows = 128;

struct Product {
  LB w, bias;  // UGHIP_ACT_SWIGLU: gate rows then up rows
  size_t n = 0, k = 0;
  int act = UGHIP_ACT_NONE;
  LB table, ids;
  size_t table_rows = 0, table_stride = 0, table_col = 0;
};
int product_mode(const LB& w) { return w.dtype() == DType::BF16 ? (int)UGHIP_PRODUCT_BF16 : (int)UGHIP_PRODUCT_F32; }

// `after`: a buffer whose op has to run first (x is scratch that it wrote).
LB product_rows(const Rows& x, size_t m, const Product& p, const LB& after = LB(), DType out_type = DType::F32) {
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
  return hip_op("product_rows", args, {m, n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    ughip_product q{};
    q.x = {in[0], off, stride};
    q.dst = {out, 0, n};
    q.w = in[1];
    if (b) q.bias = in[b];
    if (tb) q.table = in[tb], q.ids = in[ids];
    q.m = m, q.n = n, q.k = k, q.product = mode, q.act = act;
    q.table_rows = trows, q.table_stride = tstride, q.table_col = tcol;
    return ughip_product_rows(d, &q);
  }, out_type);
}

LB norm_rows(const Rows& y, size_t m, size_t n, const LB& w, float eps, DType out_type = DType::F32) {
  const size_t off = y.offset, stride = y.stride;
  return hip_op("norm_rows", {y.lb, w}, {m, n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    return ughip_add_rms_norm_rows(d, {nullptr, 0, 0}, {in[0], off, stride}, nullptr, nullptr, 0, 0, in[1], eps, {out, 0, n}, nullptr, m, n);
  }, out_type);
}

// copy (may be invalid): scratch that receives the rows as bf16
LB gather_rows(const LB& table, size_t rows, size_t stride, size_t col, size_t cols, const LB& ids, size_t m, const LB& copy = LB()) {
  std::vector<LB> args = {table, ids};
  const bool twice = copy.valid();
  if (twice) args.push_back(copy);
  return hip_op("gather_rows", args, {m, cols}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* out) {
    if (twice)
      if (int rc = ughip_gather_rows(d, in[0], rows, stride, col, cols, in[1], m, {in[2], 0, cols})) return rc;
    return ughip_gather_rows(d, in[0], rows, stride, col, cols, in[1], m, {out, 0, cols});
  });
}

// The pending output joins the residual: s.x is a plain [t, width] buffer afterwards.
void settle(StepContext& c, Stream& s) {
  if (!s.norm.valid()) return;
  const Rows x = s.x, y = s.y;
  const size_t t = c.t, n = c.width, top = s.top, y_rows = s.y_rows;
  const float eps = c.eps;
  std::vector<LB> args = {x.lb, y.lb, s.norm};
  if (top) args.push_back(s.slots), args.push_back(s.weights);
  s.x16 = c.half_rows ? scratch(DType::BF16, t * n, c.dev) : LB();
  const size_t copy = s.x16.valid() ? args.size() : 0;
  if (copy) args.push_back(s.x16);
  LB out = hip_op("add_norm", args, {t, n}, [=](ughip_device* d, const std::vector<ughip_slice*>& in, ughip_slice* dst) {
    return ughip_add_rms_norm_rows(d, {in[0], x.offset, x.stride}, {in[1], y.offset, y.stride}, top ? in[3] : nullptr, top ? in[4] : nullptr, top, y_rows, in[2], eps,
                                   {dst, 0, n}, copy ? in[copy] : nullptr, t, n);
  });
  s.x = {out, 0, n};
  s.y = Rows();
  s.norm = LB();
  s.slots = s.weights = LB();
  s.top = s.y_rows = 0;
}

// A product of the (settled) stream's rows, in the form the step's products read.
LB stream_product(const StepContext& c, const Stream& s, const Product& p, DType out_type = DType::F32) {
  if (s.x16.valid() && (c.t > kFewRows || p.act == UGHIP_ACT_SWIGLU)) return product_rows({s.x16, 0, c.width}, c.t, p, s.x.lb, out_type);
  return product_rows(s.x, c.t, p, LB(), out_type);
}
// What a producer of rows that only a product reads writes.
DType half_type(const StepContext& c) { return c.half_rows && c.t > kFewRows ? DType::BF16 : DType::F32; }

// One position: a product of one row with what stands in front of it folded in (ughip_product_row).
struct RowStep {
  Product p;
  LB norm, gate;  // v = x * silu(gate), then normed over `norm_groups` parts
  size_t norm_groups = 1, gate_offset = 0;
  float eps = 0;
};
constexpr size_t kRowStepMax = 16000;  // elements of the row a folded product meets (an expert's part counts in runs of 512)

// `pending` joins x first; keep_x: the joined row lies in front of the result (which starts at *at).
LB row_step(const Rows& x, const Stream* pending, size_t width, const RowStep& r, size_t* at, bool keep_x = true) {
  const bool join = pending && pending->norm.valid();
  std::vector<LB> args = {x.lb, r.p.w};
  auto add = [&](const LB& lb) {
    if (!lb.valid()) return (size_t)0;
    args.push_back(lb);
    return args.size() - 1;
  };
  const size_t b = add(r.p.bias), tb = add(r.p.table), ids = add(r.p.ids), nm = add(r.norm), gt = add(r.gate);
  const size_t y = join ? add(pending->y.lb) : 0, yn = join ? add(pending->norm) : 0, y_off = join ? pending->y.offset : 0, off = x.offset;
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
    if (gt) q.gate = in[gt], q.gate_offset = g_off;
    q.eps = eps, q.act = act, q.n = n, q.k = k;
    q.table_rows = trows, q.table_stride = tstride, q.table_col = tcol;
    q.dst = out, q.dst_offset = base, q.x_out = 0;
    return ughip_product_row(d, &q);
  });
}

// A product of the stream's row; what was pending joins the residual on the way, which then lies in front of the result.
LB stream_step(StepContext& c, Stream& s, RowStep r, size_t* at) {
  if (s.top) settle(c, s);
  r.eps = c.eps;
  LB out = row_step(s.x, &s, c.width, r, at);
  if (s.norm.valid()) {
    s.x = {out, 0, c.width};
    s.y = Rows();
    s.norm = LB();
  }
  return out;
}

// ---- loading --------------------------------------------------------------------------------------------------------------
struct Loader {
  WeightSource& w;
  Precision precision;
  const DevicePtr& dev;
  LB vec(const std::string& name, size_t n, float plus = 0.f) const {
    std::vector<float> v = w.get(name, {n});
    if (plus != 0.f)
      for (float& e : v) e += plus;
    return LB::copy(v.data(), DType::F32, n, Shape({n}), dev);
  }
  LB stacked_vec(const std::vector<std::pair<std::string, size_t>>& parts) const {
    std::vector<float> all;
    for (const auto& p : parts) {
      std::vector<float> v = w.get(p.first, {p.second});
      all.insert(all.end(), v.begin(), v.end());
    }
    return LB::copy(all.data(), DType::F32, all.size(), Shape({all.size()}), dev);
  }
  LB f32(const std::string& name, const std::vector<size_t>& shape) const { return w.load(name, shape, dev); }
  // a matrix (or several by rows) in the dtype the products of this model read
  LB matrix(const std::string& name, const std::vector<size_t>& shape) const { return stored(w.load(name, shape, dev)); }
  LB stacked(const std::vector<std::pair<std::string, size_t>>& parts, size_t k) const {
    size_t rows = 0;
    for (const auto& p : parts) rows += p.second;
    std::vector<float> all;
    all.reserve(rows * k);
    for (const auto& p : parts) {
      std::vector<float> v = w.get(p.first, {p.second, k});
      all.insert(all.end(), v.begin(), v.end());
    }
    return stored(LB::copy(all.data(), DType::F32, all.size(), Shape({rows, k}), dev));
  }

 private:
  LB stored(const LB& lb) const {
    if (precision == Precision::F32) return lb;
    LB n = lb.cast(DType::BF16);
    n.realize();
    n.detach();
    return n;
  }
};

// ---- latent attention -----------------------------------------------------------------------------------------------------
struct LatentAttention : Mixer {
  size_t heads, dim, rot, vdim, q_rank, rank, width;
  float scale, eps;
  long kv_from = -1;  // the layer whose cache this one reads; -1: its own
  std::shared_ptr<RopeTables> rope;
  LB down;  // [dq; dkv], or dq alone
  LB dq_norm, kv_norm, uq, uk, uv, o;
  static constexpr size_t kAbsorbMax = 736;
  // Steps of up to this many positions attend to the latents themselves instead of expanding all of them into keys and values.
  size_t absorb_up_to;

  LatentAttention(const Json& m, const std::string& p, const Loader& ld, size_t width_, float eps_, std::shared_ptr<RopeTables> rope_) : width(width_), eps(eps_), rope(std::move(rope_)) {
    heads = m.size_at("heads"), dim = m.size_at("dim"), rot = m.size_at("rot_dim"), vdim = m.size_at("vdim");
    q_rank = m.size_at("q_rank"), rank = m.size_at("kv_rank");
    scale = (float)m.num_at("scale");
    if (m.find("kv_from")) kv_from = (long)m.size_at("kv_from");
    std::vector<std::pair<std::string, size_t>> parts = {{p + "dq", q_rank}};
    if (kv_from < 0) parts.push_back({p + "dkv", rank + rot});
    down = ld.stacked(parts, width);
    dq_norm = ld.vec(p + "dq.norm", q_rank);
    if (kv_from < 0) kv_norm = ld.vec(p + "dkv.norm", rank);
    uq = ld.matrix(p + "uq", {heads * (dim + rot), q_rank});
    uk = ld.matrix(p + "uk", {heads * dim, rank});
    uv = ld.matrix(p + "uv", {heads * vdim, rank});
    o = ld.matrix(p + "o", {width, heads * vdim});
    absorb_up_to = std::max<size_t>(1, (dim + vdim) / 4);
    if (rank + rot > kAbsorbMax) absorb_up_to = 0;  // rows too long for the absorbed kernel
    else if (dim + rot > 256 || vdim > 256) absorb_up_to = (size_t)-1;  // sizes the expanded kernel is not built for
  }

  MixerState new_state(size_t capacity) const override {
    MixerState st;
    if (kv_from < 0) st.buffers.push_back(scratch(DType::F32, capacity * (rank + rot), down.device()));
    return st;
  }

  void run(StepContext& c, Stream& s, size_t layer) const override {
    const bool own = kv_from < 0;
    const size_t t = c.t, pos = c.pos, cap = c.capacity, H = heads, d = dim, r = rot, v = vdim, rk = rank, qr = q_rank, all = pos + t;
    const size_t wide = qr + (own ? rk + r : 0), trows = rope->rows;
    const float e = eps, sc = scale;
    const LB cache = c.state->layers[own ? layer : (size_t)kv_from].buffers[0];
    const bool fused = c.fused && t <= absorb_up_to && std::max({width, qr, H * v}) <= kRowStepMax;
    LB low, q;
    size_t low_at = 0, none;
    if (fused) {
      low = stream_step(c, s, {{down, LB(), wide, width}}, &low_at);
      RowStep up{{uq, LB(), H * (d + r), qr}};
      up.norm = dq_norm, up.eps = e;
      q = row_step({low, low_at, qr}, nullptr, 0, up, &none);
    } else {
      settle(c, s);
      low = stream_product(c, s, {down, LB(), wide, width});
      LB cq = norm_rows({low, 0, wide}, t, qr, dq_norm, e, half_type(c));
      q = product_rows({cq, 0, qr}, t, {uq, LB(), H * (d + r), qr});
    }
    // `low` is the first to know this step's rows: an op that reads the cache takes it as an argument, and the first one of
    // the layer that owns the cache writes the rows
    std::vector<LB> head_args = {low, cache, rope->cos, rope->sin};
    if (own) head_args.push_back(kv_norm);
    const size_t n_head = head_args.size();
    LB a;
    if (t <= absorb_up_to) {
      std::vector<LB> args = head_args;
      args.insert(args.end(), {q, uk, uv});
      a = hip_op("latent_attention_absorbed", args, {t, H * v}, [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
        return ughip_latent_attention_absorbed(dev, {in[n_head], 0, H * (d + r)}, {own ? in[0] : nullptr, low_at + qr, wide}, own ? in[4] : nullptr, e, in[n_head + 1],
                                               in[n_head + 2], in[1], cap, in[2], in[3], trows, {out, 0, H * v}, t, pos, H, d, r, v, rk, sc);
      });
    } else {
      const int mode = product_mode(uk);
      const DType kv_type = uk.dtype();
      std::vector<LB> args = head_args;
      args.push_back(uk);
      LB k = hip_op("latent_keys", args, {all, H * d},
                    [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
                      if (own)
                        if (int rc = ughip_latent_append(dev, {in[0], qr, wide}, in[4], e, in[2], in[3], trows, in[1], cap, pos, t, rk, r)) return rc;
                      ughip_product p{};
                      p.x = {in[1], 0, rk + r}, p.dst = {out, 0, H * d}, p.w = in[n_head];
                      p.m = all, p.n = H * d, p.k = rk, p.product = mode;
                      return ughip_product_rows(dev, &p);
                    },
                    kv_type);
      // values transposed: the matrix's rows against the cache's (k is an argument because its op wrote this step's rows)
      const size_t v_stride = (all + 63) & ~(size_t)63;
      LB vt = hip_op("latent_values", {uv, cache, k}, {H * v, v_stride},
                     [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
                       ughip_product p{};
                       p.x = {in[0], 0, rk}, p.dst = {out, 0, v_stride}, p.w = in[1], p.w_stride = rk + r;
                       p.m = H * v, p.n = all, p.k = rk, p.product = mode;
                       return ughip_product_rows(dev, &p);
                     },
                     kv_type);
      a = hip_op("latent_attention", {q, k, vt, cache, rope->cos, rope->sin}, {t, H * v}, [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
        return ughip_latent_attention_rows(dev, {in[0], 0, H * (d + r)}, in[1], in[2], v_stride, in[3], in[4], in[5], trows, {out, 0, H * v}, t, pos, H, d, r, v, rk, sc);
      }, half_type(c));
    }
    if (fused) s.y = {row_step({a, 0, H * v}, nullptr, 0, {{o, LB(), width, H * v}}, &none), 0, width};
    else s.y = {product_rows({a, 0, H * v}, t, {o, LB(), width, H * v}), 0, width};
  }

};

// ---- state-space mixer ----------------------------------------------------------------------------------------------------
struct Mamba2 : Mixer {
  size_t heads, vdim, state, groups, taps, norm_groups, width;
  float eps;
  LB in, conv, conv_b, dt_bias, a_log, skip, norm, o;
  size_t inner() const { return heads * vdim; }
  size_t channels() const { return inner() + 2 * groups * state; }

  Mamba2(const Json& m, const std::string& p, const Loader& ld, size_t width_, float eps_) : width(width_), eps(eps_) {
    heads = m.size_at("heads"), vdim = m.size_at("vdim"), state = m.size_at("state"), groups = m.size_at("groups"), taps = m.size_at("conv");
    norm_groups = m.size_at("norm_groups");
    in = ld.matrix(p + "in", {inner() + channels() + heads, width});
    conv = ld.f32(p + "conv", {channels(), taps});
    conv_b = ld.vec(p + "conv.b", channels());
    dt_bias = ld.vec(p + "dt_bias", heads);
    a_log = ld.vec(p + "A_log", heads);
    skip = ld.vec(p + "D", heads);
    norm = ld.vec(p + "norm", inner());
    o = ld.matrix(p + "o", {width, inner()});
  }

  MixerState new_state(size_t) const override {
    // contents are taken as zeros by the first step, whatever the memory held before
    return MixerState{{scratch(DType::F32, heads * state * vdim, in.device()), scratch(DType::F32, taps * channels(), in.device())}};
  }

  void run(StepContext& c, Stream& s, size_t layer) const override {
    const size_t t = c.t, pos = c.pos, I = inner(), ch = channels(), H = heads, vd = vdim, N = state, G = groups, nt = taps, wide = I + ch + H, ng = norm_groups;
    const float e = eps;
    const LB S = c.state->layers[layer].buffers[0], ring = c.state->layers[layer].buffers[1];
    if (c.fused && std::max(width, I) <= kRowStepMax && N <= 4096) {
      size_t at, none;
      LB p = stream_step(c, s, {{in, LB(), wide, width}}, &at);
      LB y = hip_op("ssm_step", {p, conv, conv_b, dt_bias, a_log, skip, S, ring}, {1, I}, [=](ughip_device* dev, const std::vector<ughip_slice*>& a, ughip_slice* out) {
        return ughip_ssm_step(dev, a[0], at + I, at + I + ch, a[1], a[2], nt, a[7], a[3], a[4], a[5], a[6], pos, H, vd, G, N, {out, 0, I});
      });
      RowStep last{{o, LB(), width, I}};
      last.gate = p, last.gate_offset = at, last.norm = norm, last.norm_groups = ng, last.eps = e;
      s.y = {row_step({y, 0, I}, nullptr, 0, last, &none), 0, width};
      return;
    }
    settle(c, s);
    LB p = stream_product(c, s, {in, LB(), wide, width});
    LB xbc = hip_op("conv_silu", {p, conv, conv_b, ring}, {t, ch}, [=](ughip_device* dev, const std::vector<ughip_slice*>& a, ughip_slice* out) {
      return ughip_conv_silu_rows(dev, {a[0], I, wide}, a[1], a[2], nt, a[3], pos, t, ch, {out, 0, ch});
    });
    LB y = hip_op("ssm", {xbc, p, dt_bias, a_log, skip, S, ring}, {t, I}, [=](ughip_device* dev, const std::vector<ughip_slice*>& a, ughip_slice* out) {
      if (int rc = ughip_conv_ring_store(dev, {a[1], I, wide}, nt, a[6], pos, t, ch)) return rc;
      return ughip_ssm_rows(dev, {a[0], 0, ch}, {a[1], I + ch, wide}, a[2], a[3], a[4], a[5], pos, t, H, vd, G, N, {out, 0, I});
    });
    LB yn = hip_op("gated_norm", {y, p, norm}, {t, I}, [=](ughip_device* dev, const std::vector<ughip_slice*>& a, ughip_slice* out) {
      return ughip_gated_rms_norm_rows(dev, {a[0], 0, I}, {a[1], 0, wide}, a[2], e, ng, {out, 0, I}, t, I);
    }, half_type(c));
    s.y = {product_rows({yn, 0, I}, t, {o, LB(), width, I}), 0, width};
  }
};

// ---- feed-forward ---------------------------------------------------------------------------------------------------------
struct DenseFeedForward : FeedForward {
  size_t ff, width;
  LB gate_up, gate_up_b, down, down_b;
  DenseFeedForward(const Json& m, const std::string& p, const Loader& ld, size_t width_) : width(width_) {
    ff = m.size_at("ff");
    gate_up = ld.stacked({{p + "gate", ff}, {p + "up", ff}}, width), gate_up_b = ld.stacked_vec({{p + "gate.b", ff}, {p + "up.b", ff}});
    down = ld.matrix(p + "down", {width, ff}), down_b = ld.vec(p + "down.b", width);
  }
  void run(StepContext& c, Stream& s) const override {
    const Product first{gate_up, gate_up_b, ff, width, UGHIP_ACT_SWIGLU}, second{down, down_b, width, ff};
    if (c.fused && std::max(width, ff) <= kRowStepMax) {
      size_t at, none;
      LB a = stream_step(c, s, {first}, &at);
      s.y = {row_step({a, at, ff}, nullptr, 0, {second}, &none), 0, width};
      return;
    }
    settle(c, s);
    LB a = stream_product(c, s, first, half_type(c));
    s.y = {product_rows({a, 0, ff}, c.t, second), 0, width};
  }
};

struct MoeFeedForward : FeedForward {
  size_t experts, top, count, keep, ff, width;
  LB router, correction, gate_up, down;  // the experts' matrices one after the other, every gate in front of its up
  MoeFeedForward(const Json& m, const std::string& p, const Loader& ld, size_t width_) : width(width_) {
    const Json& r = m.at("router");
    experts = r.size_at("experts"), top = r.size_at("top");
    const Json* g = r.find("groups");
    count = g ? g->size_at("count") : 1, keep = g ? g->size_at("keep") : 1;
    ff = m.at("expert").size_at("ff");
    if (!experts || !count || experts % count || !keep || keep > count || !top || top > keep * (experts / count))
      bail("configuration: a router of " + std::to_string(top) + " of " + std::to_string(experts) + " experts in " + std::to_string(keep) + " of " + std::to_string(count) + " groups");
    router = ld.f32(p + "router", {experts, width});
    correction = ld.vec(p + "correction", experts);
    std::vector<std::pair<std::string, size_t>> gs, ds;
    for (size_t e = 0; e < experts; ++e) {
      const std::string q = p + "e" + std::to_string(e);
      gs.push_back({q + ".gate", ff}), gs.push_back({q + ".up", ff}), ds.push_back({q + ".down", width});
    }
    gate_up = ld.stacked(gs, width), down = ld.stacked(ds, ff);
  }
  void run(StepContext& c, Stream& s) const override {
    if (c.fused && std::max(width, top * ((ff + 511) / 512 * 512)) <= kRowStepMax && top <= 64) return run_step(c, s);
    settle(c, s);
    const size_t t = c.t, E = experts, tp = top, w = width, f = ff, gc = count, kp = keep, pairs = t * tp;
    const int mode = product_mode(gate_up);
    const Rows x = s.x;
    const bool half = s.x16.valid();
    LB ids = scratch(DType::I32, pairs, c.dev), weights = scratch(DType::F32, pairs, c.dev), row_index = scratch(DType::I32, pairs, c.dev);
    LB slots = scratch(DType::I32, pairs, c.dev), group_end = scratch(DType::I32, E, c.dev);
    const DType act_type = gate_up.dtype();
    std::vector<LB> args = {x.lb, router, correction, gate_up, ids, weights, row_index, slots, group_end};
    if (half) args.push_back(s.x16);
    LB a = hip_op("route_gate_up", args, {pairs, f},
                  [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
                    if (int rc = ughip_route_rows(dev, {in[0], x.offset, x.stride}, in[1], in[2], t, w, E, gc, kp, tp, in[4], in[5])) return rc;
                    if (int rc = ughip_group_rows(dev, in[4], t, tp, E, in[6], in[7], in[8])) return rc;
                    ughip_product p{};
                    p.x = half ? ughip_view{in[9], 0, w} : ughip_view{in[0], x.offset, x.stride}, p.dst = {out, 0, f}, p.w = in[3];
                    p.m = pairs, p.n = f, p.k = w, p.product = mode, p.act = UGHIP_ACT_SWIGLU;
                    p.row_index = in[6], p.group_end = in[8], p.groups = E, p.x_rows = t;
                    return ughip_product_rows(dev, &p);
                  },
                  act_type);
    LB y = hip_op("experts_down", {a, down, group_end}, {pairs, w}, [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
      ughip_product p{};
      p.x = {in[0], 0, f}, p.dst = {out, 0, w}, p.w = in[1];
      p.m = pairs, p.n = w, p.k = f, p.product = mode, p.group_end = in[2], p.groups = E;
      return ughip_product_rows(dev, &p);
    });
    s.y = {y, 0, w};
    s.slots = slots, s.weights = weights, s.top = tp, s.y_rows = pairs;
  }

 private:
  void run_step(StepContext& c, Stream& s) const {
    const size_t E = experts, tp = top, w = width, f = ff, gc = count, kp = keep;
    size_t at;
    LB logits = stream_step(c, s, {{router, LB(), E, w}}, &at);
    const Rows x = s.x;
    LB ids = scratch(DType::I32, tp, c.dev), weights = scratch(DType::F32, tp, c.dev);
    auto routed = [=](const std::vector<ughip_slice*>& in, size_t first) {
      ughip_row_step q{};
      q.route_ids = in[first], q.route_weights = in[first + 1];
      q.experts = E, q.groups = gc, q.keep = kp, q.top = tp;
      return q;
    };
    LB a = hip_op("experts_gate_up_step", {x.lb, logits, correction, gate_up, ids, weights}, {1, tp * f},
                  [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
                    ughip_row_step q = routed(in, 4);
                    q.x = in[0], q.x_offset = x.offset, q.logits = in[1], q.logits_offset = at, q.correction = in[2];
                    q.w = in[3], q.act = UGHIP_ACT_SWIGLU, q.route = 1, q.n = f, q.k = w, q.dst = out;
                    return ughip_product_row(dev, &q);
                  });
    LB y = hip_op("experts_down_step", {a, down, ids, weights}, {1, w}, [=](ughip_device* dev, const std::vector<ughip_slice*>& in, ughip_slice* out) {
      ughip_row_step q = routed(in, 2);
      q.x = in[0], q.w = in[1], q.route = 2, q.n = w, q.k = f, q.dst = out;
      return ughip_product_row(dev, &q);
    });
    s.y = {y, 0, w};
  }
};

}  // namespace

void RopeTables::ensure(size_t n) {
  if (n <= rows) return;
  const size_t half = dims_ / 2;
  std::vector<float> c(n * half), s(n * half);
  for (size_t i = 0; i < half; ++i) {
    const double f = std::pow(base_, -2.0 * (double)i / (double)dims_);
    for (size_t p = 0; p < n; ++p) {
      const double a = (double)p * f;
      c[p * half + i] = (float)std::cos(a);
      s[p * half + i] = (float)std::sin(a);
    }
  }
  cos = LB::copy(c.data(), DType::F32, c.size(), Shape({n, half}), dev_);
  sin = LB::copy(s.data(), DType::F32, s.size(), Shape({n, half}), dev_);
  rows = n;
}

// ---- the model ------------------------------------------------------------------------------------------------------------
HybridModel::HybridModel(const Json& cfg, WeightSource& weights, Precision precision, const DevicePtr& dev) : dev_(dev), ops_(hip_ops()), precision_(precision) {
  vocab_ = cfg.size_at("vocab"), width_ = cfg.size_at("width");
  eps_ = (float)cfg.at("norm").num_at("eps");
  const Json& list = cfg.at("layers");
  if (list.kind != Json::Arr) bail("configuration: 'layers' is not a list");
  const size_t n_layers = list.arr.size();
  const Json* side = cfg.find("token_side");
  side_dim_ = side ? side->size_at("dim") : 0;
  Loader ld{weights, precision, dev};
  embed_ = ld.matrix("embed", {vocab_, width_});
  if (side_dim_) side_embed_ = ld.matrix("side.embed", {vocab_, n_layers * side_dim_});
  std::map<std::pair<double, size_t>, std::shared_ptr<RopeTables>> tables;
  // norms are stored around zero: the weight is 1 + what the file holds
  auto norm = [&](const std::string& name) { return ld.vec(name, width_, 1.f); };
  for (size_t i = 0; i < n_layers; ++i) {
    const Json& lc = list.arr[i];
    const Json& m = lc.at("mixer");
    const std::string p = "l" + std::to_string(i) + ".", type = lc.str_at("type");
    Layer l;
    if (type == "latent_attention") {
      const Json& rot = m.at("rot");
      const size_t dims = rot.size_at("dims");
      if (dims != m.size_at("rot_dim") || dims == 0 || dims % 2) bail("configuration: layer " + std::to_string(i) + " rotates " + std::to_string(dims) + " elements");
      std::shared_ptr<RopeTables>& tb = tables[{rot.num_at("base"), dims}];
      if (!tb) tables_.push_back(tb = std::make_shared<RopeTables>(rot.num_at("base"), dims, dev));
      if (m.find("kv_from")) {
        const size_t from = m.size_at("kv_from");
        if (from >= i || list.arr[from].str_at("type") != "latent_attention" || list.arr[from].at("mixer").find("kv_from") ||
            list.arr[from].at("mixer").size_at("kv_rank") != m.size_at("kv_rank") || list.arr[from].at("mixer").size_at("rot_dim") != dims)
          bail("configuration: layer " + std::to_string(i) + " reads the latents of layer " + std::to_string(from) + ", which has none that fit");
      }
      l.mixer = std::make_unique<LatentAttention>(m, p + "mix.", ld, width_, eps_, tb);
    } else if (type == "mamba2") {
      l.mixer = std::make_unique<Mamba2>(m, p + "mix.", ld, width_, eps_);
    } else {
      bail("configuration: unknown mixer '" + type + "'");
    }
    l.norm1 = norm(p + "norm1");
    if (const Json* mlp = lc.find("mlp")) {
      const std::string kind = mlp->str_at("kind");
      if (kind == "dense") l.mlp = std::make_unique<DenseFeedForward>(*mlp, p + "mlp.", ld, width_);
      else if (kind == "moe") l.mlp = std::make_unique<MoeFeedForward>(*mlp, p + "mlp.", ld, width_);
      else bail("configuration: unknown feed-forward '" + kind + "'");
      l.norm2 = norm(p + "norm2");
    }
    if (side_dim_) {
      l.side_gate = ld.matrix(p + "side.gate", {side_dim_, width_});
      l.side_proj = ld.matrix(p + "side.proj", {width_, side_dim_});
      l.side_norm = ld.vec(p + "side.norm", width_);
    }
    layers_.push_back(std::move(l));
  }
  final_norm_ = norm("final.norm");
  head_ = ld.matrix("head", {vocab_, width_});
}

std::unique_ptr<DecoderState> HybridModel::new_state(size_t max_tokens) const {
  auto st = std::make_unique<HybridState>();
  st->capacity = std::max<size_t>(1, max_tokens);
  for (const auto& t : tables_) t->ensure(st->capacity);
  for (const Layer& l : layers_) st->layers.push_back(l.mixer->new_state(st->capacity));
  return st;
}

void HybridModel::side(StepContext& c, Stream& s, const Layer& l, size_t index) const {
  Product p{l.side_gate, LB(), side_dim_, width_, UGHIP_ACT_GELU_MUL};
  p.table = side_embed_, p.ids = c.tokens;
  p.table_rows = vocab_, p.table_stride = layers_.size() * side_dim_, p.table_col = index * side_dim_;
  const Product proj{l.side_proj, LB(), width_, side_dim_};
  if (c.fused && std::max(width_, side_dim_) <= kRowStepMax) {
    size_t at, none;
    LB g = stream_step(c, s, {p}, &at);
    s.y = {row_step({g, at, side_dim_}, nullptr, 0, {proj}, &none), 0, width_};
  } else {
    settle(c, s);
    LB g = stream_product(c, s, p, half_type(c));
    s.y = {product_rows({g, 0, side_dim_}, c.t, proj), 0, width_};
  }
  s.norm = l.side_norm;
}

LB HybridModel::step(const LB& tokens, const LB&, DecoderState& state, const LB* rows, const std::function<void(const LB&)>* after_layer) const {
  HybridState* st = dynamic_cast<HybridState*>(&state);
  if (!st || st->layers.size() != layers_.size()) bail("this step needs a state of the same model");
  const size_t t = tokens.elem_count();
  if (t == 0) bail("a step without tokens");
  if (st->len + t > st->capacity) bail("a sequence of " + std::to_string(st->len) + " + " + std::to_string(t) + " positions exceeds its capacity of " + std::to_string(st->capacity));
  StepContext c{dev_, tokens, t, st->len, st->capacity, width_, eps_, st, precision_ == Precision::BF16 && t >= kHalfRows, t == 1 && !switch_on(SW_NO_FUSED_STEP)};
  Stream s;
  if (c.half_rows) s.x16 = scratch(DType::BF16, t * width_, dev_);
  s.x = {gather_rows(embed_, vocab_, width_, 0, width_, tokens, t, s.x16), 0, width_};
  for (size_t i = 0; i < layers_.size(); ++i) {
    const Layer& l = layers_[i];
    l.mixer->run(c, s, i);
    s.norm = l.norm1;
    if (l.mlp) {
      l.mlp->run(c, s);
      s.norm = l.norm2;
    }
    if (side_dim_) side(c, s, l, i);
    if (after_layer) {
      settle(c, s);
      (*after_layer)(s.x.lb);
    }
  }
  st->len += t;
  const Product head{head_, LB(), vocab_, width_};
  const bool one = width_ <= kRowStepMax && (c.fused ? !rows || rows->elem_count() == 1 : !rows && !switch_on(SW_NO_FUSED_STEP));
  if (one && c.t == 1 && s.top == 0) {
    size_t at;
    RowStep r{head};
    r.norm = final_norm_, r.eps = eps_;
    return row_step(s.x, &s, width_, r, &at, false);
  }
  settle(c, s);
  if (one) {
    // a prompt whose logits are read at the last position only
    size_t at;
    RowStep r{head};
    r.norm = final_norm_, r.eps = eps_;
    return row_step({s.x.lb, s.x.offset + (t - 1) * s.x.stride, width_}, nullptr, width_, r, &at);
  }
  Rows x = s.x;
  size_t r = 1;
  if (rows) {
    r = rows->elem_count();
    x = {gather_rows(x.lb, t, width_, 0, width_, *rows, r), 0, width_};
  } else {
    x.offset += (t - 1) * x.stride;
  }
  LB xn = norm_rows(x, r, width_, final_norm_, eps_);
  return product_rows({xn, 0, width_}, r, head);
}

}  // namespace ug_llama
