#include "hybrid.h"

#include <algorithm>
#include <cmath>

#include "hybrid_ops.h"

namespace ug_llama {

using namespace ug;

namespace {

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

  void run(StepContext& c, Stream& s, size_t run) const override {
    const bool own = kv_from < 0;
    const size_t t = c.t, pos = c.pos, cap = c.capacity, H = heads, d = dim, r = rot, v = vdim, rk = rank, qr = q_rank, all = pos + t;
    const size_t wide = qr + (own ? rk + r : 0), trows = rope->rows;
    const float e = eps, sc = scale;
    const LB cache = c.state->layers[own ? run : (size_t)kv_from].buffers[0];
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

  void run(StepContext& c, Stream& s, size_t run) const override {
    const size_t t = c.t, pos = c.pos, I = inner(), ch = channels(), H = heads, vd = vdim, N = state, G = groups, nt = taps, wide = I + ch + H, ng = norm_groups;
    const float e = eps;
    const LB S = c.state->layers[run].buffers[0], ring = c.state->layers[run].buffers[1];
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
  int act;
  Glu glu;
  // act: UGHIP_ACT_SWIGLU, or UGHIP_ACT_GLU as `glu` says
  DenseFeedForward(const PartBuild& b, bool bias, int act_, const Glu& glu_) : width(b.width), act(act_), glu(glu_) {
    const std::string& p = b.prefix;
    ff = b.config.size_at("ff");
    gate_up = b.ld.stacked({{p + "gate", ff}, {p + "up", ff}}, width);
    down = b.ld.matrix(p + "down", {width, ff});
    if (bias) gate_up_b = b.ld.stacked_vec({{p + "gate.b", ff}, {p + "up.b", ff}}), down_b = b.ld.vec(p + "down.b", width);
  }
  void run(StepContext& c, Stream& s) const override {
    Product first{gate_up, gate_up_b, ff, width, act};
    first.glu = glu;
    const Product second{down, down_b, width, ff};
    if (c.fused && std::max(width, ff) <= kRowStepMax) {
      size_t at, none;
      LB a = stream_step(c, s, {first}, &at);
      s.y = {row_step({a, at, ff}, nullptr, 0, {second}, &none), 0, width};
      return;
    }
    settle(c, s, true);
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
    const double f = std::pow(base_, -2.0 * (double)i / (double)dims_) / factor_;
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

void QueryFactors::ensure(size_t n) {
  if (n <= rows) return;
  std::vector<float> v(n);
  for (size_t p = 0; p < n; ++p) v[p] = (float)(1.0 + coef_ * std::log(std::floor((double)(p + 1) / every_) + 1.0));
  values = LB::copy(v.data(), DType::F32, n, Shape({n}), dev_);
  rows = n;
}

// ---- designs ----------------------------------------------------------------------------------------------------------------
const HybridDesign& tanolorn_design() {
  static const HybridDesign design = [] {
    HybridDesign d;
    d.norm_base = 1.f;
    d.mixers["latent_attention"] = [](const PartBuild& b) -> std::unique_ptr<Mixer> {
      const Json &m = b.config, &rot = m.at("rot");
      const size_t dims = rot.size_at("dims");
      if (dims != m.size_at("rot_dim") || dims == 0 || dims % 2) bail("configuration: layer " + std::to_string(b.index) + " rotates " + std::to_string(dims) + " elements");
      if (m.find("kv_from")) {
        const size_t from = m.size_at("kv_from");
        const std::vector<Json>& all = b.layers.arr;
        if (from >= b.index || all[from].str_at("type") != "latent_attention" || all[from].at("mixer").find("kv_from") ||
            all[from].at("mixer").size_at("kv_rank") != m.size_at("kv_rank") || all[from].at("mixer").size_at("rot_dim") != dims)
          bail("configuration: layer " + std::to_string(b.index) + " reads the latents of layer " + std::to_string(from) + ", which has none that fit");
      }
      return std::make_unique<LatentAttention>(m, b.prefix, b.ld, b.width, b.eps, b.rope(rot.num_at("base"), dims, 1.0));
    };
    d.mixers["mamba2"] = [](const PartBuild& b) { return std::make_unique<Mamba2>(b.config, b.prefix, b.ld, b.width, b.eps); };
    d.mlps["dense"] = [](const PartBuild& b) { return std::make_unique<DenseFeedForward>(b, true, (int)UGHIP_ACT_SWIGLU, Glu()); };
    d.mlps["moe"] = [](const PartBuild& b) { return std::make_unique<MoeFeedForward>(b.config, b.prefix, b.ld, b.width); };
    return d;
  }();
  return design;
}

const HybridDesign& tugelorn_design() {
  static const HybridDesign design = [] {
    HybridDesign d;
    d.norm_ahead = true;
    d.residual_mult = "residual_mult";
    d.mixers["attention"] = [](const PartBuild& b) { return make_grouped_attention(b, false, true, true, false); };
    d.mixers["attention_2"] = [](const PartBuild& b) { return make_grouped_attention(b, true, false, false, true); };
    d.mixers["channel_delta"] = make_channel_delta;
    d.mlps["dense"] = [](const PartBuild& b) {
      const double limit = b.config.num_at("limit");
      if (!(limit > 0)) bail("configuration: a feed-forward with the limit " + std::to_string(limit));
      return std::make_unique<DenseFeedForward>(b, false, (int)UGHIP_ACT_GLU, Glu{1.702f, 1.f, (float)limit});
    };
    return d;
  }();
  return design;
}

// ---- the model ------------------------------------------------------------------------------------------------------------
HybridModel::HybridModel(const HybridDesign& design, const Json& cfg, WeightSource& weights, Precision precision, const DevicePtr& dev)
    : dev_(dev), ops_(hip_ops()), precision_(precision), norm_ahead_(design.norm_ahead) {
  vocab_ = cfg.size_at("vocab"), width_ = cfg.size_at("width");
  eps_ = (float)cfg.at("norm").num_at("eps");
  const float mult = design.residual_mult ? (float)cfg.num_at(design.residual_mult) : 1.f;
  const Json& list = cfg.at("layers");
  if (list.kind != Json::Arr) bail("configuration: 'layers' is not a list");
  const size_t n_layers = list.arr.size();
  const Json* side = cfg.find("token_side");
  side_dim_ = side ? side->size_at("dim") : 0;
  Loader ld{weights, precision, dev};
  embed_ = ld.matrix("embed", {vocab_, width_});
  if (side_dim_) side_embed_ = ld.matrix("side.embed", {vocab_, n_layers * side_dim_});
  std::map<std::vector<double>, std::shared_ptr<RopeTables>> ropes;
  std::map<std::vector<double>, std::shared_ptr<QueryFactors>> factors;
  auto rope = [&](double base, size_t dims, double factor) {
    std::shared_ptr<RopeTables>& tb = ropes[{base, (double)dims, factor}];
    if (!tb) tables_.push_back(tb = std::make_shared<RopeTables>(base, dims, factor, dev));
    return tb;
  };
  auto query_factors = [&](double coef, double every) {
    std::shared_ptr<QueryFactors>& tb = factors[{coef, every}];
    if (!tb) tables_.push_back(tb = std::make_shared<QueryFactors>(coef, every, dev));
    return tb;
  };
  auto norm = [&](const std::string& name, float times = 1.f) { return ld.vec(name, width_, design.norm_base, times); };
  const char* behind = norm_ahead_ ? "b" : "";
  for (size_t i = 0; i < n_layers; ++i) {
    const Json& lc = list.arr[i];
    const std::string p = "l" + std::to_string(i) + ".", type = lc.str_at("type");
    auto part = [&](const Json& config, const char* name) { return PartBuild{list, i, config, p + name, ld, width_, eps_, rope, query_factors}; };
    Layer l;
    const auto mixer = design.mixers.find(type);
    if (mixer == design.mixers.end()) bail("configuration: unknown mixer '" + type + "'");
    l.mixer = mixer->second(part(lc.at("mixer"), "mix."));
    if (norm_ahead_) l.ahead1 = norm(p + "norm1");
    l.norm1 = norm(p + "norm1" + behind, mult);
    if (const Json* mlp = lc.find("mlp")) {
      const std::string kind = mlp->str_at("kind");
      const auto ff = design.mlps.find(kind);
      if (ff == design.mlps.end()) bail("configuration: unknown feed-forward '" + kind + "'");
      l.mlp = ff->second(part(*mlp, "mlp."));
      if (norm_ahead_) l.ahead2 = norm(p + "norm2");
      l.norm2 = norm(p + "norm2" + behind, mult);
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
  size_t start = 0, stop = 0, times = 1;
  if (const Json* loop = cfg.find("loop")) {
    start = loop->size_at("start"), stop = loop->size_at("stop"), times = loop->size_at("times");
    if (start > stop || stop > n_layers || times == 0)
      bail("configuration: layers " + std::to_string(start) + " .. " + std::to_string(stop) + " of " + std::to_string(n_layers) + " run " + std::to_string(times) + " times");
  }
  for (size_t i = 0; i < start; ++i) runs_.push_back({i, false});
  for (size_t pass = 0; pass < times; ++pass)
    for (size_t i = start; i < stop; ++i) runs_.push_back({i, pass > 0 && i == start});
  for (size_t i = stop; i < n_layers; ++i) runs_.push_back({i, false});
}

std::unique_ptr<DecoderState> HybridModel::new_state(size_t max_tokens) const {
  auto st = std::make_unique<HybridState>();
  st->capacity = std::max<size_t>(1, max_tokens);
  for (const auto& t : tables_) t->ensure(st->capacity);
  for (const Run& r : runs_) st->layers.push_back(layers_[r.layer].mixer->new_state(st->capacity));
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
  if (!st || st->layers.size() != runs_.size()) bail("this step needs a state of the same model");
  const size_t t = tokens.elem_count();
  if (t == 0) bail("a step without tokens");
  if (st->len + t > st->capacity) bail("a sequence of " + std::to_string(st->len) + " + " + std::to_string(t) + " positions exceeds its capacity of " + std::to_string(st->capacity));
  StepContext c{dev_, tokens, t, st->len, st->capacity, width_, eps_, st, precision_ == Precision::BF16 && t >= kHalfRows, t == 1 && !switch_on(SW_NO_FUSED_STEP), norm_ahead_};
  Stream s;
  if (c.half_rows && !norm_ahead_) s.x16 = scratch(DType::BF16, t * width_, dev_);
  s.x = {gather_rows(embed_, vocab_, width_, 0, width_, tokens, t, s.x16), 0, width_};
  const Rows embedded = s.x;
  // a sublayer, with the norm in front of it where there is one
  auto sublayer = [&](const LB& ahead, auto&& run) {
    s.ahead = ahead;
    run();
    s.ahead = s.h = s.h_by = LB();
  };
  for (size_t i = 0; i < runs_.size(); ++i) {
    const Layer& l = layers_[runs_[i].layer];
    if (runs_[i].again) s.extra = embedded;
    sublayer(l.ahead1, [&] { l.mixer->run(c, s, i); });
    s.norm = l.norm1;
    if (l.mlp) {
      sublayer(l.ahead2, [&] { l.mlp->run(c, s); });
      s.norm = l.norm2;
    }
    if (side_dim_) side(c, s, l, runs_[i].layer);
    if (after_layer) {
      // (the next layer's norm goes with it where nothing else comes first)
      if (!c.fused && i + 1 < runs_.size() && !runs_[i + 1].again) s.ahead = layers_[runs_[i + 1].layer].ahead1;
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
