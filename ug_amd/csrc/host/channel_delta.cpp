// A gated delta rule with a decay per key channel behind short convolutions, as a mixer of listed-layers decoders (hybrid.h).
#include <algorithm>

#include "hybrid_ops.h"

namespace ug_llama {

using namespace ug;

namespace {

struct ChannelDelta : Mixer {
  size_t heads, kv_heads, dim, vdim, taps, a_rank, z_rank, width;
  float eps;
  LB in;  // rows: q | k | v | what the decays and the output gate are made from | b
  LB conv, a_log, dt_bias, norm, norm_all, a2, g2, o;
  size_t inner() const { return heads * vdim; }
  size_t channels() const { return 2 * kv_heads * dim + inner(); }

  explicit ChannelDelta(const PartBuild& b) : width(b.width), eps(b.eps) {
    const Json& m = b.config;
    const std::string& p = b.prefix;
    heads = m.size_at("heads"), kv_heads = m.size_at("kv_heads"), dim = m.size_at("dim"), vdim = m.size_at("vdim"), taps = m.size_at("conv");
    if (!heads || !kv_heads || heads % kv_heads || !dim || !vdim || !taps)
      bail("configuration: layer " + std::to_string(b.index) + " has " + std::to_string(heads) + " heads on " + std::to_string(kv_heads) + " of " + std::to_string(dim) + " and " +
           std::to_string(vdim) + " elements behind " + std::to_string(taps) + " taps");
    a_rank = b.ld.rows_of(p + "a1", dim), z_rank = b.ld.rows_of(p + "g1", vdim);
    const size_t qk = kv_heads * dim;
    in = b.ld.stacked({{p + "q", qk}, {p + "k", qk}, {p + "v", inner()}, {p + "a1", a_rank}, {p + "g1", z_rank}, {p + "b", heads}}, width);
    conv = b.ld.stacked_f32({{p + "q.conv", qk}, {p + "k.conv", qk}, {p + "v.conv", inner()}}, taps);
    a2 = b.ld.matrix(p + "a2", {heads * dim, a_rank}), g2 = b.ld.matrix(p + "g2", {inner(), z_rank});
    a_log = b.ld.vec(p + "A_log", heads), dt_bias = b.ld.vec(p + "dt_bias", heads * dim);
    norm = b.ld.vec(p + "norm", vdim), norm_all = b.ld.vec(p + "norm", vdim, 0.f, 1.f, heads);
    o = b.ld.matrix(p + "o", {width, inner()});
  }

  MixerState new_state(size_t) const override {
    // contents are taken as zeros by the first step, whatever the memory held before
    return MixerState{{scratch(DType::F32, heads * dim * vdim, in.device()), scratch(DType::F32, taps * channels(), in.device())}};
  }

  void run(StepContext& c, Stream& s, size_t run) const override {
    const size_t t = c.t, pos = c.pos, I = inner(), ch = channels(), ra = a_rank, rz = z_rank, H = heads, hd = heads * dim, nt = taps, wide = ch + ra + rz + H;
    const LB S = c.state->layers[run].buffers[0], ring = c.state->layers[run].buffers[1];
    const Product first{in, LB(), wide, width}, last{o, LB(), width, I};
    ughip_delta q{};
    q.t = t, q.pos = pos, q.heads = H, q.kv_heads = kv_heads, q.dim = dim, q.vdim = vdim, q.eps = eps;
    if (c.fused && std::max(width, I) <= kRowStepMax && std::max(ra, rz) <= 4096) {
      size_t at, none;
      LB p = stream_step(c, s, {first}, &at);
      q.qkv_offset = at, q.a_offset = at + ch, q.z_offset = at + ch + ra, q.b_offset = at + ch + ra + rz, q.a_rank = ra, q.z_rank = rz, q.n_taps = nt;
      LB y = hip_op("delta_step", {p, conv, ring, a_log, dt_bias, a2, g2, S}, {1, 2 * I}, [=](ughip_device* d, const std::vector<ughip_slice*>& x, ughip_slice* out) {
        ughip_delta r = q;
        r.p = x[0], r.taps = x[1], r.ring = x[2], r.a_log = x[3], r.dt_bias = x[4], r.w_a = x[5], r.w_z = x[6], r.s = x[7], r.out = out;
        return ughip_delta_step(d, &r);
      });
      RowStep step{last};
      step.norm = norm_all, step.norm_groups = H, step.eps = eps, step.gate = y, step.gate_offset = I, step.gate_after = true;
      s.y = {row_step({y, 0, I}, nullptr, 0, step, &none), 0, width};
      return;
    }
    settle(c, s);
    LB p = stream_product(c, s, first);
    LB qkv = hip_op("conv_silu", {p, conv, ring}, {t, ch}, [=](ughip_device* d, const std::vector<ughip_slice*>& x, ughip_slice* out) {
      return ughip_conv_silu_rows(d, {x[0], 0, wide}, x[1], nullptr, nt, x[2], pos, t, ch, {out, 0, ch});
    });
    LB a = product_rows({p, ch, wide}, t, {a2, LB(), hd, ra}), z = product_rows({p, ch + ra, wide}, t, {g2, LB(), I, rz});
    LB y = hip_op("delta", {qkv, p, a, z, a_log, dt_bias, norm, S, ring}, {t, I}, [=](ughip_device* d, const std::vector<ughip_slice*>& x, ughip_slice* out) {
      if (int rc = ughip_conv_ring_store(d, {x[1], 0, wide}, nt, x[8], pos, t, ch)) return rc;
      ughip_delta r = q;
      r.qkv = {x[0], 0, ch}, r.b = {x[1], ch + ra + rz, wide}, r.a = {x[2], 0, hd}, r.z = {x[3], 0, I}, r.dst = {out, 0, I};
      r.a_log = x[4], r.dt_bias = x[5], r.norm = x[6], r.s = x[7];
      return ughip_delta_rows(d, &r);
    }, half_type(c));
    s.y = {product_rows({y, 0, I}, t, last), 0, width};
  }
};

}  // namespace

std::unique_ptr<Mixer> make_channel_delta(const PartBuild& b) { return std::make_unique<ChannelDelta>(b); }

}  // namespace ug_llama
