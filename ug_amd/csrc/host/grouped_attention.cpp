// Attention of query heads that share key / value heads in groups, as a mixer of listed-layers decoders (hybrid.h).
#include <algorithm>

#include "hybrid_ops.h"

namespace ug_llama {

using namespace ug;

namespace {

struct GroupedAttention : Mixer {
  size_t heads, kv_heads, dim, vdim, width, rot = 0, window = 0;
  float scale;
  std::shared_ptr<RopeTables> rope;        // may be null
  std::shared_ptr<QueryFactors> factors;   // may be null
  LB qkv, qkv_b, o;
  size_t wide() const { return (heads + kv_heads) * dim + kv_heads * vdim; }

  GroupedAttention(const PartBuild& b, bool bias, bool rotated, bool windowed, bool query_factors) : width(b.width) {
    const Json& m = b.config;
    const std::string &p = b.prefix, where = "configuration: layer " + std::to_string(b.index);
    heads = m.size_at("heads"), kv_heads = m.size_at("kv_heads"), dim = m.size_at("dim"), vdim = m.size_at("vdim");
    if (!heads || !kv_heads || heads % kv_heads) bail(where + " has " + std::to_string(heads) + " heads on " + std::to_string(kv_heads));
    scale = (float)m.num_at("scale");
    if (rotated) {
      const Json& r = m.at("rot");
      rot = r.size_at("dims");
      if (rot % 2 || rot > dim) bail(where + " rotates " + std::to_string(rot) + " elements of " + std::to_string(dim));
      if (rot) rope = b.rope(r.num_at("base"), rot, r.at("scaling").num_at("factor"));
    }
    if (windowed) {
      window = m.at("mask").size_at("size");
      if (!window) bail(where + " has a window of no positions");
    }
    if (query_factors) {
      const Json& t = m.at("q_temp");
      if (!(t.num_at("every") > 0)) bail(where + " changes its queries every " + std::to_string(t.num_at("every")) + " positions");
      factors = b.query_factors(t.num_at("coef"), t.num_at("every"));
    }
    qkv = b.ld.stacked({{p + "q", heads * dim}, {p + "k", kv_heads * dim}, {p + "v", kv_heads * vdim}}, width);
    if (bias) qkv_b = b.ld.stacked_vec({{p + "q.b", heads * dim}, {p + "k.b", kv_heads * dim}, {p + "v.b", kv_heads * vdim}});
    o = b.ld.matrix(p + "o", {width, heads * vdim});
    cache_sizes(1);  // (sizes the kernels are not built for are refused here)
  }

  struct Sizes {
    size_t rows, k, v;
  };
  Sizes cache_sizes(size_t capacity) const {
    Sizes z;
    if (ughip_grouped_attention_cache(kv_heads, dim, vdim, capacity, &z.rows, &z.k, &z.v)) bail(std::string("configuration: ") + ughip_last_error());
    return z;
  }

  MixerState new_state(size_t capacity) const override {
    const Sizes z = cache_sizes(capacity);
    return MixerState{{scratch(qkv.dtype(), z.k, qkv.device()), scratch(qkv.dtype(), z.v, qkv.device())}};
  }

  void run(StepContext& c, Stream& s, size_t run) const override {
    const size_t n = wide(), inner = heads * vdim;
    const Product in{qkv, qkv_b, n, width}, out{o, LB(), width, inner};
    const bool fused = c.fused && std::max(width, inner) <= kRowStepMax;
    size_t at = 0, none;
    LB p;
    if (fused) {
      p = stream_step(c, s, {in}, &at);
    } else {
      settle(c, s);
      p = stream_product(c, s, in);
    }
    const MixerState& st = c.state->layers[run];
    std::vector<LB> args = {p, st.buffers[0], st.buffers[1]};
    if (rope) args.push_back(rope->cos), args.push_back(rope->sin);
    if (factors) args.push_back(factors->values);
    ughip_attention q{};
    q.capacity = c.capacity, q.table_rows = rope ? rope->rows : 0, q.rot = rot, q.window = window;
    q.t = c.t, q.pos = c.pos, q.heads = heads, q.kv_heads = kv_heads, q.dim = dim, q.vdim = vdim, q.scale = scale;
    const bool turned = rope != nullptr, scaled = factors != nullptr;
    LB a = hip_op("grouped_attention", args, {c.t, inner}, [=](ughip_device* d, const std::vector<ughip_slice*>& x, ughip_slice* dst) {
      ughip_attention r = q;
      r.qkv = {x[0], at, n}, r.dst = {dst, 0, inner}, r.k_cache = x[1], r.v_cache = x[2];
      if (turned) r.cos = x[3], r.sin = x[4];
      if (scaled) r.q_factor = x[turned ? 5 : 3];
      return ughip_grouped_attention(d, &r);
    }, fused ? DType::F32 : half_type(c));
    if (fused) s.y = {row_step({a, 0, inner}, nullptr, 0, {out}, &none), 0, width};
    else s.y = {product_rows({a, 0, inner}, c.t, out), 0, width};
  }
};

}  // namespace

std::unique_ptr<Mixer> make_grouped_attention(const PartBuild& b, bool bias, bool rotated, bool windowed, bool query_factors) {
  return std::make_unique<GroupedAttention>(b, bias, rotated, windowed, query_factors);
}

}  // namespace ug_llama
