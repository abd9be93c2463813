#include "decoder.h"

#include <fstream>
#include <sstream>

#include "hybrid.h"
#include "llama.h"

namespace ug_llama {

using namespace ug;

namespace {

// A HF llama config.json (the fields of ug-llama/src/model.rs:10-24).
std::unique_ptr<Decoder> build_llama(const Json& c, WeightSource& w, Precision precision, const DevicePtr& dev) {
  Config cfg;
  cfg.hidden_size = c.size_at("hidden_size");
  cfg.intermediate_size = c.size_at("intermediate_size");
  cfg.max_position_embeddings = c.size_at("max_position_embeddings");
  cfg.num_attention_heads = c.size_at("num_attention_heads");
  cfg.num_key_value_heads = c.size_or("num_key_value_heads", cfg.num_attention_heads);
  cfg.num_hidden_layers = c.size_at("num_hidden_layers");
  cfg.rms_norm_eps = c.num_at("rms_norm_eps");
  cfg.rope_theta = (float)c.num_or("rope_theta", 10000.0);
  cfg.vocab_size = c.size_at("vocab_size");
  if (const Json* j = c.find("rope_interleaved")) cfg.rope_interleaved = j->num != 0;
  if (const Json* j = c.find("tie_word_embeddings")) cfg.tie_word_embeddings = j->num != 0;
  auto m = std::make_unique<Model>(cfg, true, w, dev, hip_ops(precision == Precision::BF16));
  m->set_fused_attention(3);
  if (precision == Precision::BF16) m->store_matrices_bf16();
  return m;
}

DecoderBuilder hybrid(const HybridDesign& (*design)()) {
  return [design](const Json& c, WeightSource& w, Precision precision, const DevicePtr& dev) { return std::make_unique<HybridModel>(design(), c, w, precision, dev); };
}

std::string read_file(const std::string& path) {
  std::ifstream f(path, std::ios::binary);
  if (!f) bail("cannot read " + path);
  std::stringstream s;
  s << f.rdbuf();
  return s.str();
}

}  // namespace

std::map<std::string, DecoderBuilder>& decoder_registry() {
  static std::map<std::string, DecoderBuilder> r = {{"Tanolorn", hybrid(tanolorn_design)}, {"Tugelorn", hybrid(tugelorn_design)}, {"LlamaForCausalLM", build_llama}, {"llama", build_llama}};
  return r;
}

std::unique_ptr<Decoder> build_decoder(const Json& config, WeightSource& weights, Precision precision, const DevicePtr& dev) {
  std::vector<std::string> names;
  if (const Json* j = config.find("architecture")) names.push_back(j->str);
  if (const Json* j = config.find("architectures"))
    for (const Json& e : j->arr) names.push_back(e.str);
  if (const Json* j = config.find("model_type")) names.push_back(j->str);
  for (const std::string& n : names) {
    auto it = decoder_registry().find(n);
    if (it != decoder_registry().end()) return it->second(config, weights, precision, dev);
  }
  std::string known;
  for (const auto& kv : decoder_registry()) known += (known.empty() ? "" : ", ") + kv.first;
  bail("configuration: no model named '" + (names.empty() ? std::string() : names[0]) + "' (known: " + known + ")");
}

std::unique_ptr<Decoder> load_decoder(const std::string& dir, Precision precision, const DevicePtr& dev) {
  const std::string path = dir + "/config.json", text = read_file(path);
  JsonParser jp{text.data(), text.data() + text.size(), path};
  const Json config = jp.value(0);
  auto w = safetensors_weights({dir + "/model.safetensors"});
  return build_decoder(config, *w, precision, dev);
}

std::vector<float> decoder_step(const Decoder& model, DecoderState& state, const std::vector<int32_t>& tokens, const std::vector<int32_t>& want, CompilationCache& cache,
                                std::vector<std::vector<float>>* hidden) {
  if (tokens.empty()) bail("a step without tokens");
  for (int32_t id : tokens)
    if (id < 0 || (size_t)id >= model.vocab_size()) bail("id " + std::to_string(id) + " is outside the vocabulary of " + std::to_string(model.vocab_size()));
  for (int32_t w : want)
    if (w < 0 || (size_t)w >= tokens.size()) bail("logits of place " + std::to_string(w) + " among " + std::to_string(tokens.size()) + " tokens");
  const DevicePtr& dev = model.device();
  model.prepare();
  LB ids = LB::copy(tokens.data(), DType::I32, tokens.size(), Shape({1, tokens.size()}), dev);
  const int32_t p = (int32_t)state.len;
  LB pos = LB::copy(&p, DType::I32, 1, Shape({1, 1}), dev), rows;
  if (!want.empty()) rows = LB::copy(want.data(), DType::I32, want.size(), Shape({1, want.size()}), dev);
  const std::function<void(const LB&)> keep = [&](const LB& x) {
    std::vector<float> v(x.elem_count());
    x.data_vec(v.data(), DType::F32);
    hidden->push_back(std::move(v));
  };
  LB logits = model.step(ids, pos, state, want.empty() ? nullptr : &rows, hidden ? &keep : nullptr);
  CompiledSchedule compiled = Schedule::create_one(logits).compile_and_run(cache);
  state.settle();
  std::vector<float> out;
  if (!want.empty()) {
    out.resize(logits.elem_count());
    logits.data_vec(out.data(), DType::F32);
  } else {
    dev->synchronize();
  }
  return out;
}

}  // namespace ug_llama
