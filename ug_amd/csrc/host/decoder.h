// What a decoder-only model is to the loops that drive it (generate_greedy, decoder_step): a step over new tokens of one
// sequence, with whatever the sequence keeps between steps behind DecoderState.  Model families register a builder under the
// name their config.json gives (`architecture`, `architectures[0]` or `model_type`).
#pragma once
#include <functional>
#include <map>
#include <memory>
#include <string>
#include <vector>

#include "ug/json.h"
#include "ug/lazy_buffer.h"

namespace ug_llama {

using LB = ug::LazyBuffer;
struct Ops;
struct WeightSource;

// What one sequence keeps between steps.  Dropping it gives its buffers back to the device's pool.
struct DecoderState {
  virtual ~DecoderState() = default;
  size_t len = 0;       // positions whose graph has been built so far
  size_t capacity = 0;  // positions it has room for (0: it grows)
  // Called between building a step's graph and building the next one: buffers this step writes become leaves.
  virtual void settle() {}
};

class Decoder {
 public:
  virtual ~Decoder() = default;
  virtual std::unique_ptr<DecoderState> new_state(size_t max_tokens) const = 0;
  // The graph of one step: tokens I32 [1, t] follow what `state` holds; pos I32 [1, 1] holds state.len (models that know the
  // position on the host do not read it).  Logits [.., r, vocab]: of the positions listed in `rows` (I32 [1, r], indexes into
  // this step's tokens), or of the last one at least (its row is the last) when rows is null.
  // after_layer, when given, is called with the hidden state behind every layer.
  virtual LB step(const LB& tokens, const LB& pos, DecoderState& state, const LB* rows, const std::function<void(const LB&)>* after_layer) const = 0;
  virtual size_t vocab_size() const = 0;
  virtual size_t max_positions() const = 0;  // of one sequence
  virtual void prepare() const {}            // realises what every step shares
  virtual const ug::DevicePtr& device() const = 0;
  virtual const Ops& ops() const = 0;
};

enum class Precision {
  F32,   // matrices and products in f32
  BF16,  // matrices kept and multiplied as bf16, everything else f32
};

using DecoderBuilder = std::function<std::unique_ptr<Decoder>(const ug::Json& config, WeightSource& weights, Precision precision, const ug::DevicePtr& dev)>;
std::map<std::string, DecoderBuilder>& decoder_registry();
// The registered builder for a parsed config.json; the error names what is registered.
std::unique_ptr<Decoder> build_decoder(const ug::Json& config, WeightSource& weights, Precision precision, const ug::DevicePtr& dev);
// A model folder: config.json and model.safetensors.
std::unique_ptr<Decoder> load_decoder(const std::string& dir, Precision precision, const ug::DevicePtr& dev);

// One step of one sequence, run to the end: logits [want.size(), vocab] of the wanted places among `tokens`.
// hidden != nullptr: receives the residual behind every layer, [layers][t, width].
std::vector<float> decoder_step(const Decoder& model, DecoderState& state, const std::vector<int32_t>& tokens, const std::vector<int32_t>& want,
                                ug::CompilationCache& cache, std::vector<std::vector<float>>* hidden = nullptr);

}  // namespace ug_llama
