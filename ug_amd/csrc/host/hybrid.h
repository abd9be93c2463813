// Decoders whose layers are listed one by one in their configuration: every layer has a mixer (latent attention, a
// state-space recurrence, ...) and a feed-forward (dense, routed experts, none), with norms on the sublayers' outputs and,
// optionally, a token input per layer.  Tanolorn is such a design; its rules are hybrid.cpp's builder, the mechanisms are
// parts that another design can list as well.
#pragma once
#include <memory>
#include <string>
#include <vector>

#include "llama.h"

namespace ug_llama {

// m rows inside a buffer: row i starts at offset + i * stride.
struct Rows {
  LB lb;
  size_t offset = 0, stride = 0;
};

// Rotary angles of one (base, dims): tables [rows, dims / 2], grown when a longer sequence asks for more.
class RopeTables {
 public:
  RopeTables(double base, size_t dims, const ug::DevicePtr& dev) : base_(base), dims_(dims), dev_(dev) {}
  void ensure(size_t rows);
  LB cos, sin;
  size_t rows = 0;

 private:
  double base_;
  size_t dims_;
  ug::DevicePtr dev_;
};

// What a layer's mixer keeps for one sequence; the meaning of the buffers is the mixer's.
struct MixerState {
  std::vector<LB> buffers;
};

struct HybridState : DecoderState {
  std::vector<MixerState> layers;
};

// The stream between sublayers: the residual x, and a sublayer's output y that still has to be normed and added.  Whoever
// reads the stream next either folds that in or settles it with an op of its own.
struct Stream {
  Rows x, y;
  LB x16;  // the rows of x once more as bf16, where the step's products read that (valid only while nothing is pending)
  LB norm;  // weight of the pending norm; invalid: nothing is pending
  LB slots, weights;  // y is a weighted sum of `top` rows of y_rows (routed experts)
  size_t top = 0, y_rows = 0;
};

// What the parts of a layer see of a step.
struct StepContext {
  const ug::DevicePtr& dev;
  LB tokens;
  size_t t = 0, pos = 0, capacity = 0;
  size_t width = 0;
  float eps = 0;
  HybridState* state = nullptr;
  bool half_rows = false;  // products read bf16 rows (bf16 matrices and enough positions)
  bool fused = false;  // one position, with the neighbours of every product folded into its launch
};

class Mixer {
 public:
  virtual ~Mixer() = default;
  virtual MixerState new_state(size_t capacity) const = 0;
  // Consumes the stream (s.x is settled on return, nothing pending) and leaves the output as the new pending y.
  virtual void run(StepContext& c, Stream& s, size_t layer) const = 0;
};

class FeedForward {
 public:
  virtual ~FeedForward() = default;
  virtual void run(StepContext& c, Stream& s) const = 0;
};

class HybridModel : public Decoder {
 public:
  HybridModel(const ug::Json& config, WeightSource& weights, Precision precision, const ug::DevicePtr& dev);
  std::unique_ptr<DecoderState> new_state(size_t max_tokens) const override;
  LB step(const LB& tokens, const LB& pos, DecoderState& state, const LB* rows, const std::function<void(const LB&)>* after_layer) const override;
  size_t vocab_size() const override { return vocab_; }
  size_t max_positions() const override { return (size_t)1 << 30; }
  const ug::DevicePtr& device() const override { return dev_; }
  const Ops& ops() const override { return *ops_; }

 private:
  struct Layer {
    std::unique_ptr<Mixer> mixer;
    std::unique_ptr<FeedForward> mlp;
    LB norm1, norm2;  // (1 + the stored weight)
    LB side_gate, side_proj, side_norm;
  };
  void side(StepContext& c, Stream& s, const Layer& l, size_t index) const;
  ug::DevicePtr dev_;
  std::shared_ptr<Ops> ops_;
  Precision precision_;
  size_t vocab_ = 0, width_ = 0, side_dim_ = 0;
  float eps_ = 0;
  LB embed_, side_embed_, final_norm_, head_;
  std::vector<Layer> layers_;
  std::vector<std::shared_ptr<RopeTables>> tables_;
};

}  // namespace ug_llama
