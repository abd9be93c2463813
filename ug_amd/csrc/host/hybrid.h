// Decoders whose layers are listed one by one in their configuration: every layer has a mixer (latent or grouped attention, a
// state-space recurrence, a delta rule, ...) and a feed-forward (dense, routed experts, none), with norms on the sublayers' outputs
// and, optionally, in front of them, a token input per layer, and a range of layers that runs several times.  Tanolorn and Tugelorn
// are such designs: a HybridDesign says what distinguishes them, the mechanisms are parts that another design can list as well.
#pragma once
#include <functional>
#include <map>
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

// What depends on a position only: tables with a row per position, grown when a longer sequence asks for more.
class PositionTables {
 public:
  virtual ~PositionTables() = default;
  virtual void ensure(size_t rows) = 0;
  size_t rows = 0;
};

// Rotary angles position * base^(-2 i / dims) / factor: [rows, dims / 2].
class RopeTables : public PositionTables {
 public:
  RopeTables(double base, size_t dims, double factor, const ug::DevicePtr& dev) : base_(base), factor_(factor), dims_(dims), dev_(dev) {}
  void ensure(size_t rows) override;
  LB cos, sin;

 private:
  double base_, factor_;
  size_t dims_;
  ug::DevicePtr dev_;
};

// What queries are multiplied by, 1 + coef ln(floor((position + 1) / every) + 1): [rows].
class QueryFactors : public PositionTables {
 public:
  QueryFactors(double coef, double every, const ug::DevicePtr& dev) : coef_(coef), every_(every), dev_(dev) {}
  void ensure(size_t rows) override;
  LB values;

 private:
  double coef_, every_;
  ug::DevicePtr dev_;
};

// What a layer's mixer keeps for one sequence; the meaning of the buffers is the mixer's.
struct MixerState {
  std::vector<LB> buffers;
};

struct HybridState : DecoderState {
  std::vector<MixerState> layers;  // one per layer run
};

// The stream between sublayers: the residual x, and a sublayer's output y that still has to be normed and added.  Whoever
// reads the stream next either folds that in or settles it with an op of its own.
struct Stream {
  Rows x, y;
  LB x16;  // the rows of x once more as bf16, where the step's products read that (valid only while nothing is pending)
  LB norm;  // weight of the pending norm; invalid: nothing is pending
  Rows extra;  // rows that join x besides, as they are
  // A norm in front of the sublayer to come, and the rows of x normed by it (made by the op of h_by) once settled.
  LB ahead, h, h_by;
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
  bool norm_ahead = false;  // sublayers have a norm in front of them
};

class Mixer {
 public:
  virtual ~Mixer() = default;
  virtual MixerState new_state(size_t capacity) const = 0;
  // Consumes the stream (s.x is settled on return, nothing pending) and leaves the output as the new pending y.  `run`: which of the
  // step's layer runs this is, and with it whose state.
  virtual void run(StepContext& c, Stream& s, size_t run) const = 0;
};

class FeedForward {
 public:
  virtual ~FeedForward() = default;
  virtual void run(StepContext& c, Stream& s) const = 0;
};

struct Loader;
// What the builder of a layer's part sees.
struct PartBuild {
  const ug::Json& layers;  // the whole list
  size_t index;            // this layer
  const ug::Json& config;  // the part's own
  std::string prefix;      // of its tensors
  const Loader& ld;
  size_t width;
  float eps;
  std::function<std::shared_ptr<RopeTables>(double base, size_t dims, double factor)> rope;
  std::function<std::shared_ptr<QueryFactors>(double coef, double every)> query_factors;
};
using MixerBuilder = std::function<std::unique_ptr<Mixer>(const PartBuild&)>;
using FeedForwardBuilder = std::function<std::unique_ptr<FeedForward>(const PartBuild&)>;

// A design of listed layers.
struct HybridDesign {
  bool norm_ahead = false;         // tensors norm1, norm2 stand in front of the sublayers and norm1b, norm2b behind; else norm1, norm2 behind
  float norm_base = 0.f;           // norm weights are this plus what is stored
  const char* residual_mult = nullptr;  // the key of what sublayer outputs are multiplied by
  std::map<std::string, MixerBuilder> mixers;        // by a layer's type
  std::map<std::string, FeedForwardBuilder> mlps;    // by kind
};
const HybridDesign& tanolorn_design();
const HybridDesign& tugelorn_design();

// Mixers in files of their own.
std::unique_ptr<Mixer> make_grouped_attention(const PartBuild& b, bool bias, bool rotated, bool windowed, bool query_factors);
std::unique_ptr<Mixer> make_channel_delta(const PartBuild& b);

class HybridModel : public Decoder {
 public:
  HybridModel(const HybridDesign& design, const ug::Json& config, WeightSource& weights, Precision precision, const ug::DevicePtr& dev);
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
    LB ahead1, ahead2;  // in front of the sublayers, where the design has norms there
    LB norm1, norm2;    // on their outputs (times what these are multiplied by)
    LB side_gate, side_proj, side_norm;
  };
  // A layer's turn; the layers of the configuration's loop have several, with a state each.
  struct Run {
    size_t layer;
    bool again;  // a pass but the first starts here: the embedding joins the residual
  };
  void side(StepContext& c, Stream& s, const Layer& l, size_t index) const;
  ug::DevicePtr dev_;
  std::shared_ptr<Ops> ops_;
  Precision precision_;
  size_t vocab_ = 0, width_ = 0, side_dim_ = 0;
  float eps_ = 0;
  LB embed_, side_embed_, final_norm_, head_;
  std::vector<Layer> layers_;
  std::vector<Run> runs_;
  bool norm_ahead_ = false;
  std::vector<std::shared_ptr<PositionTables>> tables_;
};

}  // namespace ug_llama
