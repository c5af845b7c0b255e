// Fuzuvik: a decoder whose layers mix tokens in one of three ways - attention within
// chunks, a gated delta rule with a decay per channel, or decaying sums - each
// followed by a feed-forward part with a norm of its own:
//   x += mixer (rms_norm (x) w1);  x += W_down gelu (W_up (rms_norm (x) w2))
// in an fp32 residual stream.  Embedding rows enter scaled; the output matrix is one
// of its own.
#ifndef __VKLLAMA_MODELS_FUZUVIK_H__
#define __VKLLAMA_MODELS_FUZUVIK_H__
#include "models/stack_model.h"

namespace vkllama
{
class ChunkedAttention;

struct FuzuvikConfig : StackConfig
{
  struct Layer
  {
    enum Type
    {
      Attention,
      Delta,
      Decay
    } type;
    MixerParams mixer; // sizes and factors; the rest is filled in by the model
    FeedForwardParams ff;
  };
  std::vector<Layer> layers;
  static absl::StatusOr<FuzuvikConfig> parse (const Json &config);
};

class Fuzuvik : public StackModel
{
public:
  static absl::StatusOr<std::unique_ptr<CausalModel> > create (const Json &config, const WeightSource &weights,
                                                               const ModelOptions &opt);

private:
  Fuzuvik () {}
  absl::Status make_block_ (int index, const MixerParams &common, std::unique_ptr<StackBlock> &block) override;
  std::vector<FuzuvikConfig::Layer> layers_;
  const WeightSource *weights_ = nullptr;      // while the model loads
  ChunkedAttention *first_mixed_ = nullptr;    // the first layer that mixes values
};
}
#endif
