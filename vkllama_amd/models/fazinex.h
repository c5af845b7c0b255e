// Fazinex: a decoder whose layers differ.  Every layer has one norm whose output
// feeds its token mixer and its feed-forward part in parallel; both add into an
// fp32 residual stream:
//   h = rms_norm (x) w;  x += mixer (h) + W_down relu (W_up h)^2
// Mixers: shared key/value attention and gated latent attention (src/ops).  The
// configuration may have a stretch of layers repeated, each run with a cache of
// its own.  The embedding table, normed on the way in, is the output matrix too; the
// logits are soft-capped.
#ifndef __VKLLAMA_MODELS_FAZINEX_H__
#define __VKLLAMA_MODELS_FAZINEX_H__
#include "models/stack_model.h"

namespace vkllama
{
struct FazinexConfig : StackConfig
{
  struct Layer
  {
    enum Type
    {
      SharedKV,
      Latent
    } type;
    MixerParams mixer; // sizes and factors; the rest is filled in by the model
    FeedForwardParams ff;
  };
  std::vector<Layer> layers;
  static absl::StatusOr<FazinexConfig> parse (const Json &config);
};

class Fazinex : public StackModel
{
public:
  static absl::StatusOr<std::unique_ptr<CausalModel> > create (const Json &config, const WeightSource &weights,
                                                               const ModelOptions &opt);

private:
  Fazinex () {}
  absl::Status make_block_ (int index, const MixerParams &common, std::unique_ptr<StackBlock> &block) override;
  std::vector<FazinexConfig::Layer> layers_;
};
}
#endif
