// Fazinex: a decoder whose layers differ.  Every layer has one norm whose output
// feeds its token mixer and its feed-forward part in parallel; both add into an
// fp32 residual stream:
//   h = rms_norm (x) w;  x += mixer (h) + W_down relu (W_up h)^2
// Mixers: shared key/value attention and gated latent attention (src/ops).  The
// configuration may have a stretch of layers repeated, each run with a cache of
// its own.  The embedding table, normed on the way in, is the output matrix too; the
// logits are soft-capped.
//
// A layer is two products: [queries | keys or latent | gates | feed-forward up]
// of h, and [heads | feed-forward] back, added into x.  Weights are bf16;
// activations and caches are bf16 or fp32 (ModelOptions::dtype).
#ifndef __VKLLAMA_MODELS_FAZINEX_H__
#define __VKLLAMA_MODELS_FAZINEX_H__
#include "models/causal_model.h"
#include "models/json.h"
#include "models/registry.h"
#include "models/stack_plan.h"
#include "models/weights.h"
#include "src/core/command.h"
#include "src/ops/row_mixer.h"

namespace vkllama
{
struct FazinexConfig
{
  struct Layer
  {
    enum Type
    {
      SharedKV,
      Latent
    } type;
    RowMixerParams mixer; // sizes and factors; the rest is filled in by the model
    int ff = 0;           // 0: no feed-forward part
  };
  int vocab = 0, width = 0;
  float eps = 0.f, logit_softcap = 0.f; // 0: no soft cap
  std::vector<Layer> layers;
  std::vector<int> order;               // layer numbers in the order they run
  static absl::StatusOr<FazinexConfig> parse (const Json &config);
};

// y = x W^T with segmented outputs, and the one-norm layer around it
class ParallelBlock
{
public:
  struct Buffers // shared by the blocks of a model: they run in order
  {
    Tensor h;   // the normed input, [rows, width_p]
    Tensor cat; // what the second product reads, [rows, widest]
    int cat_stride = 0;
  };
  ParallelBlock (GPUDevice *dev, Command *command, const FazinexConfig &cfg, int index, int runs,
                 const ModelOptions &opt);
  absl::Status load (const WeightSource &w);
  // x [S, width_p] fp32, in place
  absl::Status operator() (Tensor &x, int S, size_t offset, int run, Buffers &b);
  void describe (vkl_stack_layer &l, int run);
  int out_width () const { return k_out_; }
  size_t weight_bytes () const { return weight_bytes_; }
  RowMixer &mixer () { return *mixer_; }

private:
  GPUDevice *dev_;
  Command *command_;
  std::string prefix_;
  int width_, width_p_, ff_, up_row_, ff_col_, k_out_, n_in_;
  float eps_;
  DType dtype_;
  size_t weight_bytes_ = 0;
  std::unique_ptr<RowMixer> mixer_;
  Tensor norm_, w_in_, w_out_;
};

class Fazinex : public CausalModel
{
public:
  ~Fazinex () override;
  static absl::StatusOr<std::unique_ptr<CausalModel> > create (const Json &config, const WeightSource &weights,
                                                               const ModelOptions &opt);
  size_t decode_step_bytes (size_t L) const override;
  // testing aid: the residual stream [layer runs, rows, width] of a pass on the
  // operator chain
  absl::StatusOr<std::vector<float> > residual_streams (std::vector<uint32_t> const &toks, size_t offset);

private:
  Fazinex () {}
  absl::Status init_ (const Json &config, const WeightSource &weights, const ModelOptions &opt);
  absl::StatusOr<Tensor> forward_ (std::vector<uint32_t> const &toks, const size_t offset,
                                   std::vector<uint32_t> const &rows) override;
  absl::Status pass_ (const uint32_t *toks, int S, size_t offset, std::vector<float> *streams);
  absl::Status logits_ (const std::vector<uint32_t> &rows, float *out);
  absl::Status wait_all_ () override;
  StepPlan *plan_ptr_ () override { return plan_.get (); }

  FazinexConfig cfg_;
  DType dtype_ = BF16;
  int width_p_ = 0;
  std::unique_ptr<Command> command_;
  std::vector<std::unique_ptr<ParallelBlock> > blocks_;
  ParallelBlock::Buffers buf_;
  Tensor embed_, embed_norm_, final_norm_;
  Tensor x_, toks_, rows_, out_h_;
  std::unique_ptr<StackPlan> plan_;
};
}
#endif
