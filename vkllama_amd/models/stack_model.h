// StackModel: decoders whose layers differ from one another, around an fp32 residual
// stream: embedding, layers (StackBlock) in the order the configuration gives,
// final norm and output matrix; long prompts in portions; the one-token step from
// the blocks' descriptions (StackPlan).  Weights are bf16; activations and caches
// are bf16 or fp32 (ModelOptions::dtype).  A model family says what its configuration
// means and makes the blocks.
#ifndef __VKLLAMA_MODELS_STACK_MODEL_H__
#define __VKLLAMA_MODELS_STACK_MODEL_H__
#include "models/causal_model.h"
#include "models/json.h"
#include "models/registry.h"
#include "models/stack_plan.h"
#include "models/weights.h"
#include "src/core/command.h"
#include "src/ops/token_mixer.h"
#include <algorithm>
#include <memory>

namespace vkllama
{
// the feed-forward part of a layer, ff 0: none
struct FeedForwardParams
{
  int ff = 0;
  int act = VKL_ACT_NONE;
};

class StackBlock
{
public:
  struct Buffers // shared by the blocks of a model: they run in order
  {
    Tensor h;   // a normed input, [rows, width_p]
    Tensor cat; // what a product back into the residual stream reads, [rows, widest]
    int cat_stride = 0;
  };
  // name: "l0." etc.; mixer: made from parameters with the model's width, eps, ...
  StackBlock (GPUDevice *dev, Command *command, const std::string &name, std::unique_ptr<TokenMixer> mixer,
              const MixerParams &mp, const FeedForwardParams &ff);
  virtual ~StackBlock () {}
  virtual absl::Status load (const WeightSource &w) = 0;
  // x [S, width_p] fp32, in place
  virtual absl::Status operator() (Tensor &x, int S, size_t offset, int run, Buffers &b) = 0;
  virtual void describe (vkl_stack_layer &l, int run) = 0;
  // columns of `cat` the block needs
  virtual int cat_width () const = 0;
  size_t weight_bytes () const { return weight_bytes_ + mixer_->weight_bytes (); }
  TokenMixer &mixer () { return *mixer_; }

protected:
  absl::StatusOr<Tensor> norm_weights_ (const WeightSource &w, const std::string &name);
  // h = rms_norm (x) w
  absl::Status norm_input_ (Tensor &x, int S, Tensor &w, Buffers &b);
  // x += cat W^T over the first k columns of cat
  absl::Status add_product_ (Tensor &x, int S, Tensor &w, int k, Buffers &b);
  GPUDevice *dev_;
  Command *command_;
  std::string prefix_;
  int width_, width_p_;
  float eps_;
  DType dtype_;
  FeedForwardParams ff_;
  size_t weight_bytes_ = 0;
  std::unique_ptr<TokenMixer> mixer_;
};

// One norm feeds the mixer and the feed-forward part, both add into x.  A layer is
// two products: [the mixer's rows | feed-forward up] of h, and [heads |
// feed-forward] back.
class ParallelBlock : public StackBlock
{
public:
  ParallelBlock (GPUDevice *dev, Command *command, const std::string &name, std::unique_ptr<TokenMixer> mixer,
                 const MixerParams &mp, const FeedForwardParams &ff);
  absl::Status load (const WeightSource &w) override;
  absl::Status operator() (Tensor &x, int S, size_t offset, int run, Buffers &b) override;
  void describe (vkl_stack_layer &l, int run) override;
  int cat_width () const override { return k_out_; }

private:
  int up_row_, ff_col_, k_out_, n_in_;
  Tensor norm_, w_in_, w_out_;
};

// Two norms: x += mixer (norm1 (x)), then x += W_down act (W_up norm2 (x)).
class SequentialBlock : public StackBlock
{
public:
  SequentialBlock (GPUDevice *dev, Command *command, const std::string &name, std::unique_ptr<TokenMixer> mixer,
                   const MixerParams &mp, const FeedForwardParams &ff);
  absl::Status load (const WeightSource &w) override;
  absl::Status operator() (Tensor &x, int S, size_t offset, int run, Buffers &b) override;
  void describe (vkl_stack_layer &l, int run) override;
  int cat_width () const override { return std::max (k_out_, ff_p_); }

private:
  int n_in_, k_out_, ff_p_;
  Tensor norm1_, norm2_, w_in_, w_out_, w_up_, w_down_;
};

// what a family's configuration says about the model around its layers
struct StackConfig
{
  int vocab = 0, width = 0;
  float eps = 0.f;
  float logit_softcap = 0.f;  // 0: no soft cap
  float embed_scale = 1.f;    // factor of the embedding rows, where they are not normed
  bool embed_norm = false;    // rows normed with the weights "embed.norm"
  bool tied = false;          // the output matrix is "embed", else "head"
  std::vector<int> order;     // layer numbers in the order they run
};

class StackModel : public CausalModel
{
public:
  ~StackModel () override;
  size_t decode_step_bytes (size_t L) const override;
  // testing aid: the residual stream [layer runs, rows, width] of a pass on the
  // operator chain
  absl::StatusOr<std::vector<float> > residual_streams (std::vector<uint32_t> const &toks, size_t offset);

protected:
  StackModel () {}
  // makes the block of a layer, from parameters that have the model's part filled
  // in (sizes around the mixer, runs, format); called in the order of the layers
  virtual absl::Status make_block_ (int index, const MixerParams &common, std::unique_ptr<StackBlock> &block) = 0;
  absl::Status init_ (const StackConfig &cfg, int layers, const WeightSource &weights, const ModelOptions &opt);
  Command *command () { return command_.get (); }

private:
  absl::StatusOr<Tensor> forward_ (std::vector<uint32_t> const &toks, const size_t offset,
                                   std::vector<uint32_t> const &rows) override;
  absl::Status pass_ (const uint32_t *toks, int S, size_t offset, std::vector<float> *streams);
  absl::Status logits_ (const std::vector<uint32_t> &rows, float *out);
  absl::Status wait_all_ () override;
  StepPlan *plan_ptr_ () override { return plan_.get (); }

  StackConfig cfg_;
  DType dtype_ = BF16;
  int width_p_ = 0;
  std::unique_ptr<Command> command_;
  std::vector<std::unique_ptr<StackBlock> > blocks_;
  StackBlock::Buffers buf_;
  Tensor embed_, head_, embed_norm_, final_norm_;
  Tensor x_, toks_, rows_, out_h_;
  std::unique_ptr<StackPlan> plan_;
};
}
#endif
