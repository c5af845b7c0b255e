// LatentAttention: attention without rotation whose keys and values are linear
// in a normed latent row per token, the only thing cached; each head's output
// is scaled by a sigmoid gate of the layer input.  Not part of the reference.
//
// Two equal forms: over many tokens keys and values are expanded from the latents
// for the matrix cores; over few, the expansions move to the other side of the
// scores - q -> W_uk^T q, output -> W_uv output - and attention runs on the
// latents themselves, which are then keys and values of all heads.
#ifndef __VKLLAMA_LATENT_ATTENTION_H__
#define __VKLLAMA_LATENT_ATTENTION_H__
#include "src/ops/row_mixer.h"

namespace vkllama
{
class LatentAttention : public RowMixer
{
public:
  LatentAttention (GPUDevice *dev, Command *command, const MixerParams &p);
  absl::Status load (const WeightSource &w, const std::string &prefix) override;
  int in_rows () const override;
  absl::Status pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const override;
  absl::StatusOr<std::vector<vkl_out_seg> > segments (int S, size_t offset, int run) override;
  absl::Status mix (int S, size_t offset, int run, void *out, size_t os) override;
  void describe (vkl_stack_layer &l, int run) override;
  size_t weight_bytes () const override { return ukt_.bytes () + uv_.bytes () + c_norm_.bytes (); }

protected:
  int cache_width_ () const override { return rank_; }

private:
  int c_row_ () const { return p_.heads * dim_; }
  int g_row_ () const { return c_row_ () + round_up (p_.kv_rank, 8); }
  int rank_ = 0;    // latent size, padded
  Tensor c_norm_;
  Tensor ukt_, uv_; // per head: [rank_, dim_] and [vdim_, rank_]
  Tensor ukv_;      // expansion: [heads*dim_ | heads*vdim_, rank_]
  Tensor c_, g_;    // fp32 down-projections and gates of the tokens at hand
  Tensor qa_, oa_;  // queries and outputs on the latent side, fp32
  Tensor kv_;       // expanded keys and values
};
}
#endif
