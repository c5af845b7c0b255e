// RecurrentMixer: token mixers that keep a state of fixed size per head instead of
// rows, in fp32.  A pass at position 0 starts from an empty state; any other
// continues from the state the pass before it left.  Not part of the reference.
#ifndef __VKLLAMA_RECURRENT_MIXER_H__
#define __VKLLAMA_RECURRENT_MIXER_H__
#include "src/ops/token_mixer.h"

namespace vkllama
{
class RecurrentMixer : public TokenMixer
{
public:
  RecurrentMixer (GPUDevice *dev, Command *command, const MixerParams &p);
  absl::Status init () noexcept override;
  size_t state_bytes () const override { return states_.empty () ? 0 : states_[0].bytes (); }
  size_t rows_read (size_t) const override { return 0; }

protected:
  // the projections q | k | v of the tokens at hand: columns and their places
  int qk_cols_ () const { return p_.kv_heads * dim_; }
  int qkv_cols_ () const { return 2 * qk_cols_ () + p_.heads * vdim_; }
  absl::Status pack_qkv_ (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const;
  // a vector per head, in padded heads
  absl::StatusOr<Tensor> upload_heads_ (const std::vector<float> &v, int n, int np);
  // runs the recurrence over qkv [S, qkv_cols_] into o_; a: what is particular to the mixer
  absl::Status recur_ (vkl_recurrence_args a, const void *qkv, int S, size_t offset, int run);
  void sizes_ (vkl_recurrence_args &a) const;
  void describe_ (vkl_stack_layer &l, int run);
  std::vector<Tensor> states_;
  Tensor qkv_, o_, scratch_;
};

// The gated delta rule with a decay per key channel: q, k, v pass a short
// convolution, q and k become unit vectors, a head's output is normed and gated.
// Decays and gates come from the layer input through two matrices of low rank each.
class ChannelDelta : public RecurrentMixer
{
public:
  using RecurrentMixer::RecurrentMixer;
  absl::Status load (const WeightSource &w, const std::string &prefix) override;
  int in_rows () const override { return g_row_ () + r_g_; }
  absl::Status pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const override;
  absl::StatusOr<std::vector<vkl_out_seg> > segments (int S, size_t offset, int run) override;
  absl::Status mix (int S, size_t offset, int run, void *out, size_t os) override;
  void describe (vkl_stack_layer &l, int run) override;
  size_t weight_bytes () const override { return w_a2_.bytes () + w_g2_.bytes () + conv_.bytes (); }
  // (the ranks are the tensors' shapes: read before in_rows)
  absl::Status read_ranks (const WeightSource &w, const std::string &prefix);

private:
  int b_row_ () const { return qkv_cols_ (); }
  int a_row_ () const { return b_row_ () + round_up (p_.heads, 8); }
  int g_row_ () const { return a_row_ () + r_a_; }
  int rank_a_ = 0, rank_g_ = 0; // of the decays and the gates
  int r_a_ = 0, r_g_ = 0;       // padded to multiples of 64
  float qscale_ = 1.f;
  Tensor conv_, w_a2_, w_g2_, dt_bias_, rate_, norm_;
  std::vector<Tensor> rings_;   // the convolution's last inputs
  Tensor conv_out_, b_, a1_, g1_, z_;
};

// Linear attention whose state decays by a constant factor per head ("lightning"):
// SiLU on q, k and v; the concatenated heads are normed together and gated.
class DecayAttention : public RecurrentMixer
{
public:
  using RecurrentMixer::RecurrentMixer;
  absl::Status load (const WeightSource &w, const std::string &prefix) override;
  int in_rows () const override { return qkv_cols_ () + p_.heads * vdim_; }
  absl::Status pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const override;
  absl::StatusOr<std::vector<vkl_out_seg> > segments (int S, size_t offset, int run) override;
  absl::Status mix (int S, size_t offset, int run, void *out, size_t os) override;
  void describe (vkl_stack_layer &l, int run) override;

private:
  Tensor log_decay_, norm_, gate_;
};
}
#endif
