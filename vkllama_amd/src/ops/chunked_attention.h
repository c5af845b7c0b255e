// ChunkedAttention: grouped-query attention over keys and values of their own.
// Queries and keys are rotated and then divided by their root mean square; a
// position sees its own chunk of positions; the softmax may have a sink; values
// may be mixed with those of the first layer that does so.  Each of these is a
// parameter (MixerParams).  Not part of the reference.
//
// Keys and values share a padded head size: one attention kernel serves both.
// Values are cached as they enter the attention, so the first mixing layer's cache
// is where the others find its values.
#ifndef __VKLLAMA_CHUNKED_ATTENTION_H__
#define __VKLLAMA_CHUNKED_ATTENTION_H__
#include "src/ops/token_mixer.h"

namespace vkllama
{
class ChunkedAttention : public TokenMixer
{
public:
  // first: the first layer that mixes values (null: this is it, or values are not mixed)
  ChunkedAttention (GPUDevice *dev, Command *command, const MixerParams &p, ChunkedAttention *first);
  absl::Status init () noexcept override;
  absl::Status load (const WeightSource &w, const std::string &prefix) override;
  int in_rows () const override;
  absl::Status pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const override;
  absl::StatusOr<std::vector<vkl_out_seg> > segments (int S, size_t offset, int run) override;
  absl::Status mix (int S, size_t offset, int run, void *out, size_t os) override;
  void describe (vkl_stack_layer &l, int run) override;
  size_t row_bytes () const override { return kcaches_.empty () ? 0 : 2 * kcaches_[0].hs (); }
  size_t rows_read (size_t pos) const override { return p_.chunk ? pos % (size_t)p_.chunk + 1 : pos + 1; }

private:
  void *row_ (Tensor &cache, size_t pos) { return (uint8_t *)cache.data () + pos * cache.hs (); }
  ChunkedAttention *first_;
  float mix_ = 0.f;
  std::vector<Tensor> kcaches_, vcaches_;
  Tensor freq_, q_, scratch_;
};
}
#endif
