// SharedKVAttention: grouped-query attention in which one projection serves as
// keys and as values, without rotation; positions enter through the mask and a
// logarithmic factor on the queries.  Not part of the reference.
#ifndef __VKLLAMA_SHARED_KV_ATTENTION_H__
#define __VKLLAMA_SHARED_KV_ATTENTION_H__
#include "src/ops/row_mixer.h"

namespace vkllama
{
class SharedKVAttention : public RowMixer
{
public:
  SharedKVAttention (GPUDevice *dev, Command *command, const MixerParams &p);
  absl::Status load (const WeightSource &w, const std::string &prefix) override;
  int in_rows () const override;
  absl::Status pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const override;
  absl::StatusOr<std::vector<vkl_out_seg> > segments (int S, size_t offset, int run) override;
  absl::Status mix (int S, size_t offset, int run, void *out, size_t os) override;
  void describe (vkl_stack_layer &l, int run) override;

protected:
  int cache_width_ () const override { return p_.kv_heads * dim_; }
};
}
#endif
