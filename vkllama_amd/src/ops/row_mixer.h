// RowMixer: a token mixer whose cached rows serve as keys and values at once.  A
// projection writes the rows in place.
#ifndef __VKLLAMA_ROW_MIXER_H__
#define __VKLLAMA_ROW_MIXER_H__
#include "src/ops/token_mixer.h"

namespace vkllama
{
class RowMixer : public TokenMixer
{
public:
  RowMixer (GPUDevice *dev, Command *command, const MixerParams &p) : TokenMixer (dev, command, p) {}
  absl::Status init () noexcept override;
  size_t row_bytes () const override { return caches_.empty () ? 0 : caches_[0].hs (); }

protected:
  void *cache_row_ (int run, size_t pos);
  virtual int cache_width_ () const = 0;
  // attention over a cache with the row kernel (values = keys)
  absl::Status attend_rows_ (const void *q, int qtype, size_t qs, int run, int groups, int dim, int S, size_t offset,
                             void *out, int otype, size_t os);
  std::vector<Tensor> caches_;
  Tensor q_, scratch_;
};
}
#endif
