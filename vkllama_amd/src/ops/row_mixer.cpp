#include "src/ops/row_mixer.h"
#include "vkl_hip.h"

namespace vkllama
{
absl::Status
RowMixer::init () noexcept
{
  VKLLAMA_STATUS_OK (TokenMixer::init ());
  caches_.resize ((size_t)p_.runs);
  for (Tensor &c : caches_)
    VKLLAMA_STATUS_OK (grow_zeroed_ (c, p_.maxlen, cache_width_ (), p_.dtype));
  return absl::OkStatus ();
}

void *
RowMixer::cache_row_ (int run, size_t pos)
{
  Tensor &c = caches_[(size_t)run];
  return (uint8_t *)c.data () + pos * c.hs ();
}

absl::Status
RowMixer::attend_rows_ (const void *q, int qtype, size_t qs, int run, int groups, int dim, int S, size_t offset,
                        void *out, int otype, size_t os)
{
  const size_t need = vkl_attn_rows_scratch_bytes (type_ (), p_.heads, groups, dim, S);
  if (scratch_.bytes () < need)
    {
      scratch_ = Tensor (1, 1, (int)need, dev_, INT8);
      VKLLAMA_STATUS_OK (scratch_.create ());
      if (int e = vkl_memset (scratch_.data (), 0, need, dev_->stream ()))
        return launch_status ("clearing attention scratch", e);
    }
  Tensor &c = caches_[(size_t)run];
  return launch_status ("attention over rows",
                        vkl_attn_rows (q, qtype, qs, c.data (), type_ (), c.width (), p_.heads, groups, dim, S,
                                       (uint32_t)offset, p_.scale, p_.temp_coef, p_.temp_every, out, otype, os,
                                       scratch_.data (), dev_->stream ()));
}
}
