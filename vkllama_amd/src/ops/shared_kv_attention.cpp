// Input rows: q (heads of dim_ rows) | k (kv_heads of dim_ rows).  The product
// writes k straight into the cache; attention then runs on the matrix cores
// (many query rows, bf16) or on the row kernel (few rows, fp32, wide heads).
#include "src/ops/shared_kv_attention.h"
#include "models/weights.h"
#include "src/core/command.h"

namespace vkllama
{
SharedKVAttention::SharedKVAttention (GPUDevice *dev, Command *command, const MixerParams &p)
    : RowMixer (dev, command, p)
{
  dim_ = vdim_ = round_up (p.dim, 32);
}

absl::Status
SharedKVAttention::load (const WeightSource &, const std::string &)
{
  if (p_.vdim != p_.dim)
    return absl::InvalidArgumentError (absl::StrFormat (
        "attention whose values are its keys: value size %d differs from key size %d", p_.vdim, p_.dim));
  if (dim_ > 1024)
    return absl::InvalidArgumentError ("attention: head sizes up to 1024 are supported");
  return absl::OkStatus ();
}

int
SharedKVAttention::in_rows () const
{
  return (p_.heads + p_.kv_heads) * dim_;
}

absl::Status
SharedKVAttention::pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  auto q = w.matrix (prefix + "q", (size_t)p_.heads * p_.dim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (q);
  auto k = w.matrix (prefix + "k", (size_t)p_.kv_heads * p_.dim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (k);
  m.put_heads (*q, p_.heads, p_.dim, dim_, p_.width, 0);
  m.put_heads (*k, p_.kv_heads, p_.dim, dim_, p_.width, p_.heads * dim_);
  return absl::OkStatus ();
}

absl::StatusOr<std::vector<vkl_out_seg> >
SharedKVAttention::segments (int S, size_t offset, int run)
{
  const int nq = p_.heads * dim_, nk = p_.kv_heads * dim_;
  VKLLAMA_STATUS_OK (grow_ (q_, S, nq, dev_, p_.dtype));
  return std::vector<vkl_out_seg>{
    { 0, nq, q_.data (), (size_t)nq, type_ (), 0, nullptr, 0.f },
    { nq, nk, cache_row_ (run, offset), (size_t)nk, type_ (), 0, nullptr, 0.f }
  };
}

absl::Status
SharedKVAttention::mix (int S, size_t offset, int run, void *out, size_t os)
{
  const size_t nq = (size_t)p_.heads * dim_, nk = (size_t)p_.kv_heads * dim_;
  timer_.start (dev_);
  absl::Status st = absl::OkStatus ();
  if (p_.dtype == FP32 || dim_ > 256 || S <= kFewRows)
    st = attend_rows_ (q_.data (), type_ (), nq, run, p_.kv_heads, dim_, S, offset, out, type_ (), os);
  else
    {
      const void *rows = caches_[(size_t)run].data ();
      st = launch_status ("attention",
                          vkl_attn_prefill_causal_bf16 (q_.data (), rows, rows, p_.heads, p_.kv_heads, S,
                                                        (int)offset + S, dim_, nq, nk, nk, p_.scale, p_.temp_coef,
                                                        p_.temp_every, nullptr, 0, out, os, dev_->stream ()));
    }
  timer_.stop (dev_);
  return st;
}

void
SharedKVAttention::describe (vkl_stack_layer &l, int run)
{
  l.mixer = VKL_MIX_SHARED_KV;
  l.H = p_.heads, l.G = p_.kv_heads, l.dim = dim_, l.vdim = vdim_;
  l.scale = p_.scale, l.temp_coef = p_.temp_coef, l.temp_every = p_.temp_every;
  l.kv0 = p_.heads * dim_;
  l.cache = caches_[(size_t)run].data ();
}
}
