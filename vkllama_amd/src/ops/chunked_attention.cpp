// Input rows: q (heads of dim_ rows) | k | v (kv_heads of dim_ rows each).  The
// product writes keys and values straight into their cache rows, where they are
// then rotated, normed and mixed in place.
#include "src/ops/chunked_attention.h"
#include "models/weights.h"
#include "src/core/command.h"
#include "vkl_hip.h"
#include <algorithm>

namespace vkllama
{
ChunkedAttention::ChunkedAttention (GPUDevice *dev, Command *command, const MixerParams &p, ChunkedAttention *first)
    : TokenMixer (dev, command, p), first_ (first)
{
  dim_ = vdim_ = round_up (std::max (p.dim, p.vdim), 32);
}

absl::Status
ChunkedAttention::init () noexcept
{
  VKLLAMA_STATUS_OK (TokenMixer::init ());
  if (dim_ > 1024)
    return absl::InvalidArgumentError ("attention: head sizes up to 1024 are supported");
  if (2 * p_.freq.size () > (size_t)p_.dim)
    return absl::InvalidArgumentError (absl::StrFormat (
        "attention: rotation over %zu values of a head of %d", 2 * p_.freq.size (), p_.dim));
  if (first_ && (first_->p_.kv_heads != p_.kv_heads || first_->p_.vdim != p_.vdim))
    return absl::InvalidArgumentError ("attention: layers that mix values need key/value heads of the same sizes");
  kcaches_.resize ((size_t)p_.runs), vcaches_.resize ((size_t)p_.runs);
  for (int i = 0; i < p_.runs; ++i)
    {
      VKLLAMA_STATUS_OK (grow_zeroed_ (kcaches_[(size_t)i], p_.maxlen, p_.kv_heads * dim_, p_.dtype));
      VKLLAMA_STATUS_OK (grow_zeroed_ (vcaches_[(size_t)i], p_.maxlen, p_.kv_heads * dim_, p_.dtype));
    }
  return absl::OkStatus ();
}

absl::Status
ChunkedAttention::load (const WeightSource &w, const std::string &prefix)
{
  if (p_.v_mix)
    {
      auto v = w.scalar (prefix + "vmix");
      VKLLAMA_STATUS_OK (v);
      mix_ = *v;
    }
  if (p_.freq.empty ())
    return absl::OkStatus ();
  const size_t bytes = p_.freq.size () * sizeof (double);
  freq_ = Tensor (1, 1, (int)bytes, dev_, INT8);
  VKLLAMA_STATUS_OK (freq_.create ());
  return command_->upload ((const int8_t *)p_.freq.data (), bytes, freq_);
}

int
ChunkedAttention::in_rows () const
{
  return (p_.heads + 2 * p_.kv_heads) * dim_;
}

absl::Status
ChunkedAttention::pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  auto q = w.matrix (prefix + "q", (size_t)p_.heads * p_.dim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (q);
  auto k = w.matrix (prefix + "k", (size_t)p_.kv_heads * p_.dim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (k);
  auto v = w.matrix (prefix + "v", (size_t)p_.kv_heads * p_.vdim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (v);
  m.put_heads (*q, p_.heads, p_.dim, dim_, p_.width, 0);
  m.put_heads (*k, p_.kv_heads, p_.dim, dim_, p_.width, p_.heads * dim_);
  m.put_heads (*v, p_.kv_heads, p_.vdim, dim_, p_.width, (p_.heads + p_.kv_heads) * dim_);
  return absl::OkStatus ();
}

absl::StatusOr<std::vector<vkl_out_seg> >
ChunkedAttention::segments (int S, size_t offset, int run)
{
  const int nq = p_.heads * dim_, nk = p_.kv_heads * dim_;
  VKLLAMA_STATUS_OK (grow_ (q_, S, nq, dev_, p_.dtype));
  return std::vector<vkl_out_seg>{
    { 0, nq, q_.data (), (size_t)nq, type_ (), VKL_ACT_NONE, nullptr, 0.f },
    { nq, nk, row_ (kcaches_[(size_t)run], offset), (size_t)nk, type_ (), VKL_ACT_NONE, nullptr, 0.f },
    { nq + nk, nk, row_ (vcaches_[(size_t)run], offset), (size_t)nk, type_ (), VKL_ACT_NONE, nullptr, 0.f }
  };
}

absl::Status
ChunkedAttention::mix (int S, size_t offset, int run, void *out, size_t os)
{
  const size_t nq = (size_t)p_.heads * dim_, nk = (size_t)p_.kv_heads * dim_;
  Tensor &kc = kcaches_[(size_t)run], &vc = vcaches_[(size_t)run];
  vkl_attn_rows_prep r = {};
  r.H = p_.heads, r.G = p_.kv_heads, r.dim = dim_, r.n = p_.dim, r.eps = p_.eps;
  r.npair = (int)p_.freq.size (), r.freq = (const double *)freq_.data ();
  r.q = r.qo = q_.data (), r.qs = r.qos = nq, r.qtype = r.qotype = r.kvtype = r.ctype = type_ ();
  r.k = row_ (kc, offset), r.ko = kc.data (), r.kvs = nk, r.vo = vc.data ();
  if (first_)
    r.v = row_ (vc, offset), r.first = first_->vcaches_[0].data (), r.fdim = first_->dim_, r.mix = mix_;
  timer_.start (dev_);
  int err = vkl_attn_prepare (&r, S, (uint32_t)offset, dev_->stream ());
  if (!err && (p_.dtype == FP32 || dim_ > 256 || S <= kFewRows))
    {
      const size_t need = vkl_attn_kv_rows_scratch_bytes (type_ (), p_.heads, p_.kv_heads, dim_, S);
      VKLLAMA_STATUS_OK (grow_zeroed_ (scratch_, 1, std::max ((int)need, (int)scratch_.width ()), INT8));
      err = vkl_attn_kv_rows (q_.data (), type_ (), nq, kc.data (), vc.data (), type_ (), nk, p_.heads, p_.kv_heads,
                              dim_, S, (uint32_t)offset, p_.scale, p_.chunk, p_.sink, out, type_ (), os,
                              scratch_.data (), dev_->stream ());
    }
  else if (!err)
    err = vkl_attn_prefill_chunked_bf16 (q_.data (), kc.data (), vc.data (), p_.heads, p_.kv_heads, S, (int)offset + S,
                                         dim_, nq, nk, nk, p_.scale, p_.chunk, p_.sink, out, os, dev_->stream ());
  timer_.stop (dev_);
  return launch_status ("chunked attention", err);
}

void
ChunkedAttention::describe (vkl_stack_layer &l, int run)
{
  l.mixer = VKL_MIX_KV;
  l.H = p_.heads, l.G = p_.kv_heads, l.dim = dim_, l.vdim = vdim_, l.n = p_.dim;
  l.scale = p_.scale, l.chunk = p_.chunk, l.sink = p_.sink;
  l.kv0 = p_.heads * dim_, l.v0 = (p_.heads + p_.kv_heads) * dim_;
  l.npair = (int)p_.freq.size (), l.freq = (const double *)freq_.data ();
  l.cache = kcaches_[(size_t)run].data (), l.vcache = vcaches_[(size_t)run].data ();
  l.vfirst = first_ ? first_->vcaches_[0].data () : nullptr, l.fdim = first_ ? first_->dim_ : 0, l.vmix = mix_;
}
}
