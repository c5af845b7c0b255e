#include "src/ops/latent_attention.h"
#include "models/weights.h"
#include "src/core/command.h"
#include <algorithm>

namespace vkllama
{
// (keys and values share the padded head size: one attention kernel serves both)
LatentAttention::LatentAttention (GPUDevice *dev, Command *command, const MixerParams &p)
    : RowMixer (dev, command, p)
{
  dim_ = vdim_ = round_up (std::max (p.dim, p.vdim), 32);
  rank_ = round_up (p.kv_rank, 64);
}

absl::Status
LatentAttention::load (const WeightSource &w, const std::string &prefix)
{
  if (p_.kv_rank <= 0 || rank_ > 1024)
    return absl::InvalidArgumentError ("latent attention: latent sizes up to 1024 are supported");
  const int H = p_.heads;
  auto norm = w.vector (prefix + "dkv.norm", (size_t)p_.kv_rank);
  VKLLAMA_STATUS_OK (norm);
  auto uk = w.matrix (prefix + "uk", (size_t)H * p_.dim, (size_t)p_.kv_rank);
  VKLLAMA_STATUS_OK (uk);
  auto uv = w.matrix (prefix + "uv", (size_t)H * p_.vdim, (size_t)p_.kv_rank);
  VKLLAMA_STATUS_OK (uv);
  auto cn = upload_vector (dev_, command_, *norm, rank_);
  VKLLAMA_STATUS_OK (cn);
  c_norm_ = *cn;
  PackedMatrix t (H * rank_, dim_), v (H * vdim_, rank_), kv (H * (dim_ + vdim_), rank_);
  for (int h = 0; h < H; ++h)
    for (int d = 0; d < p_.dim; ++d)
      for (int r = 0; r < p_.kv_rank; ++r)
        t.data[((size_t)h * rank_ + r) * dim_ + d] = (*uk)[((size_t)h * p_.dim + d) * p_.kv_rank + r];
  v.put_heads (*uv, H, p_.vdim, vdim_, p_.kv_rank, 0);
  kv.put_heads (*uk, H, p_.dim, dim_, p_.kv_rank, 0);
  kv.put_heads (*uv, H, p_.vdim, vdim_, p_.kv_rank, H * dim_);
  auto dt = t.upload (dev_, command_);
  VKLLAMA_STATUS_OK (dt);
  auto dv = v.upload (dev_, command_);
  VKLLAMA_STATUS_OK (dv);
  ukt_ = *dt, uv_ = *dv;
  if (p_.dtype == BF16 && dim_ <= 256)
    {
      auto dkv = kv.upload (dev_, command_);
      VKLLAMA_STATUS_OK (dkv);
      ukv_ = *dkv;
    }
  return absl::OkStatus ();
}

int
LatentAttention::in_rows () const
{
  return g_row_ () + round_up (p_.heads, 8);
}

absl::Status
LatentAttention::pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  auto q = w.matrix (prefix + "q", (size_t)p_.heads * p_.dim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (q);
  auto c = w.matrix (prefix + "dkv", (size_t)p_.kv_rank, (size_t)p_.width);
  VKLLAMA_STATUS_OK (c);
  auto g = w.matrix (prefix + "g", (size_t)p_.heads, (size_t)p_.width);
  VKLLAMA_STATUS_OK (g);
  m.put_heads (*q, p_.heads, p_.dim, dim_, p_.width, 0);
  m.put (*c, p_.kv_rank, p_.width, c_row_ ());
  m.put (*g, p_.heads, p_.width, g_row_ ());
  return absl::OkStatus ();
}

absl::StatusOr<std::vector<vkl_out_seg> >
LatentAttention::segments (int S, size_t, int)
{
  const int nq = p_.heads * dim_, gs = round_up (p_.heads, 8);
  VKLLAMA_STATUS_OK (grow_ (q_, S, nq, dev_, p_.dtype));
  VKLLAMA_STATUS_OK (grow_ (c_, S, rank_, dev_, FP32));
  VKLLAMA_STATUS_OK (grow_ (g_, S, gs, dev_, FP32));
  return std::vector<vkl_out_seg>{
    { 0, nq, q_.data (), (size_t)nq, type_ (), 0, nullptr, 0.f },
    { c_row_ (), p_.kv_rank, c_.data (), (size_t)rank_, VKL_TYPE_F32, 0, nullptr, 0.f },
    { g_row_ (), p_.heads, g_.data (), (size_t)gs, VKL_TYPE_F32, 0, nullptr, 0.f }
  };
}

absl::Status
LatentAttention::mix (int S, size_t offset, int run, void *out, size_t os)
{
  const int H = p_.heads, gs = round_up (H, 8);
  const size_t nq = (size_t)H * dim_, na = (size_t)H * rank_;
  void *s = dev_->stream ();
  timer_.start (dev_);
  int err = vkl_rmsnorm_f32 ((const float *)c_.data (), (size_t)rank_, nullptr, S, p_.kv_rank,
                             (const float *)c_norm_.data (), p_.eps, cache_row_ (run, offset), type_ (),
                             (size_t)rank_, rank_, s);
  if (!err && (ukv_.size () == 0 || S <= kFewRows))
    {
      VKLLAMA_STATUS_OK (grow_ (qa_, S, (int)na, dev_, FP32));
      VKLLAMA_STATUS_OK (grow_ (oa_, S, (int)na, dev_, FP32));
      err = vkl_head_matvec (ukt_.data (), H, rank_, dim_, q_.data (), type_ (), nq, (size_t)dim_, qa_.data (),
                             VKL_TYPE_F32, na, (size_t)rank_, nullptr, 0, S, s);
      if (!err)
        {
          VKLLAMA_STATUS_OK (attend_rows_ (qa_.data (), VKL_TYPE_F32, na, run, 1, rank_, S, offset, oa_.data (),
                                           VKL_TYPE_F32, na));
          err = vkl_head_matvec (uv_.data (), H, vdim_, rank_, oa_.data (), VKL_TYPE_F32, na, (size_t)rank_, out,
                                 type_ (), os, (size_t)vdim_, (const float *)g_.data (), (size_t)gs, S, s);
        }
    }
  else if (!err)
    {
      const int L = (int)offset + S;
      const size_t nk = nq, nkv = 2 * nq;
      VKLLAMA_STATUS_OK (grow_ (kv_, L, (int)nkv, dev_, BF16));
      const vkl_out_seg seg = { 0, (int)nkv, kv_.data (), nkv, VKL_TYPE_BF16, 0, nullptr, 0.f };
      err = vkl_project_bf16w (cache_row_ (run, 0), VKL_TYPE_BF16, (size_t)rank_, ukv_.data (), L, (int)nkv, rank_,
                               &seg, 1, s);
      if (!err)
        err = vkl_attn_prefill_causal_bf16 (q_.data (), kv_.data (), (const uint16_t *)kv_.data () + nk, H, H, S, L,
                                            dim_, nq, nkv, nkv, p_.scale, p_.temp_coef, p_.temp_every,
                                            (const float *)g_.data (), (size_t)gs, out, os, s);
    }
  timer_.stop (dev_);
  return launch_status ("latent attention", err);
}

void
LatentAttention::describe (vkl_stack_layer &l, int run)
{
  l.mixer = VKL_MIX_LATENT;
  l.H = p_.heads, l.G = 1, l.dim = dim_, l.vdim = vdim_;
  l.rank = p_.kv_rank, l.rank_p = rank_;
  l.scale = p_.scale, l.temp_coef = p_.temp_coef, l.temp_every = p_.temp_every;
  l.kv0 = c_row_ (), l.g0 = g_row_ ();
  l.w_ukt = ukt_.data (), l.w_uv = uv_.data (), l.c_norm = (const float *)c_norm_.data ();
  l.cache = caches_[(size_t)run].data ();
}
}
