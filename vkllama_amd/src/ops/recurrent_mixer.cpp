#include "src/ops/recurrent_mixer.h"
#include "models/weights.h"
#include "src/core/command.h"
#include "vkl_hip.h"
#include <algorithm>
#include <cmath>
#include <string.h>

namespace vkllama
{
namespace
{
// inside the root of the unit vectors of the delta rule
constexpr float kUnitEps = 1e-6f;
// tokens whose products the chunked form holds at once
constexpr int kPiece = 2048;

vkl_out_seg
segment (int row, int n, Tensor &y, int type, int act)
{
  return { row, n, y.data (), y.width (), type, act, nullptr, 0.f };
}
}

RecurrentMixer::RecurrentMixer (GPUDevice *dev, Command *command, const MixerParams &p) : TokenMixer (dev, command, p)
{
  dim_ = round_up (p.dim, 32), vdim_ = round_up (p.vdim, 32);
}

absl::Status
RecurrentMixer::init () noexcept
{
  VKLLAMA_STATUS_OK (TokenMixer::init ());
  if (dim_ > 256 || vdim_ > 256)
    return absl::InvalidArgumentError ("recurrent mixer: head sizes up to 256 are supported");
  states_.resize ((size_t)p_.runs);
  for (Tensor &s : states_)
    VKLLAMA_STATUS_OK (grow_zeroed_ (s, p_.heads * dim_, vdim_, FP32));
  return absl::OkStatus ();
}

absl::Status
RecurrentMixer::pack_qkv_ (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  const int nqk = qk_cols_ ();
  for (int i = 0; i < 2; ++i)
    {
      auto x = w.matrix (prefix + (i ? "k" : "q"), (size_t)p_.kv_heads * p_.dim, (size_t)p_.width);
      VKLLAMA_STATUS_OK (x);
      m.put_heads (*x, p_.kv_heads, p_.dim, dim_, p_.width, i * nqk);
    }
  auto v = w.matrix (prefix + "v", (size_t)p_.heads * p_.vdim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (v);
  m.put_heads (*v, p_.heads, p_.vdim, vdim_, p_.width, 2 * nqk);
  return absl::OkStatus ();
}

absl::StatusOr<Tensor>
RecurrentMixer::upload_heads_ (const std::vector<float> &v, int n, int np)
{
  const size_t heads = v.size () / (size_t)n;
  std::vector<float> z (heads * (size_t)np, 0.f);
  for (size_t h = 0; h < heads; ++h)
    std::copy (v.begin () + h * (size_t)n, v.begin () + (h + 1) * (size_t)n, z.begin () + h * (size_t)np);
  return upload_vector (dev_, command_, z, (int)z.size ());
}

absl::Status
RecurrentMixer::recur_ (vkl_recurrence_args a, const void *qkv, int S, size_t offset, int run)
{
  const size_t es = p_.dtype == FP32 ? 4 : 2, nqk = (size_t)qk_cols_ ();
  const int no = p_.heads * vdim_;
  VKLLAMA_STATUS_OK (grow_ (o_, S, no, dev_, FP32));
  sizes_ (a);
  a.q = qkv, a.k = (const uint8_t *)qkv + nqk * es, a.v = (const uint8_t *)qkv + 2 * nqk * es;
  a.type = type_ (), a.qs = a.ks = a.vs = (size_t)qkv_cols_ ();
  a.state = (float *)states_[(size_t)run].data ();
  a.out = (float *)o_.data (), a.os = (size_t)no;
  if (vkl_recurrence_chunked (&a, S))
    {
      const size_t need = vkl_recurrence_scratch_bytes (&a, std::min (S, kPiece)), row = 4096;
      VKLLAMA_STATUS_OK (grow_ (scratch_, (int)((need + row - 1) / row), (int)row / 4, dev_, FP32));
    }
  return launch_status ("recurrence", vkl_recurrence (&a, S, (uint32_t)offset, VKL_RECUR_AUTO, scratch_.data (),
                                                      scratch_.bytes (), dev_->stream ()));
}

void
RecurrentMixer::sizes_ (vkl_recurrence_args &a) const
{
  a.H = p_.heads, a.rep = p_.heads / p_.kv_heads, a.dim = dim_, a.vdim = vdim_;
}

void
RecurrentMixer::describe_ (vkl_stack_layer &l, int run)
{
  l.H = p_.heads, l.G = p_.kv_heads, l.dim = dim_, l.vdim = vdim_, l.n = p_.dim, l.vn = p_.vdim;
  l.kv0 = qk_cols_ (), l.v0 = 2 * qk_cols_ ();
  l.state = (float *)states_[(size_t)run].data ();
}

// ---------------------------------------------------------------------------
// delta rule
// ---------------------------------------------------------------------------
absl::Status
ChannelDelta::read_ranks (const WeightSource &w, const std::string &prefix)
{
  for (int i = 0; i < 2; ++i)
    {
      auto t = w.find (prefix + (i ? "g1" : "a1"));
      VKLLAMA_STATUS_OK (t);
      if (t->shape.size () != 2 || t->shape[0] < 1 || t->shape[0] > 4096)
        return absl::InvalidArgumentError ("model tensor " + prefix + (i ? "g1" : "a1")
                                           + ": a matrix of at most 4096 rows is needed");
      (i ? rank_g_ : rank_a_) = (int)t->shape[0];
    }
  r_a_ = round_up (rank_a_, 64), r_g_ = round_up (rank_g_, 64);
  return absl::OkStatus ();
}

absl::Status
ChannelDelta::load (const WeightSource &w, const std::string &prefix)
{
  if (p_.taps < 1 || p_.taps > 16)
    return absl::InvalidArgumentError ("short convolution: 1 to 16 taps are supported");
  const int H = p_.heads, G = p_.kv_heads, n = qkv_cols_ ();
  qscale_ = (float)(1.0 / std::sqrt ((double)p_.dim));
  // convolution weights [taps, columns of q | k | v]
  std::vector<float> conv ((size_t)p_.taps * n, 0.f);
  const char *names[3] = { "q.conv", "k.conv", "v.conv" };
  int at = 0;
  for (int i = 0; i < 3; ++i)
    {
      const int heads = i < 2 ? G : H, hn = i < 2 ? p_.dim : p_.vdim, hp = i < 2 ? dim_ : vdim_;
      auto c = w.matrix (prefix + names[i], (size_t)heads * hn, (size_t)p_.taps);
      VKLLAMA_STATUS_OK (c);
      for (int h = 0; h < heads; ++h)
        for (int d = 0; d < hn; ++d)
          for (int j = 0; j < p_.taps; ++j)
            {
              const uint32_t u = (uint32_t)(*c)[((size_t)h * hn + d) * p_.taps + j] << 16;
              memcpy (&conv[(size_t)j * n + at + h * hp + d], &u, 4);
            }
      at += heads * hp;
    }
  VKL_TAKE (conv_, upload_vector (dev_, command_, conv, (int)conv.size ()));
  auto dt = w.vector (prefix + "dt_bias", (size_t)H * p_.dim);
  VKLLAMA_STATUS_OK (dt);
  VKL_TAKE (dt_bias_, upload_heads_ (*dt, p_.dim, dim_));
  auto al = w.vector (prefix + "A_log", (size_t)H);
  VKLLAMA_STATUS_OK (al);
  for (float &x : *al)
    x = (float)std::exp ((double)x);
  VKL_TAKE (rate_, upload_vector (dev_, command_, *al, H));
  auto norm = w.vector (prefix + "norm", (size_t)p_.vdim);
  VKLLAMA_STATUS_OK (norm);
  VKL_TAKE (norm_, upload_heads_ (*norm, p_.vdim, vdim_));
  auto a2 = w.matrix (prefix + "a2", (size_t)H * p_.dim, (size_t)rank_a_);
  VKLLAMA_STATUS_OK (a2);
  auto g2 = w.matrix (prefix + "g2", (size_t)H * p_.vdim, (size_t)rank_g_);
  VKLLAMA_STATUS_OK (g2);
  PackedMatrix pa (H * dim_, r_a_), pg (H * vdim_, r_g_);
  pa.put_heads (*a2, H, p_.dim, dim_, rank_a_, 0);
  pg.put_heads (*g2, H, p_.vdim, vdim_, rank_g_, 0);
  VKL_TAKE (w_a2_, pa.upload (dev_, command_));
  VKL_TAKE (w_g2_, pg.upload (dev_, command_));
  rings_.resize ((size_t)p_.runs);
  for (Tensor &r : rings_)
    VKLLAMA_STATUS_OK (grow_zeroed_ (r, p_.taps, n, FP32));
  return absl::OkStatus ();
}

absl::Status
ChannelDelta::pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  VKLLAMA_STATUS_OK (pack_qkv_ (w, prefix, m));
  const struct
  {
    const char *name;
    int n, row;
  } parts[3] = { { "b", p_.heads, b_row_ () }, { "a1", rank_a_, a_row_ () }, { "g1", rank_g_, g_row_ () } };
  for (const auto &p : parts)
    {
      auto x = w.matrix (prefix + p.name, (size_t)p.n, (size_t)p_.width);
      VKLLAMA_STATUS_OK (x);
      m.put (*x, p.n, p_.width, p.row);
    }
  return absl::OkStatus ();
}

absl::StatusOr<std::vector<vkl_out_seg> >
ChannelDelta::segments (int S, size_t, int)
{
  // (rows behind a rank are zero in the matrix: the padding of a1 and g1 is written)
  VKLLAMA_STATUS_OK (grow_ (qkv_, S, qkv_cols_ (), dev_, p_.dtype));
  VKLLAMA_STATUS_OK (grow_ (b_, S, round_up (p_.heads, 8), dev_, FP32));
  VKLLAMA_STATUS_OK (grow_ (a1_, S, r_a_, dev_, p_.dtype));
  VKLLAMA_STATUS_OK (grow_ (g1_, S, r_g_, dev_, p_.dtype));
  return std::vector<vkl_out_seg>{ segment (0, qkv_cols_ (), qkv_, type_ (), VKL_ACT_NONE),
                                   segment (b_row_ (), p_.heads, b_, VKL_TYPE_F32, VKL_ACT_NONE),
                                   segment (a_row_ (), r_a_, a1_, type_ (), VKL_ACT_NONE),
                                   segment (g_row_ (), r_g_, g1_, type_ (), VKL_ACT_NONE) };
}

absl::Status
ChannelDelta::mix (int S, size_t offset, int run, void *out, size_t os)
{
  const int nz = p_.heads * dim_, no = p_.heads * vdim_, n = qkv_cols_ ();
  void *s = dev_->stream ();
  VKLLAMA_STATUS_OK (grow_ (conv_out_, S, n, dev_, p_.dtype));
  timer_.start (dev_);
  int err = vkl_short_conv_silu (qkv_.data (), type_ (), (size_t)n, (const float *)conv_.data (), n, p_.taps,
                                 (float *)rings_[(size_t)run].data (), (uint32_t)offset, S, conv_out_.data (),
                                 (size_t)n, s);
  vkl_recurrence_args a = {};
  a.qscale = qscale_, a.unit_eps = kUnitEps;
  a.b = (const float *)b_.data (), a.bs = b_.width ();
  a.dt_bias = (const float *)dt_bias_.data (), a.rate = (const float *)rate_.data ();
  sizes_ (a);
  if (vkl_recurrence_chunked (&a, S))
    a.a1 = a1_.data (), a.as = (size_t)r_a_, a.w_a2 = w_a2_.data (), a.r_a = r_a_;
  else
    {
      VKLLAMA_STATUS_OK (grow_ (z_, S, nz, dev_, FP32));
      const vkl_out_seg zs = segment (0, nz, z_, VKL_TYPE_F32, VKL_ACT_NONE);
      if (!err)
        err = vkl_project_bf16w (a1_.data (), type_ (), (size_t)r_a_, w_a2_.data (), S, nz, r_a_, &zs, 1, s);
      a.z = (const float *)z_.data (), a.zs = (size_t)nz;
    }
  VKLLAMA_STATUS_OK (launch_status ("delta rule inputs", err));
  VKLLAMA_STATUS_OK (recur_ (a, conv_out_.data (), S, offset, run));
  err = vkl_low_rank_gated_norm ((const float *)o_.data (), (size_t)no, p_.heads, vdim_, p_.vdim,
                                 (const float *)norm_.data (), p_.eps, g1_.data (), (size_t)r_g_, w_g2_.data (), r_g_,
                                 type_ (), S, out, os, s);
  timer_.stop (dev_);
  return launch_status ("delta rule output", err);
}

void
ChannelDelta::describe (vkl_stack_layer &l, int run)
{
  l.mixer = VKL_MIX_DELTA;
  describe_ (l, run);
  l.b0 = b_row_ (), l.a0 = a_row_ (), l.g0 = g_row_ (), l.taps = p_.taps;
  l.r_a = r_a_, l.r_g = r_g_, l.w_a2 = w_a2_.data (), l.w_g2 = w_g2_.data ();
  l.conv = (const float *)conv_.data (), l.ring = (float *)rings_[(size_t)run].data ();
  l.dt_bias = (const float *)dt_bias_.data (), l.rate = (const float *)rate_.data ();
  l.gnorm = (const float *)norm_.data ();
  l.qscale = qscale_, l.unit_eps = kUnitEps;
}

// ---------------------------------------------------------------------------
// decaying sums
// ---------------------------------------------------------------------------
absl::Status
DecayAttention::load (const WeightSource &w, const std::string &prefix)
{
  if (p_.kv_heads != p_.heads || p_.decay.size () != (size_t)p_.heads)
    return absl::InvalidArgumentError ("decaying sums: one decay and one key head per head are needed");
  std::vector<float> ld;
  for (double d : p_.decay)
    ld.push_back ((float)std::max (std::log (d), -1.0e4));
  VKL_TAKE (log_decay_, upload_vector (dev_, command_, ld, p_.heads));
  auto norm = w.vector (prefix + "norm", (size_t)p_.heads * p_.vdim);
  VKLLAMA_STATUS_OK (norm);
  // (as long as a row of the output matrix: the one-token step norms that many)
  std::vector<float> z ((size_t)round_up (p_.heads * vdim_, 64), 0.f);
  for (int h = 0; h < p_.heads; ++h)
    std::copy (norm->begin () + h * p_.vdim, norm->begin () + (h + 1) * p_.vdim, z.begin () + h * vdim_);
  VKL_TAKE (norm_, upload_vector (dev_, command_, z, (int)z.size ()));
  return absl::OkStatus ();
}

absl::Status
DecayAttention::pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  VKLLAMA_STATUS_OK (pack_qkv_ (w, prefix, m));
  auto g = w.matrix (prefix + "g", (size_t)p_.heads * p_.vdim, (size_t)p_.width);
  VKLLAMA_STATUS_OK (g);
  m.put_heads (*g, p_.heads, p_.vdim, vdim_, p_.width, qkv_cols_ ());
  return absl::OkStatus ();
}

absl::StatusOr<std::vector<vkl_out_seg> >
DecayAttention::segments (int S, size_t, int)
{
  VKLLAMA_STATUS_OK (grow_ (qkv_, S, qkv_cols_ (), dev_, p_.dtype));
  VKLLAMA_STATUS_OK (grow_ (gate_, S, p_.heads * vdim_, dev_, p_.dtype));
  return std::vector<vkl_out_seg>{ segment (0, qkv_cols_ (), qkv_, type_ (), VKL_ACT_SILU),
                                   segment (qkv_cols_ (), p_.heads * vdim_, gate_, type_ (), VKL_ACT_NONE) };
}

absl::Status
DecayAttention::mix (int S, size_t offset, int run, void *out, size_t os)
{
  const int no = p_.heads * vdim_;
  timer_.start (dev_);
  vkl_recurrence_args a = {};
  a.qscale = 1.f, a.log_decay = (const float *)log_decay_.data ();
  VKLLAMA_STATUS_OK (recur_ (a, qkv_.data (), S, offset, run));
  const int err = vkl_gated_norm ((const float *)o_.data (), (size_t)no, 1, no, p_.heads * p_.vdim,
                                  (const float *)norm_.data (), p_.eps, gate_.data (), (size_t)no, type_ (), S, out, os,
                                  dev_->stream ());
  timer_.stop (dev_);
  return launch_status ("decaying sums", err);
}

void
DecayAttention::describe (vkl_stack_layer &l, int run)
{
  l.mixer = VKL_MIX_DECAY;
  describe_ (l, run);
  l.g0 = qkv_cols_ (), l.qscale = 1.f;
  l.log_decay = (const float *)log_decay_.data (), l.gnorm = (const float *)norm_.data ();
}
}
