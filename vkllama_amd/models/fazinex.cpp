#include "models/fazinex.h"
#include "absl/strings/str_format.h"
#include "src/ops/latent_attention.h"
#include "src/ops/shared_kv_attention.h"
#include "vkl_hip.h"
#include <algorithm>
#include <string.h>

namespace vkllama
{
namespace
{
// tokens of a prompt that go through the layers together; a longer prompt runs in
// portions of this size, which bounds the activation buffers
constexpr int kPortion = 4096;

absl::Status
launched (const char *what, int e)
{
  if (!e)
    return absl::OkStatus ();
  if (e == 1) // hipErrorInvalidValue: rejected before any launch
    return absl::InvalidArgumentError (absl::StrFormat ("%s: shapes rejected by the HIP layer", what));
  return absl::InternalError (absl::StrFormat ("%s: %s", what, vkl_error_string (e)));
}

// a buffer of at least `rows` rows, zeroed when it is made
absl::Status
reserve (Tensor &t, int rows, int width, GPUDevice *dev, DType dtype)
{
  if ((int)t.height () >= rows && (int)t.width () == width && t.dtype () == dtype)
    return absl::OkStatus ();
  t = Tensor (1, rows, width, dev, dtype);
  VKLLAMA_STATUS_OK (t.create ());
  return launched ("clearing a buffer", vkl_memset (t.data (), 0, t.bytes (), dev->stream ()));
}
}

// ---------------------------------------------------------------------------
// configuration
// ---------------------------------------------------------------------------
#define VKL_TAKE(dst, expr)                                                   \
  do                                                                          \
    {                                                                         \
      auto v__ = (expr);                                                      \
      if (!v__.ok ())                                                         \
        return v__.status ();                                                 \
      dst = *v__;                                                             \
    }                                                                         \
  while (0)

absl::StatusOr<FazinexConfig>
FazinexConfig::parse (const Json &j)
{
  FazinexConfig c;
  VKL_TAKE (c.vocab, j.need_int ("vocab", 1, "model"));
  VKL_TAKE (c.width, j.need_int ("width", 1, "model"));
  double v = 0;
  VKL_TAKE (v, j["norm"].need_number ("eps", "norm"));
  c.eps = (float)v;
  if (!j["logit_softcap"].is_null ())
    {
      VKL_TAKE (v, j.need_number ("logit_softcap", "model"));
      if (v <= 0)
        return absl::InvalidArgumentError ("configuration: logit_softcap must be positive");
      c.logit_softcap = (float)v;
    }
  if (j["layers"].items ().empty ())
    return absl::InvalidArgumentError ("configuration: layers must be a list of layers");
  for (size_t i = 0; i < j["layers"].items ().size (); ++i)
    {
      const Json &e = j["layers"].items ()[i], &m = e["mixer"];
      const std::string where = absl::StrFormat ("layers[%zu]", i), mw = where + ".mixer";
      Layer l;
      std::string type;
      VKL_TAKE (type, e.need_string ("type", where));
      VKL_TAKE (l.mixer.heads, m.need_int ("heads", 1, mw));
      VKL_TAKE (l.mixer.dim, m.need_int ("dim", 1, mw));
      VKL_TAKE (l.mixer.vdim, m.need_int ("vdim", 1, mw));
      VKL_TAKE (v, m.need_number ("scale", mw));
      l.mixer.scale = (float)v;
      if (type == "latent_attention")
        {
          l.type = Layer::Latent;
          VKL_TAKE (l.mixer.kv_rank, m.need_int ("kv_rank", 1, mw));
        }
      else if (type == "attention")
        {
          l.type = Layer::SharedKV;
          VKL_TAKE (l.mixer.kv_heads, m.need_int ("kv_heads", 1, mw));
          if (l.mixer.heads % l.mixer.kv_heads)
            return absl::InvalidArgumentError ("configuration: " + mw + ".heads must be a multiple of kv_heads");
          if (!m["q_temp"].is_null ())
            {
              VKL_TAKE (v, m["q_temp"].need_number ("coef", mw + ".q_temp"));
              l.mixer.temp_coef = (float)v;
              VKL_TAKE (l.mixer.temp_every, m["q_temp"].need_int ("every", 1, mw + ".q_temp"));
            }
        }
      else
        return absl::InvalidArgumentError ("configuration: " + where + ": unknown mixer " + type);
      const Json &f = e["mlp"];
      if (!f.is_null ())
        {
          std::string kind;
          VKL_TAKE (kind, f.need_string ("kind", where + ".mlp"));
          if (kind != "dense")
            return absl::InvalidArgumentError ("configuration: " + where + ": unknown feed-forward kind " + kind);
          VKL_TAKE (l.ff, f.need_int ("ff", 1, where + ".mlp"));
        }
      c.layers.push_back (l);
    }
  const int n = (int)c.layers.size ();
  int start = 0, stop = 0, times = 1;
  if (!j["loop"].is_null ())
    {
      VKL_TAKE (start, j["loop"].need_int ("start", 0, "loop"));
      VKL_TAKE (stop, j["loop"].need_int ("stop", 0, "loop"));
      VKL_TAKE (times, j["loop"].need_int ("times", 1, "loop"));
      if (start > stop || stop > n)
        return absl::InvalidArgumentError ("configuration: loop must lie within the layers");
    }
  for (int i = 0; i < start; ++i)
    c.order.push_back (i);
  for (int t = 0; t < times; ++t)
    for (int i = start; i < stop; ++i)
      c.order.push_back (i);
  for (int i = stop; i < n; ++i)
    c.order.push_back (i);
  return c;
}
#undef VKL_TAKE

// ---------------------------------------------------------------------------
// a layer
// ---------------------------------------------------------------------------
ParallelBlock::ParallelBlock (GPUDevice *dev, Command *command, const FazinexConfig &cfg, int index, int runs,
                              const ModelOptions &opt)
    : dev_ (dev), command_ (command), prefix_ (absl::StrFormat ("l%d.", index)), width_ (cfg.width),
      width_p_ (round_up (cfg.width, 64)), ff_ (cfg.layers[(size_t)index].ff), eps_ (cfg.eps), dtype_ (opt.dtype)
{
  RowMixerParams p = cfg.layers[(size_t)index].mixer;
  p.width = cfg.width, p.eps = cfg.eps, p.maxlen = (int)opt.max_tokens, p.runs = runs, p.dtype = opt.dtype;
  if (cfg.layers[(size_t)index].type == FazinexConfig::Layer::Latent)
    mixer_.reset (new LatentAttention (dev, command, p));
  else
    mixer_.reset (new SharedKVAttention (dev, command, p));
  up_row_ = mixer_->in_rows ();
  n_in_ = up_row_ + round_up (ff_, 8);
  ff_col_ = mixer_->out_cols ();
  k_out_ = round_up (ff_col_ + ff_, 64);
}

absl::Status
ParallelBlock::load (const WeightSource &w)
{
  VKLLAMA_STATUS_OK (mixer_->init ());
  VKLLAMA_STATUS_OK (mixer_->load (w, prefix_ + "mix."));
  auto norm = w.vector (prefix_ + "norm1", (size_t)width_);
  VKLLAMA_STATUS_OK (norm);
  auto dn = upload_vector (dev_, command_, *norm, width_p_);
  VKLLAMA_STATUS_OK (dn);
  norm_ = *dn;
  PackedMatrix in (n_in_, width_p_), out (width_, k_out_);
  VKLLAMA_STATUS_OK (mixer_->pack_in (w, prefix_ + "mix.", in));
  VKLLAMA_STATUS_OK (mixer_->pack_out (w, prefix_ + "mix.", out));
  if (ff_)
    {
      auto up = w.matrix (prefix_ + "mlp.up", (size_t)ff_, (size_t)width_);
      VKLLAMA_STATUS_OK (up);
      auto down = w.matrix (prefix_ + "mlp.down", (size_t)width_, (size_t)ff_);
      VKLLAMA_STATUS_OK (down);
      in.put (*up, ff_, width_, up_row_);
      out.put (*down, width_, ff_, 0, ff_col_);
    }
  auto di = in.upload (dev_, command_);
  VKLLAMA_STATUS_OK (di);
  auto dout = out.upload (dev_, command_);
  VKLLAMA_STATUS_OK (dout);
  w_in_ = *di, w_out_ = *dout;
  weight_bytes_ = w_in_.bytes () + w_out_.bytes () + norm_.bytes ();
  return absl::OkStatus ();
}

absl::Status
ParallelBlock::operator() (Tensor &x, int S, size_t offset, int run, Buffers &b)
{
  const int type = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  const size_t esize = dtype_ == FP32 ? 4 : 2, cs = (size_t)b.cat_stride;
  void *s = dev_->stream ();
  float *xp = (float *)x.data ();
  VKLLAMA_STATUS_OK (launched ("layer norm", vkl_rmsnorm_f32 (xp, (size_t)width_p_, nullptr, S, width_,
                                                              (const float *)norm_.data (), eps_, b.h.data (), type,
                                                              (size_t)width_p_, width_p_, s)));
  auto segs = mixer_->segments (S, offset, run);
  VKLLAMA_STATUS_OK (segs);
  if (ff_)
    segs->push_back ({ up_row_, ff_, (uint8_t *)b.cat.data () + (size_t)ff_col_ * esize, cs, type, 2, nullptr, 0.f });
  VKLLAMA_STATUS_OK (launched ("layer input product",
                               vkl_project_bf16w (b.h.data (), type, (size_t)width_p_, w_in_.data (), S, n_in_,
                                                  width_p_, segs->data (), (int)segs->size (), s)));
  VKLLAMA_STATUS_OK (mixer_->mix (S, offset, run, b.cat.data (), cs));
  const vkl_out_seg back = { 0, width_, xp, (size_t)width_p_, VKL_TYPE_F32, 0, xp, 0.f };
  return launched ("layer output product", vkl_project_bf16w (b.cat.data (), type, cs, w_out_.data (), S, width_,
                                                              k_out_, &back, 1, s));
}

void
ParallelBlock::describe (vkl_stack_layer &l, int run)
{
  mixer_->describe (l, run);
  l.ff = ff_;
  l.norm = (const float *)norm_.data ();
  l.w_in = w_in_.data (), l.n_in = n_in_, l.up0 = up_row_;
  l.w_out = w_out_.data (), l.k_out = k_out_, l.ff_col = ff_col_;
}

// ---------------------------------------------------------------------------
// the model
// ---------------------------------------------------------------------------
Fazinex::~Fazinex ()
{
  if (gpu_ && gpu_->stream ())
    vkl_stream_sync (gpu_->stream ());
  plan_.reset ();
  blocks_.clear ();
  buf_ = ParallelBlock::Buffers ();
  embed_ = embed_norm_ = final_norm_ = x_ = toks_ = rows_ = out_h_ = Tensor ();
  release_buffers_ ();
  command_.reset ();
  delete gpu_;
}

absl::StatusOr<std::unique_ptr<CausalModel> >
Fazinex::create (const Json &config, const WeightSource &weights, const ModelOptions &opt)
{
  std::unique_ptr<Fazinex> m (new Fazinex ());
  VKLLAMA_STATUS_OK (m->init_ (config, weights, opt));
  return std::unique_ptr<CausalModel> (std::move (m));
}

absl::Status
Fazinex::init_ (const Json &config, const WeightSource &w, const ModelOptions &options)
{
  auto cfg = FazinexConfig::parse (config);
  VKLLAMA_STATUS_OK (cfg);
  cfg_ = *cfg;
  ModelOptions opt = options;
  if (opt.max_tokens == 0)
    opt.max_tokens = 4096;
  if (opt.max_tokens > (size_t)1 << 24)
    return absl::InvalidArgumentError ("at most 2^24 cached tokens are supported");
  dtype_ = opt.dtype;
  if (dtype_ != BF16 && dtype_ != FP32)
    return absl::InvalidArgumentError ("this model runs in bf16 or fp32");
  vocab_ = (size_t)cfg_.vocab, maxlen_ = opt.max_tokens;
  width_p_ = round_up (cfg_.width, 64);
  gpu_ = new GPUDevice (opt.device);
  VKLLAMA_STATUS_OK (gpu_->init ());
  command_.reset (new Command (gpu_));
  VKLLAMA_STATUS_OK (command_->init ());

  auto table = w.matrix ("embed", vocab_, (size_t)cfg_.width);
  VKLLAMA_STATUS_OK (table);
  PackedMatrix pm (cfg_.vocab, width_p_);
  pm.put (*table, cfg_.vocab, cfg_.width, 0);
  auto de = pm.upload (gpu_, command_.get ());
  VKLLAMA_STATUS_OK (de);
  embed_ = *de;
  for (int i = 0; i < 2; ++i)
    {
      auto v = w.vector (i ? "final.norm" : "embed.norm", (size_t)cfg_.width);
      VKLLAMA_STATUS_OK (v);
      auto d = upload_vector (gpu_, command_.get (), *v, width_p_);
      VKLLAMA_STATUS_OK (d);
      (i ? final_norm_ : embed_norm_) = *d;
    }
  for (int i = 0; i < (int)cfg_.layers.size (); ++i)
    {
      const int runs = (int)std::count (cfg_.order.begin (), cfg_.order.end (), i);
      blocks_.emplace_back (new ParallelBlock (gpu_, command_.get (), cfg_, i, std::max (runs, 1), opt));
      VKLLAMA_STATUS_OK (blocks_.back ()->load (w));
      buf_.cat_stride = std::max (buf_.cat_stride, blocks_.back ()->out_width ());
    }

  vkl_stack_model d = {};
  d.width = cfg_.width, d.width_p = width_p_, d.vocab = cfg_.vocab, d.maxlen = (int)maxlen_;
  d.ctype = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  d.eps = cfg_.eps, d.logit_cap = cfg_.logit_softcap;
  d.embed = embed_.data ();
  d.embed_norm = (const float *)embed_norm_.data (), d.final_norm = (const float *)final_norm_.data ();
  std::vector<vkl_stack_layer> layers;
  std::vector<int> seen (blocks_.size (), 0);
  for (int i : cfg_.order)
    {
      vkl_stack_layer l = {};
      blocks_[(size_t)i]->describe (l, seen[(size_t)i]++);
      layers.push_back (l);
    }
  auto plan = std::make_unique<StackPlan> ();
  VKLLAMA_STATUS_OK (plan->build (gpu_, d, layers));
  plan_ = std::move (plan);
  return command_->wait ();
}

absl::Status
Fazinex::wait_all_ ()
{
  return command_->wait ();
}

// S tokens through every layer; leaves the residual stream in x_
absl::Status
Fazinex::pass_ (const uint32_t *toks, int S, size_t offset, std::vector<float> *streams)
{
  void *s = gpu_->stream ();
  VKLLAMA_STATUS_OK (reserve (x_, S, width_p_, gpu_, FP32));
  VKLLAMA_STATUS_OK (reserve (buf_.h, S, width_p_, gpu_, dtype_));
  VKLLAMA_STATUS_OK (reserve (buf_.cat, S, buf_.cat_stride, gpu_, dtype_));
  VKLLAMA_STATUS_OK (reserve (toks_, 1, S, gpu_, UINT32));
  VKLLAMA_STATUS_OK (command_->upload (toks, (size_t)S, toks_));
  VKLLAMA_STATUS_OK (launched ("embedding", vkl_embed_norm_bf16 (embed_.data (), (uint32_t)vocab_, width_p_,
                                                                 cfg_.width, (const uint32_t *)toks_.data (),
                                                                 (uint32_t)S, (const float *)embed_norm_.data (),
                                                                 cfg_.eps, (float *)x_.data (), (size_t)width_p_, s)));
  std::vector<int> seen (blocks_.size (), 0);
  for (int i : cfg_.order)
    {
      VKLLAMA_STATUS_OK ((*blocks_[(size_t)i]) (x_, S, offset, seen[(size_t)i]++, buf_));
      if (streams)
        {
          std::vector<float> rows ((size_t)S * width_p_);
          VKLLAMA_STATUS_OK (launched ("download", vkl_memcpy_d2h (rows.data (), x_.data (), rows.size () * 4, s)));
          VKLLAMA_STATUS_OK (launched ("download", vkl_stream_sync (s)));
          for (int r = 0; r < S; ++r)
            streams->insert (streams->end (), rows.begin () + (size_t)r * width_p_,
                             rows.begin () + (size_t)r * width_p_ + cfg_.width);
        }
    }
  return absl::OkStatus ();
}

// logits of those rows of x_ -> out [rows, vocab] (device)
absl::Status
Fazinex::logits_ (const std::vector<uint32_t> &rows, float *out)
{
  const int type = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16, n = (int)rows.size ();
  void *s = gpu_->stream ();
  VKLLAMA_STATUS_OK (reserve (rows_, 1, n, gpu_, UINT32));
  VKLLAMA_STATUS_OK (reserve (out_h_, n, width_p_, gpu_, dtype_));
  VKLLAMA_STATUS_OK (command_->upload (rows.data (), rows.size (), rows_));
  VKLLAMA_STATUS_OK (launched ("final norm",
                               vkl_rmsnorm_f32 ((const float *)x_.data (), (size_t)width_p_,
                                                (const uint32_t *)rows_.data (), n, cfg_.width,
                                                (const float *)final_norm_.data (), cfg_.eps, out_h_.data (), type,
                                                (size_t)width_p_, width_p_, s)));
  const vkl_out_seg seg = { 0, cfg_.vocab, out, vocab_, VKL_TYPE_F32, 0, nullptr, cfg_.logit_softcap };
  return launched ("output product", vkl_project_bf16w (out_h_.data (), type, (size_t)width_p_, embed_.data (), n,
                                                        cfg_.vocab, width_p_, &seg, 1, s));
}

absl::StatusOr<Tensor>
Fazinex::forward_ (std::vector<uint32_t> const &toks, const size_t offset, std::vector<uint32_t> const &rows)
{
  VKLLAMA_STATUS_OK (check_span_ (toks.size (), offset));
  Tensor out (1, (int)std::max<size_t> (rows.size (), 1), (int)vocab_, gpu_, FP32);
  VKLLAMA_STATUS_OK (out.create ());
  for (size_t at = 0; at < toks.size (); at += kPortion)
    {
      const int S = (int)std::min<size_t> (kPortion, toks.size () - at);
      VKLLAMA_STATUS_OK (pass_ (toks.data () + at, S, offset + at, nullptr));
      // runs of wanted rows that fall into this portion (in the order asked for)
      for (size_t i = 0; i < rows.size ();)
        {
          std::vector<uint32_t> here;
          const size_t first = i;
          while (i < rows.size () && rows[i] >= at && rows[i] < at + (size_t)S)
            here.push_back (rows[i++] - (uint32_t)at);
          if (here.empty ())
            {
              ++i;
              continue;
            }
          VKLLAMA_STATUS_OK (logits_ (here, (float *)out.data () + first * vocab_));
        }
    }
  return out;
}

absl::StatusOr<std::vector<float> >
Fazinex::residual_streams (std::vector<uint32_t> const &toks, size_t offset)
{
  VKLLAMA_STATUS_OK (check_span_ (toks.size (), offset));
  if (toks.size () > (size_t)kPortion)
    return absl::InvalidArgumentError ("residual streams: one portion at most");
  std::vector<float> out;
  VKLLAMA_STATUS_OK (pass_ (toks.data (), (int)toks.size (), offset, &out));
  return out;
}

size_t
Fazinex::decode_step_bytes (size_t L) const
{
  size_t n = embed_.bytes () + final_norm_.bytes () + (size_t)width_p_ * 2;
  for (int i : cfg_.order)
    n += blocks_[(size_t)i]->weight_bytes () + blocks_[(size_t)i]->mixer ().weight_bytes ()
         + (L + 1) * blocks_[(size_t)i]->mixer ().row_bytes ();
  return n;
}
}
