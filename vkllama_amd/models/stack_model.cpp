#include "models/stack_model.h"
#include "absl/strings/str_format.h"
#include "vkl_hip.h"
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
// layers
// ---------------------------------------------------------------------------
StackBlock::StackBlock (GPUDevice *dev, Command *command, const std::string &name, std::unique_ptr<TokenMixer> mixer,
                        const MixerParams &mp, const FeedForwardParams &ff)
    : dev_ (dev), command_ (command), prefix_ (name), width_ (mp.width), width_p_ (round_up (mp.width, 64)),
      eps_ (mp.eps), dtype_ (mp.dtype), ff_ (ff), mixer_ (std::move (mixer))
{
}

absl::StatusOr<Tensor>
StackBlock::norm_weights_ (const WeightSource &w, const std::string &name)
{
  auto v = w.vector (prefix_ + name, (size_t)width_);
  VKLLAMA_STATUS_OK (v);
  weight_bytes_ += (size_t)width_p_ * 4;
  return upload_vector (dev_, command_, *v, width_p_);
}

absl::Status
StackBlock::norm_input_ (Tensor &x, int S, Tensor &w, Buffers &b)
{
  const int type = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  return launched ("layer norm",
                   vkl_rmsnorm_f32 ((const float *)x.data (), (size_t)width_p_, nullptr, S, width_,
                                    (const float *)w.data (), eps_, b.h.data (), type, (size_t)width_p_, width_p_,
                                    dev_->stream ()));
}

absl::Status
StackBlock::add_product_ (Tensor &x, int S, Tensor &w, int k, Buffers &b)
{
  const int type = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  float *xp = (float *)x.data ();
  const vkl_out_seg back = { 0, width_, xp, (size_t)width_p_, VKL_TYPE_F32, VKL_ACT_NONE, xp, 0.f };
  return launched ("layer output product",
                   vkl_project_bf16w (b.cat.data (), type, (size_t)b.cat_stride, w.data (), S, width_, k, &back, 1,
                                      dev_->stream ()));
}

ParallelBlock::ParallelBlock (GPUDevice *dev, Command *command, const std::string &name,
                              std::unique_ptr<TokenMixer> mixer, const MixerParams &mp, const FeedForwardParams &ff)
    : StackBlock (dev, command, name, std::move (mixer), mp, ff)
{
  up_row_ = mixer_->in_rows ();
  n_in_ = up_row_ + round_up (ff_.ff, 8);
  ff_col_ = mixer_->out_cols ();
  k_out_ = round_up (ff_col_ + ff_.ff, 64);
}

absl::Status
ParallelBlock::load (const WeightSource &w)
{
  VKLLAMA_STATUS_OK (mixer_->init ());
  VKLLAMA_STATUS_OK (mixer_->load (w, prefix_ + "mix."));
  VKL_TAKE (norm_, norm_weights_ (w, "norm1"));
  PackedMatrix in (n_in_, width_p_), out (width_, k_out_);
  VKLLAMA_STATUS_OK (mixer_->pack_in (w, prefix_ + "mix.", in));
  VKLLAMA_STATUS_OK (mixer_->pack_out (w, prefix_ + "mix.", out));
  if (ff_.ff)
    {
      auto up = w.matrix (prefix_ + "mlp.up", (size_t)ff_.ff, (size_t)width_);
      VKLLAMA_STATUS_OK (up);
      auto down = w.matrix (prefix_ + "mlp.down", (size_t)width_, (size_t)ff_.ff);
      VKLLAMA_STATUS_OK (down);
      in.put (*up, ff_.ff, width_, up_row_);
      out.put (*down, width_, ff_.ff, 0, ff_col_);
    }
  VKL_TAKE (w_in_, in.upload (dev_, command_));
  VKL_TAKE (w_out_, out.upload (dev_, command_));
  weight_bytes_ += w_in_.bytes () + w_out_.bytes ();
  return absl::OkStatus ();
}

absl::Status
ParallelBlock::operator() (Tensor &x, int S, size_t offset, int run, Buffers &b)
{
  const int type = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  const size_t esize = dtype_ == FP32 ? 4 : 2, cs = (size_t)b.cat_stride;
  VKLLAMA_STATUS_OK (norm_input_ (x, S, norm_, b));
  auto segs = mixer_->segments (S, offset, run);
  VKLLAMA_STATUS_OK (segs);
  if (ff_.ff)
    segs->push_back ({ up_row_, ff_.ff, (uint8_t *)b.cat.data () + (size_t)ff_col_ * esize, cs, type, ff_.act, nullptr,
                       0.f });
  VKLLAMA_STATUS_OK (launched ("layer input product",
                               vkl_project_bf16w (b.h.data (), type, (size_t)width_p_, w_in_.data (), S, n_in_,
                                                  width_p_, segs->data (), (int)segs->size (), dev_->stream ())));
  VKLLAMA_STATUS_OK (mixer_->mix (S, offset, run, b.cat.data (), cs));
  return add_product_ (x, S, w_out_, k_out_, b);
}

void
ParallelBlock::describe (vkl_stack_layer &l, int run)
{
  mixer_->describe (l, run);
  l.ff = ff_.ff, l.ff_act = ff_.act;
  l.norm = (const float *)norm_.data ();
  l.w_in = w_in_.data (), l.n_in = n_in_, l.up0 = up_row_;
  l.w_out = w_out_.data (), l.k_out = k_out_, l.ff_col = ff_col_;
}

SequentialBlock::SequentialBlock (GPUDevice *dev, Command *command, const std::string &name,
                                  std::unique_ptr<TokenMixer> mixer, const MixerParams &mp,
                                  const FeedForwardParams &ff)
    : StackBlock (dev, command, name, std::move (mixer), mp, ff)
{
  n_in_ = mixer_->in_rows ();
  k_out_ = round_up (mixer_->out_cols (), 64);
  ff_p_ = round_up (ff_.ff, 64);
}

absl::Status
SequentialBlock::load (const WeightSource &w)
{
  VKLLAMA_STATUS_OK (mixer_->init ());
  VKLLAMA_STATUS_OK (mixer_->load (w, prefix_ + "mix."));
  VKL_TAKE (norm1_, norm_weights_ (w, "norm1"));
  PackedMatrix in (n_in_, width_p_), out (width_, k_out_);
  VKLLAMA_STATUS_OK (mixer_->pack_in (w, prefix_ + "mix.", in));
  VKLLAMA_STATUS_OK (mixer_->pack_out (w, prefix_ + "mix.", out));
  VKL_TAKE (w_in_, in.upload (dev_, command_));
  VKL_TAKE (w_out_, out.upload (dev_, command_));
  weight_bytes_ += w_in_.bytes () + w_out_.bytes ();
  if (!ff_.ff)
    return absl::OkStatus ();
  VKL_TAKE (norm2_, norm_weights_ (w, "norm2"));
  auto up = w.matrix (prefix_ + "mlp.up", (size_t)ff_.ff, (size_t)width_);
  VKLLAMA_STATUS_OK (up);
  auto down = w.matrix (prefix_ + "mlp.down", (size_t)width_, (size_t)ff_.ff);
  VKLLAMA_STATUS_OK (down);
  // (up to the padded count: the rows behind put zeros where the product back reads)
  PackedMatrix pu (ff_p_, width_p_), pd (width_, ff_p_);
  pu.put (*up, ff_.ff, width_, 0);
  pd.put (*down, width_, ff_.ff, 0);
  VKL_TAKE (w_up_, pu.upload (dev_, command_));
  VKL_TAKE (w_down_, pd.upload (dev_, command_));
  weight_bytes_ += w_up_.bytes () + w_down_.bytes ();
  return absl::OkStatus ();
}

absl::Status
SequentialBlock::operator() (Tensor &x, int S, size_t offset, int run, Buffers &b)
{
  const int type = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  const size_t cs = (size_t)b.cat_stride;
  VKLLAMA_STATUS_OK (norm_input_ (x, S, norm1_, b));
  auto segs = mixer_->segments (S, offset, run);
  VKLLAMA_STATUS_OK (segs);
  VKLLAMA_STATUS_OK (launched ("mixer input product",
                               vkl_project_bf16w (b.h.data (), type, (size_t)width_p_, w_in_.data (), S, n_in_,
                                                  width_p_, segs->data (), (int)segs->size (), dev_->stream ())));
  VKLLAMA_STATUS_OK (mixer_->mix (S, offset, run, b.cat.data (), cs));
  VKLLAMA_STATUS_OK (add_product_ (x, S, w_out_, k_out_, b));
  if (!ff_.ff)
    return absl::OkStatus ();
  VKLLAMA_STATUS_OK (norm_input_ (x, S, norm2_, b));
  const vkl_out_seg up = { 0, ff_p_, b.cat.data (), cs, type, ff_.act, nullptr, 0.f };
  VKLLAMA_STATUS_OK (launched ("feed-forward product",
                               vkl_project_bf16w (b.h.data (), type, (size_t)width_p_, w_up_.data (), S, ff_p_,
                                                  width_p_, &up, 1, dev_->stream ())));
  return add_product_ (x, S, w_down_, ff_p_, b);
}

void
SequentialBlock::describe (vkl_stack_layer &l, int run)
{
  mixer_->describe (l, run);
  l.ff = ff_.ff, l.ff_act = ff_.act, l.ff_p = ff_p_;
  l.norm = (const float *)norm1_.data ();
  l.w_in = w_in_.data (), l.n_in = n_in_, l.up0 = n_in_;
  l.w_out = w_out_.data (), l.k_out = k_out_, l.ff_col = k_out_;
  if (!ff_.ff)
    return;
  l.norm2 = (const float *)norm2_.data ();
  l.w_up = w_up_.data (), l.w_down = w_down_.data ();
}

// ---------------------------------------------------------------------------
// the model
// ---------------------------------------------------------------------------
StackModel::~StackModel ()
{
  if (gpu_ && gpu_->stream ())
    vkl_stream_sync (gpu_->stream ());
  plan_.reset ();
  blocks_.clear ();
  buf_ = StackBlock::Buffers ();
  embed_ = head_ = embed_norm_ = final_norm_ = x_ = toks_ = rows_ = out_h_ = Tensor ();
  release_buffers_ ();
  command_.reset ();
  delete gpu_;
}

absl::Status
StackModel::init_ (const StackConfig &cfg, int layers, const WeightSource &w, const ModelOptions &options)
{
  cfg_ = cfg;
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

  for (int i = 0; i < (cfg_.tied ? 1 : 2); ++i)
    {
      auto table = w.matrix (i ? "head" : "embed", vocab_, (size_t)cfg_.width);
      VKLLAMA_STATUS_OK (table);
      PackedMatrix pm (cfg_.vocab, width_p_);
      pm.put (*table, cfg_.vocab, cfg_.width, 0);
      VKL_TAKE ((i ? head_ : embed_), pm.upload (gpu_, command_.get ()));
    }
  for (int i = cfg_.embed_norm ? 0 : 1; i < 2; ++i)
    {
      auto v = w.vector (i ? "final.norm" : "embed.norm", (size_t)cfg_.width);
      VKLLAMA_STATUS_OK (v);
      VKL_TAKE ((i ? final_norm_ : embed_norm_), upload_vector (gpu_, command_.get (), *v, width_p_));
    }
  MixerParams common;
  common.width = cfg_.width, common.eps = cfg_.eps, common.maxlen = (int)opt.max_tokens, common.dtype = opt.dtype;
  for (int i = 0; i < layers; ++i)
    {
      common.runs = std::max (1, (int)std::count (cfg_.order.begin (), cfg_.order.end (), i));
      std::unique_ptr<StackBlock> b;
      VKLLAMA_STATUS_OK (make_block_ (i, common, b));
      blocks_.push_back (std::move (b));
      VKLLAMA_STATUS_OK (blocks_.back ()->load (w));
      if (blocks_.back ()->mixer ().state_bytes ())
        stateful_ = true;
      buf_.cat_stride = std::max (buf_.cat_stride, blocks_.back ()->cat_width ());
    }

  vkl_stack_model d = {};
  d.width = cfg_.width, d.width_p = width_p_, d.vocab = cfg_.vocab, d.maxlen = (int)maxlen_;
  d.ctype = dtype_ == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16;
  d.eps = cfg_.eps, d.logit_cap = cfg_.logit_softcap, d.embed_scale = cfg_.embed_scale;
  d.embed = embed_.data (), d.head = cfg_.tied ? nullptr : head_.data ();
  d.embed_norm = cfg_.embed_norm ? (const float *)embed_norm_.data () : nullptr;
  d.final_norm = (const float *)final_norm_.data ();
  std::vector<vkl_stack_layer> table;
  std::vector<int> seen (blocks_.size (), 0);
  for (int i : cfg_.order)
    {
      vkl_stack_layer l = {};
      blocks_[(size_t)i]->describe (l, seen[(size_t)i]++);
      table.push_back (l);
    }
  auto plan = std::make_unique<StackPlan> ();
  VKLLAMA_STATUS_OK (plan->build (gpu_, d, table));
  plan_ = std::move (plan);
  return command_->wait ();
}

absl::Status
StackModel::wait_all_ ()
{
  return command_->wait ();
}

// S tokens through every layer; leaves the residual stream in x_
absl::Status
StackModel::pass_ (const uint32_t *toks, int S, size_t offset, std::vector<float> *streams)
{
  void *s = gpu_->stream ();
  VKLLAMA_STATUS_OK (reserve (x_, S, width_p_, gpu_, FP32));
  VKLLAMA_STATUS_OK (reserve (buf_.h, S, width_p_, gpu_, dtype_));
  VKLLAMA_STATUS_OK (reserve (buf_.cat, S, buf_.cat_stride, gpu_, dtype_));
  VKLLAMA_STATUS_OK (reserve (toks_, 1, S, gpu_, UINT32));
  VKLLAMA_STATUS_OK (command_->upload (toks, (size_t)S, toks_));
  const uint32_t *ids = (const uint32_t *)toks_.data ();
  float *xp = (float *)x_.data ();
  VKLLAMA_STATUS_OK (launched (
      "embedding", cfg_.embed_norm ? vkl_embed_norm_bf16 (embed_.data (), (uint32_t)vocab_, width_p_, cfg_.width, ids,
                                                          (uint32_t)S, (const float *)embed_norm_.data (), cfg_.eps,
                                                          xp, (size_t)width_p_, s)
                                   : vkl_embed_rows_bf16 (embed_.data (), (uint32_t)vocab_, width_p_, cfg_.width, ids,
                                                          (uint32_t)S, cfg_.embed_scale, xp, (size_t)width_p_, s)));
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
StackModel::logits_ (const std::vector<uint32_t> &rows, float *out)
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
  return launched ("output product", vkl_project_bf16w (out_h_.data (), type, (size_t)width_p_,
                                                        (cfg_.tied ? embed_ : head_).data (), n, cfg_.vocab, width_p_,
                                                        &seg, 1, s));
}

absl::StatusOr<Tensor>
StackModel::forward_ (std::vector<uint32_t> const &toks, const size_t offset, std::vector<uint32_t> const &rows)
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
StackModel::residual_streams (std::vector<uint32_t> const &toks, size_t offset)
{
  VKLLAMA_STATUS_OK (check_span_ (toks.size (), offset));
  if (toks.size () > (size_t)kPortion)
    return absl::InvalidArgumentError ("residual streams: one portion at most");
  std::vector<float> out;
  VKLLAMA_STATUS_OK (begin_pass_ (offset));
  VKLLAMA_STATUS_OK (pass_ (toks.data (), (int)toks.size (), offset, &out));
  end_pass_ (offset + toks.size ());
  return out;
}

size_t
StackModel::decode_step_bytes (size_t L) const
{
  size_t n = (cfg_.tied ? embed_ : head_).bytes () + final_norm_.bytes () + (size_t)width_p_ * 2;
  for (int i : cfg_.order)
    {
      TokenMixer &mixer = blocks_[(size_t)i]->mixer ();
      n += blocks_[(size_t)i]->weight_bytes () + mixer.rows_read (L) * mixer.row_bytes () + 2 * mixer.state_bytes ();
    }
  return n;
}
}
