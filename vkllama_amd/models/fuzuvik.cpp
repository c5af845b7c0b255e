#include "models/fuzuvik.h"
#include "absl/strings/str_format.h"
#include "src/ops/chunked_attention.h"
#include "src/ops/recurrent_mixer.h"
#include <cmath>

namespace vkllama
{
namespace
{
// A frequency per pair, base^(-2i/dims); with scaling, long wavelengths (beyond
// original / low) are slowed down by a factor, short ones (below original / high)
// stay, and those between are blended.
absl::StatusOr<std::vector<double> >
rotation (const Json &rot, const std::string &where)
{
  std::vector<double> f;
  if (rot.is_null ())
    return f;
  int dims = 0;
  double base = 0, factor = 1, low = 1, high = 1, original = 0;
  VKL_TAKE (dims, rot.need_int ("dims", 0, where));
  VKL_TAKE (base, rot.need_number ("base", where));
  if (dims % 2 || base <= 0)
    return absl::InvalidArgumentError ("configuration: " + where + ": dims must be even and base positive");
  const Json &sc = rot["scaling"];
  if (!sc.is_null ())
    {
      const std::string sw = where + ".scaling";
      VKL_TAKE (factor, sc.need_number ("factor", sw));
      VKL_TAKE (low, sc.need_number ("low", sw));
      VKL_TAKE (high, sc.need_number ("high", sw));
      VKL_TAKE (original, sc.need_number ("original", sw));
      if (factor <= 0 || low <= 0 || high < low || original <= 0)
        return absl::InvalidArgumentError ("configuration: " + sw + ": values must be positive, high not below low");
    }
  for (int i = 0; i < dims / 2; ++i)
    {
      double x = std::pow (base, -2.0 * i / dims);
      if (!sc.is_null ())
        {
          const double length = 2 * M_PI / x;
          if (length > original / low)
            x /= factor;
          else if (length >= original / high)
            {
              const double s = high > low ? (original / length - low) / (high - low) : 1.0;
              x = (1 - s) * x / factor + s * x;
            }
        }
      f.push_back (x);
    }
  return f;
}

absl::StatusOr<bool>
flag (const Json &j, const std::string &name, const std::string &where)
{
  const Json &v = j[name];
  if (!v.is_null () && v.kind () != Json::Bool)
    return absl::InvalidArgumentError ("configuration: " + where + "." + name + " must be true or false");
  return !v.is_null () && v.number () != 0;
}
}

absl::StatusOr<FuzuvikConfig>
FuzuvikConfig::parse (const Json &j)
{
  FuzuvikConfig c;
  double v = 0;
  VKL_TAKE (c.vocab, j.need_int ("vocab", 1, "model"));
  VKL_TAKE (c.width, j.need_int ("width", 1, "model"));
  VKL_TAKE (v, j["norm"].need_number ("eps", "norm"));
  c.eps = (float)v;
  if (!j["embedding"].is_null ())
    {
      VKL_TAKE (v, j["embedding"].need_number ("scale", "embedding"));
      c.embed_scale = (float)v;
    }
  if (j["layers"].items ().empty ())
    return absl::InvalidArgumentError ("configuration: layers must be a list of layers");
  for (size_t i = 0; i < j["layers"].items ().size (); ++i)
    {
      const Json &e = j["layers"].items ()[i], &m = e["mixer"];
      const std::string where = absl::StrFormat ("layers[%zu]", i), mw = where + ".mixer";
      Layer l;
      MixerParams &p = l.mixer;
      std::string type;
      VKL_TAKE (type, e.need_string ("type", where));
      VKL_TAKE (p.heads, m.need_int ("heads", 1, mw));
      VKL_TAKE (p.dim, m.need_int ("dim", 1, mw));
      VKL_TAKE (p.vdim, m.need_int ("vdim", 1, mw));
      p.kv_heads = p.heads;
      if (type == "attention" || type == "channel_delta")
        {
          VKL_TAKE (p.kv_heads, m.need_int ("kv_heads", 1, mw));
          if (p.heads % p.kv_heads)
            return absl::InvalidArgumentError ("configuration: " + mw + ".heads must be a multiple of kv_heads");
        }
      if (type == "attention")
        {
          l.type = Layer::Attention;
          VKL_TAKE (v, m.need_number ("scale", mw));
          p.scale = (float)v, p.sink = true;
          VKL_TAKE (p.freq, rotation (m["rot"], mw + ".rot"));
          if (2 * p.freq.size () > (size_t)p.dim)
            return absl::InvalidArgumentError ("configuration: " + mw + ".rot: dims exceed the head size dim");
          if (!m["mask"].is_null ())
            VKL_TAKE (p.chunk, m["mask"].need_int ("size", 1, mw + ".mask"));
          VKL_TAKE (p.v_mix, flag (m, "v_mix", mw));
        }
      else if (type == "channel_delta")
        {
          l.type = Layer::Delta;
          VKL_TAKE (p.taps, m.need_int ("conv", 1, mw));
        }
      else if (type == "lightning")
        {
          l.type = Layer::Decay;
          for (const Json &d : m["decay"].items ())
            {
              if (d.kind () != Json::Number || d.number () < 0 || d.number () > 1)
                return absl::InvalidArgumentError ("configuration: " + mw + ".decay: factors from 0 to 1 are needed");
              p.decay.push_back (d.number ());
            }
          if (p.decay.size () != (size_t)p.heads)
            return absl::InvalidArgumentError ("configuration: " + mw + ".decay: one factor per head is needed");
        }
      else
        return absl::InvalidArgumentError ("configuration: " + where + ": unknown mixer type " + type);
      const Json &f = e["mlp"];
      if (!f.is_null ())
        {
          std::string kind;
          VKL_TAKE (kind, f.need_string ("kind", where + ".mlp"));
          if (kind != "dense")
            return absl::InvalidArgumentError ("configuration: " + where + ": unknown feed-forward kind " + kind);
          VKL_TAKE (l.ff.ff, f.need_int ("ff", 1, where + ".mlp"));
          l.ff.act = VKL_ACT_GELU;
        }
      c.layers.push_back (l);
      c.order.push_back ((int)i);
    }
  return c;
}

absl::StatusOr<std::unique_ptr<CausalModel> >
Fuzuvik::create (const Json &config, const WeightSource &weights, const ModelOptions &opt)
{
  auto cfg = FuzuvikConfig::parse (config);
  VKLLAMA_STATUS_OK (cfg);
  std::unique_ptr<Fuzuvik> m (new Fuzuvik ());
  m->layers_ = cfg->layers;
  m->weights_ = &weights;
  VKLLAMA_STATUS_OK (m->init_ (*cfg, (int)cfg->layers.size (), weights, opt));
  m->weights_ = nullptr;
  return std::unique_ptr<CausalModel> (std::move (m));
}

absl::Status
Fuzuvik::make_block_ (int index, const MixerParams &common, std::unique_ptr<StackBlock> &block)
{
  const FuzuvikConfig::Layer &l = layers_[(size_t)index];
  const std::string name = absl::StrFormat ("l%d.", index);
  MixerParams p = l.mixer;
  p.width = common.width, p.eps = common.eps, p.maxlen = common.maxlen, p.runs = common.runs, p.dtype = common.dtype;
  std::unique_ptr<TokenMixer> mixer;
  if (l.type == FuzuvikConfig::Layer::Attention)
    {
      auto *a = new ChunkedAttention (gpu_, command (), p, p.v_mix ? first_mixed_ : nullptr);
      mixer.reset (a);
      if (p.v_mix && !first_mixed_)
        first_mixed_ = a;
    }
  else if (l.type == FuzuvikConfig::Layer::Delta)
    {
      auto *d = new ChannelDelta (gpu_, command (), p);
      mixer.reset (d);
      VKLLAMA_STATUS_OK (d->read_ranks (*weights_, name + "mix."));
    }
  else
    mixer.reset (new DecayAttention (gpu_, command (), p));
  block.reset (new SequentialBlock (gpu_, command (), name, std::move (mixer), p, l.ff));
  return absl::OkStatus ();
}
}
