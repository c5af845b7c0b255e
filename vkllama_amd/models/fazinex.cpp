#include "models/fazinex.h"
#include "absl/strings/str_format.h"
#include "src/ops/latent_attention.h"
#include "src/ops/shared_kv_attention.h"

namespace vkllama
{
// ---------------------------------------------------------------------------
// configuration
// ---------------------------------------------------------------------------
absl::StatusOr<FazinexConfig>
FazinexConfig::parse (const Json &j)
{
  FazinexConfig c;
  VKL_TAKE (c.vocab, j.need_int ("vocab", 1, "model"));
  VKL_TAKE (c.width, j.need_int ("width", 1, "model"));
  double v = 0;
  VKL_TAKE (v, j["norm"].need_number ("eps", "norm"));
  c.eps = (float)v, c.embed_norm = c.tied = true;
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
          VKL_TAKE (l.ff.ff, f.need_int ("ff", 1, where + ".mlp"));
          l.ff.act = VKL_ACT_RELU2;
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
absl::StatusOr<std::unique_ptr<CausalModel> >
Fazinex::create (const Json &config, const WeightSource &weights, const ModelOptions &opt)
{
  auto cfg = FazinexConfig::parse (config);
  VKLLAMA_STATUS_OK (cfg);
  std::unique_ptr<Fazinex> m (new Fazinex ());
  m->layers_ = cfg->layers;
  VKLLAMA_STATUS_OK (m->init_ (*cfg, (int)cfg->layers.size (), weights, opt));
  return std::unique_ptr<CausalModel> (std::move (m));
}

absl::Status
Fazinex::make_block_ (int index, const MixerParams &common, std::unique_ptr<StackBlock> &block)
{
  const FazinexConfig::Layer &l = layers_[(size_t)index];
  MixerParams p = l.mixer;
  p.width = common.width, p.eps = common.eps, p.maxlen = common.maxlen, p.runs = common.runs, p.dtype = common.dtype;
  std::unique_ptr<TokenMixer> mixer;
  if (l.type == FazinexConfig::Layer::Latent)
    mixer.reset (new LatentAttention (gpu_, command (), p));
  else
    mixer.reset (new SharedKVAttention (gpu_, command (), p));
  block.reset (new ParallelBlock (gpu_, command (), absl::StrFormat ("l%d.", index), std::move (mixer), p, l.ff));
  return absl::OkStatus ();
}
}
