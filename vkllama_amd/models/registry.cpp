#include "models/registry.h"
#include "models/fazinex.h"
#include "models/fuzuvik.h"
#include "models/llama2.h"
#include <fstream>
#include <sstream>
#include <sys/stat.h>

namespace vkllama
{
namespace
{
struct Entry
{
  const char *name;
  ModelFactory factory;
};
const Entry kEntries[] = { { "Fazinex", Fazinex::create }, { "Fuzuvik", Fuzuvik::create } };

absl::StatusOr<std::unique_ptr<CausalModel> >
load_gguf (const std::string &path, const ModelOptions &opt)
{
  if (opt.dtype == FP32)
    return absl::UnimplementedError ("models from GGUF files run with fp16 activations only");
  gguf_ctx *g = gguf_open (path.c_str ());
  if (!g)
    return absl::NotFoundError ("not a readable GGUF file: " + path);
  std::map<std::string, gguf_key> kv;
  std::map<std::string, gguf_tensor> ts;
  gguf_key key;
  while (gguf_get_key (g, &key))
    kv[std::string (key.name, key.namelen)] = key;
  gguf_tensor t;
  while (gguf_get_tensor (g, &t))
    ts[std::string (t.name, t.namelen)] = t;
  auto m = std::make_unique<Model> (opt.device);
  const absl::Status s = m->init (kv, ts);
  gguf_close (g); // every weight has been copied to the device by now
  VKLLAMA_STATUS_OK (s);
  return std::unique_ptr<CausalModel> (std::move (m));
}
}

ModelFactory
find_architecture (const std::string &name)
{
  for (const Entry &e : kEntries)
    if (name == e.name)
      return e.factory;
  return nullptr;
}

std::vector<std::string>
architectures ()
{
  std::vector<std::string> v;
  for (const Entry &e : kEntries)
    v.push_back (e.name);
  return v;
}

absl::StatusOr<std::unique_ptr<CausalModel> >
create_model (const std::string &config, const WeightSource &w, const ModelOptions &opt)
{
  auto json = Json::parse (config.data (), config.size ());
  VKLLAMA_STATUS_OK (json);
  auto arch = json->need_string ("architecture", "model");
  VKLLAMA_STATUS_OK (arch);
  const ModelFactory f = find_architecture (*arch);
  if (!f)
    return absl::UnimplementedError ("no model class for architecture " + *arch);
  return f (*json, w, opt);
}

absl::StatusOr<std::unique_ptr<CausalModel> >
load_model (const std::string &path, const ModelOptions &opt)
{
  struct stat st;
  if (stat (path.c_str (), &st) != 0)
    return absl::NotFoundError ("neither a GGUF file nor a model folder: " + path);
  if (!S_ISDIR (st.st_mode))
    return load_gguf (path, opt);
  std::ifstream in (path + "/config.json", std::ios::binary);
  std::stringstream text;
  text << in.rdbuf ();
  if (!in)
    return absl::NotFoundError ("cannot read " + path + "/config.json");
  auto file = SafetensorsFile::open (path + "/model.safetensors");
  VKLLAMA_STATUS_OK (file);
  return create_model (text.str (), **file, opt);
}
}
