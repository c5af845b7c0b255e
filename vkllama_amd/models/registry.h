// Which class serves which model: GGUF files (architecture "llama") and folders
// with a config.json, whose "architecture" names an entry of the table.
#ifndef __VKLLAMA_MODELS_REGISTRY_H__
#define __VKLLAMA_MODELS_REGISTRY_H__
#include "absl/status/statusor.h"
#include "models/causal_model.h"
#include "models/json.h"
#include "models/weights.h"
#include <memory>
#include <string>
#include <vector>

namespace vkllama
{
struct ModelOptions
{
  int device = 0;
  DType dtype = BF16;    // stored activations and caches: BF16 or FP32; models
                         // with a fixed format refuse FP32
  size_t max_tokens = 0; // cache rows of a model whose file names no context length (0: 4096)
};

typedef absl::StatusOr<std::unique_ptr<CausalModel> > (*ModelFactory) (const Json &config, const WeightSource &w,
                                                                      const ModelOptions &opt);
// null if there is no such architecture
ModelFactory find_architecture (const std::string &name);
std::vector<std::string> architectures ();

// a model from its configuration text and tensors
absl::StatusOr<std::unique_ptr<CausalModel> > create_model (const std::string &config, const WeightSource &w,
                                                            const ModelOptions &opt);
// a model from a path: a GGUF file, or a folder with config.json and
// model.safetensors
absl::StatusOr<std::unique_ptr<CausalModel> > load_model (const std::string &path, const ModelOptions &opt);
}
#endif
