// Named tensors of a model, wherever they come from: a safetensors file or
// memory.
#ifndef __VKLLAMA_MODELS_WEIGHTS_H__
#define __VKLLAMA_MODELS_WEIGHTS_H__
#include "absl/status/statusor.h"
#include "src/core/common.h"
#include <map>
#include <memory>
#include <stdint.h>
#include <string>
#include <vector>

namespace vkllama
{
struct WeightView
{
  DType dtype = BF16;
  std::vector<size_t> shape;
  const uint8_t *data = nullptr;
  size_t bytes = 0;
};

class WeightSource
{
public:
  virtual ~WeightSource () {}
  absl::StatusOr<WeightView> find (const std::string &name) const;
  // a bf16 matrix [rows, cols] / vector [n], checked
  absl::StatusOr<const uint16_t *> matrix (const std::string &name, size_t rows, size_t cols) const;
  absl::StatusOr<std::vector<float> > vector (const std::string &name, size_t n) const;
  // a bf16 tensor of one value, whatever its shape
  absl::StatusOr<float> scalar (const std::string &name) const;
  void add (const std::string &name, const WeightView &v) { views_[name] = v; }

protected:
  std::map<std::string, WeightView> views_;
};

// A mapped safetensors file: u64 header length, a JSON object name -> {dtype,
// shape, data_offsets}, then the data.
class SafetensorsFile : public WeightSource
{
public:
  static absl::StatusOr<std::shared_ptr<SafetensorsFile> > open (const std::string &path);
  ~SafetensorsFile () override;

private:
  SafetensorsFile () = default;
  void *map_ = nullptr;
  size_t size_ = 0;
};
}
#endif
