// DecodePlan: the device-pointer view of a loaded Llama-2 model that the fused
// one-token decode step (include/vkl_decode.h) consumes.
#ifndef __VKLLAMA_MODELS_DECODE_PLAN_H__
#define __VKLLAMA_MODELS_DECODE_PLAN_H__
#include "absl/status/status.h"
#include "models/step_plan.h"
#include "src/core/tensor.h"
#include "vkl_decode.h"
#include <vector>

namespace vkllama
{
class GPUDevice;
class InputLayer;
class OutputLayer;
class Llama2Block;
class Model;

struct DecodePlan : public StepPlan
{
  DecodePlan ();
  ~DecodePlan () override;
  absl::Status build (Model &model, GPUDevice *gpu, InputLayer *in,
                      std::vector<Llama2Block *> &blocks, OutputLayer *out,
                      float eps);
  // true when the fused kernels cover this model (Q8_0, head width 64/128)
  bool usable () const override { return usable_; }
  void set_mode (int mode) override { mode_ = mode; }
  bool set_option (const char *name, int value) override;
  const vkl_decode_model &desc () const { return desc_; }
  absl::Status step_device_token (const uint32_t *tok, size_t offset,
                                  uint32_t *next_tok = nullptr) override;
  absl::Status loop (uint32_t *ids, size_t pos0, size_t n_steps) override;
  absl::Status loop_sampled (uint32_t *ids, size_t pos0, size_t n_steps, int topk,
                             float topp, uint64_t seed) override;
  int mode () const { return mode_; }
  // Did a wait between workgroups inside a launch give up
  // (vkl_decode_status)?  If so the plan switches to the launches that wait for
  // nothing (mode 0, attention and Wo apart) and the status is Unavailable.
  absl::Status check () override;

private:
  bool usable_;
  int mode_;
  vkl_decode_model desc_;
  Tensor layers_;   // device array of vkl_layer_weights
  std::vector<vkl_layer_weights> layers_h_; // host mirror
  Tensor scratch_;
};
}
#endif
