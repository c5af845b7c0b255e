// StackPlan: the one-token step (include/vkl_stack.h) of a decoder stack whose
// layers differ.
#ifndef __VKLLAMA_MODELS_STACK_PLAN_H__
#define __VKLLAMA_MODELS_STACK_PLAN_H__
#include "models/step_plan.h"
#include "vkl_stack.h"
#include <vector>

namespace vkllama
{
class StackPlan : public StepPlan
{
public:
  ~StackPlan () override;
  // desc: everything but layers_h and scratch; one layer entry per run
  absl::Status build (GPUDevice *gpu, const vkl_stack_model &desc, std::vector<vkl_stack_layer> layers);
  bool usable () const override { return usable_; }
  absl::Status step_device_token (const uint32_t *tok, size_t offset, uint32_t *next_tok = nullptr) override;
  absl::Status loop (uint32_t *ids, size_t pos0, size_t n_steps) override;
  absl::Status loop_sampled (uint32_t *ids, size_t pos0, size_t n_steps, int topk, float topp,
                             uint64_t seed) override;

private:
  bool usable_ = false;
  vkl_stack_model desc_ = {};
  std::vector<vkl_stack_layer> layers_;
  Tensor scratch_;
};
}
#endif
