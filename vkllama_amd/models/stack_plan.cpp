#include "models/stack_plan.h"
#include "absl/strings/str_format.h"
#include "src/core/gpu_device.h"
#include "vkl_hip.h"

namespace vkllama
{
StackPlan::~StackPlan ()
{
  if (usable_)
    vkl_stack_release (&desc_);
}

absl::Status
StackPlan::build (GPUDevice *gpu, const vkl_stack_model &desc, std::vector<vkl_stack_layer> layers)
{
  VKLLAMA_STATUS_OK (create_buffers (gpu, (size_t)desc.vocab));
  desc_ = desc;
  layers_ = std::move (layers);
  desc_.layers_h = layers_.data (), desc_.n_runs = (int)layers_.size ();
  const size_t bytes = vkl_stack_scratch_bytes (&desc_);
  scratch_ = Tensor (1, 1, (int)bytes, gpu, INT8, false);
  VKLLAMA_STATUS_OK (scratch_.create ());
  VKLLAMA_STATUS_OK (hip_status ("clearing step scratch", vkl_memset (scratch_.data (), 0, bytes, gpu->stream ())));
  desc_.scratch = scratch_.data ();
  usable_ = vkl_stack_supported (&desc_) != 0; // (else the operator chain serves single tokens too)
  return absl::OkStatus ();
}

absl::Status
StackPlan::step_device_token (const uint32_t *tok, size_t offset, uint32_t *next_tok)
{
  if (!usable_)
    return absl::FailedPreconditionError ("the one-token step does not cover this model");
  adopted_valid_ = false;
  return hip_status ("decode step", vkl_stack_step (&desc_, tok, (uint32_t)offset, (float *)logits32_.data (),
                                                    next_tok, gpu_->stream ()));
}

absl::Status
StackPlan::loop (uint32_t *ids, size_t pos0, size_t n_steps)
{
  if (!usable_)
    return absl::FailedPreconditionError ("the one-token step does not cover this model");
  adopted_valid_ = false;
  return hip_status ("decode loop", vkl_stack_loop (&desc_, ids, (uint32_t)pos0, (int)n_steps,
                                                    (float *)logits32_.data (), gpu_->stream ()));
}

absl::Status
StackPlan::loop_sampled (uint32_t *ids, size_t pos0, size_t n_steps, int topk, float topp, uint64_t seed)
{
  if (!usable_)
    return absl::FailedPreconditionError ("the one-token step does not cover this model");
  adopted_valid_ = false;
  return hip_status ("sampled decode loop",
                     vkl_stack_loop_sampled (&desc_, ids, (uint32_t)pos0, (int)n_steps, (float *)logits32_.data (),
                                             topk, topp, seed, gpu_->stream ()));
}
}
