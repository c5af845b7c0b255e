#include "models/step_plan.h"
#include "absl/strings/str_format.h"
#include "src/core/gpu_device.h"
#include "vkl_decode.h"
#include "vkl_hip.h"

namespace vkllama
{
absl::Status
StepPlan::hip_status (const char *what, int e)
{
  if (!e)
    return absl::OkStatus ();
  if (e == 1)
    return absl::InvalidArgumentError (absl::StrFormat ("%s: rejected by the HIP layer", what));
  return absl::InternalError (absl::StrFormat ("%s: %s", what, vkl_error_string (e)));
}

absl::Status
StepPlan::create_buffers (GPUDevice *gpu, size_t vocab)
{
  gpu_ = gpu;
  vocab_ = vocab;
  tok_slot_ = Tensor (1, 1, 1, gpu, UINT32, true);
  VKLLAMA_STATUS_OK (tok_slot_.create ());
  logits32_ = Tensor (1, 1, (int)vocab_, gpu, FP32, false);
  return logits32_.create ();
}

absl::Status
StepPlan::step_host_token (uint32_t tok, size_t offset)
{
  // the slot may still be read by a queued step
  VKLLAMA_STATUS_OK (hip_status ("waiting for the stream", vkl_stream_sync (gpu_->stream ())));
  *(uint32_t *)tok_slot_.host () = tok;
  return step_device_token ((const uint32_t *)tok_slot_.data (), offset);
}

absl::Status
StepPlan::adopt_logits (Tensor logits32)
{
  if (logits32.dtype () != FP32 || logits32.size () < vocab_)
    return absl::InvalidArgumentError ("logits tensor has the wrong type");
  adopted_ = logits32;
  adopted_valid_ = true;
  return absl::OkStatus ();
}

const float *
StepPlan::current_logits () const
{
  const Tensor &src = adopted_valid_ ? adopted_ : logits32_;
  return (const float *)src.data () + (src.size () - vocab_);
}

absl::Status
StepPlan::read_logits (float *dst)
{
  VKLLAMA_STATUS_OK (hip_status ("downloading logits", vkl_memcpy_d2h (dst, current_logits (), vocab_ * sizeof (float),
                                                                       gpu_->stream ())));
  VKLLAMA_STATUS_OK (hip_status ("downloading logits", vkl_stream_sync (gpu_->stream ())));
  return check ();
}

absl::Status
StepPlan::argmax_logits (uint32_t *dst)
{
  return hip_status ("argmax", vkl_argmax_f32 (current_logits (), (int)vocab_, dst, gpu_->stream ()));
}

absl::Status
StepPlan::sample_logits (uint32_t *dst, int topk, float topp, uint64_t seed, uint32_t counter)
{
  return hip_status ("sample", vkl_sample_f32 (current_logits (), (int)vocab_, topk, topp, seed, counter, nullptr, dst,
                                               nullptr, nullptr, nullptr, gpu_->stream ()));
}
}
