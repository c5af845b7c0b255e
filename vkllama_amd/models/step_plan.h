// StepPlan: the one-token step of a loaded model on the device (its fused
// launches), plus the small state the token loop keeps there: the current
// logits and a slot for a token id that comes from the host.  DecodePlan
// (Llama-2 blocks) and StackPlan (stacks of differing layers) implement it.
#ifndef __VKLLAMA_MODELS_STEP_PLAN_H__
#define __VKLLAMA_MODELS_STEP_PLAN_H__
#include "absl/status/status.h"
#include "src/core/tensor.h"

namespace vkllama
{
class GPUDevice;

class StepPlan
{
public:
  virtual ~StepPlan () {}
  // true when the fused kernels cover this model
  virtual bool usable () const = 0;
  // token id read from device-visible memory; next_tok (optional,
  // device-visible) receives the arg-max id of this step
  virtual absl::Status step_device_token (const uint32_t *tok, size_t offset, uint32_t *next_tok = nullptr) = 0;
  // n_steps greedy tokens replayed from a captured graph; ids is device memory,
  // ids[0] the first input token
  virtual absl::Status loop (uint32_t *ids, size_t pos0, size_t n_steps) = 0;
  // the same with a draw from the top-k / top-p candidates instead of the
  // arg-max at the end of every replayed step
  virtual absl::Status loop_sampled (uint32_t *ids, size_t pos0, size_t n_steps, int topk, float topp,
                                     uint64_t seed)
      = 0;
  // After the stream has been synchronised: Unavailable if the steps since the
  // last call are invalid and the caller has to repeat them.
  virtual absl::Status check () { return absl::OkStatus (); }
  // options of this model's steps; false for an unknown name or a bad value
  virtual bool set_option (const char *, int) { return false; }
  virtual void set_mode (int) {}

  // token id given by the host
  absl::Status step_host_token (uint32_t tok, size_t offset);
  // copies the fp32 logits of the last step (fused or adopted) to the host
  absl::Status read_logits (float *dst);
  // remember the fp32 logits tensor of an operator-chain pass
  absl::Status adopt_logits (Tensor logits32);
  // arg-max of the current logits into device-visible memory
  absl::Status argmax_logits (uint32_t *dst);
  // a token drawn from the current logits on the device (vkl_sample_f32):
  // topp < 0 keeps the topk largest logits, else the top-p set
  absl::Status sample_logits (uint32_t *dst, int topk, float topp, uint64_t seed, uint32_t counter);

protected:
  absl::Status create_buffers (GPUDevice *gpu, size_t vocab);
  static absl::Status hip_status (const char *what, int e);
  const float *current_logits () const;
  GPUDevice *gpu_ = nullptr;
  Tensor logits32_; // fp32 [vocab] written by the fused step
  Tensor tok_slot_; // pinned uint32
  Tensor adopted_;  // logits of the operator chain, if newer
  bool adopted_valid_ = false;
  size_t vocab_ = 0;
};
}
#endif
