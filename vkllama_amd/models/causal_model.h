// CausalModel: what every model of this library offers - a pass over the next
// tokens of a sequence at a cache position, and generation - with the token
// loop itself: prompt pass, token pick on the device, the one-token step
// replayed from a graph.  A model family supplies its prompt pass and its
// StepPlan.  The loop is that of the reference's app/llama2_infer.cpp:140-218.
#ifndef __VKLLAMA_MODELS_CAUSAL_MODEL_H__
#define __VKLLAMA_MODELS_CAUSAL_MODEL_H__
#include "absl/status/statusor.h"
#include "models/step_plan.h"
#include "src/core/gpu_device.h"
#include "src/core/tensor.h"
#include <memory>
#include <string>
#include <vector>

namespace vkllama
{
class CausalModel
{
public:
  virtual ~CausalModel () {}
  CausalModel (const CausalModel &) = delete;
  CausalModel &operator= (const CausalModel &) = delete;

  // one pass over `toks` at cache position `offset`: logits of the last row
  absl::StatusOr<std::vector<float> > operator() (std::vector<uint32_t> const &toks, const size_t offset);
  // the same with the logits of the given rows of `toks` (in that order, may be
  // none): [rows, vocab]
  absl::StatusOr<std::vector<float> > forward_rows (std::vector<uint32_t> const &toks, const size_t offset,
                                                    std::vector<uint32_t> const &rows);

  // single tokens on the fused step (default) or on the operator chain
  void set_fused_decode (bool on) { fused_decode_ = on; }
  // greedy loop replayed from a captured HIP graph (default) or launched step
  // by step
  void set_decode_graph (bool on) { decode_graph_ = on; }
  // options of the model family: InvalidArgument for an unknown name or a bad
  // value
  virtual absl::Status set_option (const std::string &name, int value);

  // Greedy loop of app/llama2_infer.cpp:140-218: prompt at offset 0, then one
  // token at a time at offset toks.size()-1; n_gen ids are written to out.
  // The wall-clock times of the two phases are returned in milliseconds.
  absl::Status generate_greedy (std::vector<uint32_t> const &prompt, size_t n_gen, std::vector<uint32_t> &out,
                                double *prefill_ms = nullptr, double *decode_ms = nullptr);
  // The same loop with the token drawn on the device from the top-k
  // (topp < 0) or top-p candidates of every step's logits
  // (models/samplers.cpp:37-101 as a kernel): logits never leave the device.
  // The draw at position pos uses the uniform number of (seed, pos).
  absl::Status generate_sampled (std::vector<uint32_t> const &prompt, size_t n_gen, int topk, float topp,
                                 uint64_t seed, std::vector<uint32_t> &out, double *prefill_ms = nullptr,
                                 double *decode_ms = nullptr);

  GPUDevice *device () { return gpu_; }
  size_t vocab_size () const { return vocab_; }
  size_t context_length () const { return maxlen_; }
  // algorithmic bytes one decode step at context length L reads and writes
  virtual size_t decode_step_bytes (size_t L) const = 0;
  // how often a decode step or generation was repeated because a wait between
  // workgroups inside a launch had given up (StepPlan::check)
  size_t decode_recoveries () const { return decode_recoveries_; }

protected:
  CausalModel () {}
  // One pass of the operator chain; fp32 logits [1, rows, vocab] of the given
  // rows, last row only for a family that offers no other
  virtual absl::StatusOr<Tensor> forward_ (std::vector<uint32_t> const &toks, const size_t offset,
                                           std::vector<uint32_t> const &rows)
      = 0;
  // waits for queued work and runs what was deferred until then
  virtual absl::Status wait_all_ () = 0;
  virtual StepPlan *plan_ptr_ () = 0;
  absl::Status check_span_ (size_t n, size_t offset) const;
  // A family with a recurrent state (stateful_) goes through a sequence in order: a
  // pass starts where the last one ended, or at 0.  begin_pass_ checks that, and the
  // state has no position until end_pass_ gives it the new one.
  absl::Status begin_pass_ (size_t offset);
  void end_pass_ (size_t next) { next_pos_ = next; }

  GPUDevice *gpu_ = nullptr;
  size_t vocab_ = 0, maxlen_ = 0;
  bool fused_decode_ = true;
  bool decode_graph_ = true;
  size_t decode_recoveries_ = 0;
  bool stateful_ = false;

private:
  size_t next_pos_ = 0;
  Tensor next_tok_;
  // sampling on the device during generate_*(): off = arg-max
  bool samp_on_ = false;
  int samp_k_ = 1;
  float samp_p_ = -1.f;
  uint64_t samp_seed_ = 0;
  absl::Status pick_token_ (uint32_t *dst, size_t position);
  absl::Status generate_once_ (std::vector<uint32_t> const &prompt, size_t n_gen, std::vector<uint32_t> &out,
                               double *prefill_ms, double *decode_ms);

protected:
  // (the id buffer belongs to the device: a family's destructor drops it before
  // the device goes)
  void release_buffers_ () { next_tok_ = Tensor (); }
};
}
#endif
