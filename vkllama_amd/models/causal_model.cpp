#include "models/causal_model.h"
#include "absl/strings/str_format.h"
#include "vkl_decode.h"
#include "vkl_hip.h"
#include <algorithm>
#include <chrono>

namespace vkllama
{
absl::Status
CausalModel::set_option (const std::string &name, int value)
{
  if (name == "fused_decode")
    set_fused_decode (value != 0);
  else if (name == "decode_graph")
    set_decode_graph (value != 0);
  else
    return absl::InvalidArgumentError ("unknown option " + name);
  return absl::OkStatus ();
}

absl::Status
CausalModel::check_span_ (size_t n, size_t offset) const
{
  if (n == 0)
    return absl::InvalidArgumentError ("model called with no tokens");
  if (offset + n > maxlen_)
    return absl::OutOfRangeError (absl::StrFormat ("positions [%zu, %zu) exceed the context length %zu", offset,
                                                   offset + n, maxlen_));
  return absl::OkStatus ();
}

absl::Status
CausalModel::begin_pass_ (size_t offset)
{
  if (stateful_ && offset != 0 && offset != next_pos_)
    return absl::FailedPreconditionError (absl::StrFormat (
        "a pass at position %zu: the recurrent state is not there (a pass continues the last one or starts at 0)",
        offset));
  next_pos_ = (size_t)-1;
  return absl::OkStatus ();
}

absl::StatusOr<std::vector<float> >
CausalModel::operator() (std::vector<uint32_t> const &toks, const size_t offset)
{
  return forward_rows (toks, offset, { (uint32_t)(toks.empty () ? 0 : toks.size () - 1) });
}

absl::StatusOr<std::vector<float> >
CausalModel::forward_rows (std::vector<uint32_t> const &toks, const size_t offset, std::vector<uint32_t> const &rows)
{
  StepPlan *plan = plan_ptr_ ();
  if (!plan)
    return absl::InternalError ("model used before init()");
  VKLLAMA_STATUS_OK (check_span_ (toks.size (), offset));
  for (uint32_t r : rows)
    if (r >= toks.size ())
      return absl::OutOfRangeError (absl::StrFormat ("row %u of a pass over %zu tokens", r, toks.size ()));
  VKLLAMA_STATUS_OK (begin_pass_ (offset));
  std::vector<float> out (rows.size () * vocab_);
  if (fused_decode_ && toks.size () == 1 && plan->usable ())
    {
      VKLLAMA_STATUS_OK (wait_all_ ());
      VKLLAMA_STATUS_OK (plan->step_host_token (toks[0], offset));
      std::vector<float> one (vocab_);
      auto rs = plan->read_logits (one.data ());
      if (absl::IsUnavailable (rs))
        {
          // a wait between workgroups gave up; the plan has switched to the
          // launches that wait for nothing: the same step once more
          ++decode_recoveries_;
          VKLLAMA_STATUS_OK (plan->step_host_token (toks[0], offset));
          rs = plan->read_logits (one.data ());
        }
      VKLLAMA_STATUS_OK (rs);
      for (size_t i = 0; i < rows.size (); ++i)
        std::copy (one.begin (), one.end (), out.begin () + i * vocab_);
      end_pass_ (offset + 1);
      return out;
    }
  auto logits = forward_ (toks, offset, rows);
  VKLLAMA_STATUS_OK (logits);
  if (!rows.empty ())
    if (int e = vkl_memcpy_d2h (out.data (), logits->data (), out.size () * sizeof (float), gpu_->stream ()))
      return absl::InternalError (vkl_error_string (e));
  VKLLAMA_STATUS_OK (wait_all_ ());
  end_pass_ (offset + toks.size ());
  return out;
}

// the next token from the logits of the last pass: arg-max, or a draw from
// the top-k / top-p candidates with the uniform number of (seed, position)
absl::Status
CausalModel::pick_token_ (uint32_t *dst, size_t position)
{
  if (!samp_on_)
    return plan_ptr_ ()->argmax_logits (dst);
  return plan_ptr_ ()->sample_logits (dst, samp_k_, samp_p_, samp_seed_,
                               (uint32_t)position);
}

absl::Status
CausalModel::generate_sampled (std::vector<uint32_t> const &prompt, size_t n_gen,
                               int topk, float topp, uint64_t seed,
                         std::vector<uint32_t> &out, double *prefill_ms,
                         double *decode_ms)
{
  if (topp < 0.f && topk < 1)
    return absl::InvalidArgumentError ("top-k sampling needs k >= 1");
  if (topp > 1.f)
    return absl::InvalidArgumentError ("top-p sampling needs p in [0, 1]");
  samp_on_ = true, samp_k_ = topk, samp_p_ = topp, samp_seed_ = seed;
  auto s = generate_greedy (prompt, n_gen, out, prefill_ms, decode_ms);
  samp_on_ = false;
  return s;
}

absl::Status
CausalModel::generate_greedy (std::vector<uint32_t> const &prompt, size_t n_gen,
                        std::vector<uint32_t> &out, double *prefill_ms,
                        double *decode_ms)
{
  auto s = generate_once_ (prompt, n_gen, out, prefill_ms, decode_ms);
  if (absl::IsUnavailable (s))
    {
      // a wait between workgroups gave up somewhere in the loop; the plan has
      // switched to the launches that wait for nothing.  The generation is
      // repeated from the prompt: KV rows written so far are rewritten with
      // the same values.
      ++decode_recoveries_;
      s = generate_once_ (prompt, n_gen, out, prefill_ms, decode_ms);
    }
  return s;
}

absl::Status
CausalModel::generate_once_ (std::vector<uint32_t> const &prompt, size_t n_gen,
                       std::vector<uint32_t> &out, double *prefill_ms,
                       double *decode_ms)
{
  using clock = std::chrono::steady_clock;
  out.clear ();
  if (n_gen == 0)
    return absl::OkStatus ();
  if (prompt.empty ())
    return absl::InvalidArgumentError ("empty prompt");
  if (prompt.size () + n_gen - 1 > maxlen_)
    return absl::OutOfRangeError (absl::StrFormat (
        "prompt of %zu + %zu generated tokens exceed the context length %zu",
        prompt.size (), n_gen, maxlen_));
  StepPlan *plan = plan_ptr_ ();
  if (!plan)
    return absl::InternalError ("model used before init()");
  // generated ids stay in device memory between steps (the arg-max of step i
  // is the input token of step i + 1) and are copied out once at the end
  if (next_tok_.width () < n_gen)
    {
      VKLLAMA_STATUS_OK (wait_all_ ());
      next_tok_ = Tensor (1, 1, n_gen, gpu_, UINT32, false);
      VKLLAMA_STATUS_OK (next_tok_.create ());
    }
  uint32_t *ids = (uint32_t *)next_tok_.data ();
  void *s = gpu_->stream ();
  VKLLAMA_STATUS_OK (begin_pass_ (0));

  const auto t0 = clock::now ();
  // prompt pass; arg-max of its fp16 logits becomes ids[0]
  if (fused_decode_ && prompt.size () == 1 && plan->usable ())
    {
      VKLLAMA_STATUS_OK (plan->step_host_token (prompt[0], 0));
    }
  else
    {
      auto logits32 = forward_ (prompt, 0, { (uint32_t)(prompt.size () - 1) });
      VKLLAMA_STATUS_OK (logits32);
      VKLLAMA_STATUS_OK (plan->adopt_logits (*logits32));
    }
  VKLLAMA_STATUS_OK (pick_token_ (ids + 0, prompt.size ()));
  if (int e = vkl_stream_sync (s))
    return absl::InternalError (vkl_error_string (e));
  const auto t1 = clock::now ();
  size_t n_toks = prompt.size () + 1;
  size_t i0 = 1;
  if (fused_decode_ && plan->usable () && decode_graph_ && n_gen > 1)
    {
      // ids[0] is at position prompt.size (); each replay appends one id
      if (samp_on_)
        {
          VKLLAMA_STATUS_OK (plan->loop_sampled (ids, prompt.size (), n_gen - 1, samp_k_,
                                                  samp_p_, samp_seed_));
        }
      else
        {
          VKLLAMA_STATUS_OK (plan->loop (ids, prompt.size (), n_gen - 1));
        }
      i0 = n_gen;
    }
  for (size_t i = i0; i < n_gen; ++i, ++n_toks)
    {
      if (fused_decode_ && plan->usable ())
        {
          // the step's last launch reduces the arg-max partials into ids[i]
          VKLLAMA_STATUS_OK (plan->step_device_token (
              ids + (i - 1), n_toks - 1, samp_on_ ? nullptr : ids + i));
          if (samp_on_)
            VKLLAMA_STATUS_OK (pick_token_ (ids + i, n_toks));
          continue;
        }
      else
        {
          uint32_t prev = 0;
          if (int e = vkl_memcpy_d2h (&prev, ids + (i - 1), sizeof (prev), s))
            return absl::InternalError (vkl_error_string (e));
          if (int e = vkl_stream_sync (s))
            return absl::InternalError (vkl_error_string (e));
          auto logits32 = forward_ ({ prev }, n_toks - 1, { 0u });
          VKLLAMA_STATUS_OK (logits32);
          VKLLAMA_STATUS_OK (plan->adopt_logits (*logits32));
        }
      VKLLAMA_STATUS_OK (pick_token_ (ids + i, n_toks));
    }
  if (int e = vkl_stream_sync (s))
    return absl::InternalError (vkl_error_string (e));
  const auto t2 = clock::now ();
  VKLLAMA_STATUS_OK (plan->check ());
  // run deferred work the operator chain may have queued
  VKLLAMA_STATUS_OK (wait_all_ ());
  end_pass_ (prompt.size () + n_gen - 1);
  out.resize (n_gen);
  if (int e = vkl_memcpy_d2h (out.data (), ids, n_gen * sizeof (uint32_t), s))
    return absl::InternalError (vkl_error_string (e));
  if (int e = vkl_stream_sync (s))
    return absl::InternalError (vkl_error_string (e));
  if (prefill_ms)
    *prefill_ms = std::chrono::duration<double, std::milli> (t1 - t0).count ();
  if (decode_ms)
    *decode_ms = std::chrono::duration<double, std::milli> (t2 - t1).count ();
  return absl::OkStatus ();
}
}
