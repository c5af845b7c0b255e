#include "src/ops/row_mixer.h"
#include "models/weights.h"
#include "src/core/command.h"
#include "vkl_hip.h"
#include <string.h>

namespace vkllama
{
void
PackedMatrix::put (const uint16_t *src, int n, int src_cols, int r0, int c0)
{
  for (int r = 0; r < n; ++r)
    memcpy (data.data () + (size_t)(r0 + r) * cols + c0, src + (size_t)r * src_cols, (size_t)src_cols * 2);
}

void
PackedMatrix::put_heads (const uint16_t *src, int H, int n, int np, int src_cols, int r0)
{
  for (int h = 0; h < H; ++h)
    put (src + (size_t)h * n * src_cols, n, src_cols, r0 + h * np);
}

void
PackedMatrix::put_head_columns (const uint16_t *src, int H, int n, int np)
{
  for (int r = 0; r < rows; ++r)
    for (int h = 0; h < H; ++h)
      memcpy (data.data () + (size_t)r * cols + (size_t)h * np, src + ((size_t)r * H + h) * n, (size_t)n * 2);
}

absl::StatusOr<Tensor>
PackedMatrix::upload (GPUDevice *dev, Command *command) const
{
  Tensor t (1, rows, cols, dev, BF16);
  VKLLAMA_STATUS_OK (t.create ());
  VKLLAMA_STATUS_OK (command->upload (data.data (), data.size (), t));
  return t;
}

absl::StatusOr<Tensor>
upload_vector (GPUDevice *dev, Command *command, const std::vector<float> &v, int padded)
{
  std::vector<float> z (v);
  z.resize ((size_t)padded, 0.f);
  Tensor t (1, 1, padded, dev, FP32);
  VKLLAMA_STATUS_OK (t.create ());
  VKLLAMA_STATUS_OK (command->upload (z.data (), z.size (), t));
  return t;
}

absl::Status
RowMixer::init () noexcept
{
  if (p_.dtype != BF16 && p_.dtype != FP32)
    return absl::InvalidArgumentError ("row mixer: only bf16 and fp32 activations are supported.");
  if (p_.heads <= 0 || p_.kv_heads <= 0 || p_.heads % p_.kv_heads || p_.dim <= 0 || p_.vdim <= 0 || p_.maxlen <= 0
      || p_.runs <= 0 || p_.temp_every <= 0)
    return absl::InvalidArgumentError (
        absl::StrFormat ("row mixer: sizes do not fit: %d heads, %d key/value heads, head sizes %d and %d", p_.heads,
                         p_.kv_heads, p_.dim, p_.vdim));
  for (int i = 0; i < p_.runs; ++i)
    {
      Tensor c (1, p_.maxlen, cache_width_ (), dev_, p_.dtype);
      VKLLAMA_STATUS_OK (c.create ());
      if (int e = vkl_memset (c.data (), 0, c.bytes (), dev_->stream ()))
        return launch_status ("clearing a cache", e);
      caches_.push_back (c);
    }
  return absl::OkStatus ();
}

absl::Status
RowMixer::pack_out (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  auto o = w.matrix (prefix + "o", (size_t)p_.width, (size_t)p_.heads * p_.vdim);
  VKLLAMA_STATUS_OK (o);
  m.put_head_columns (*o, p_.heads, p_.vdim, vdim_);
  return absl::OkStatus ();
}

void *
RowMixer::cache_row_ (int run, size_t pos)
{
  Tensor &c = caches_[(size_t)run];
  return (uint8_t *)c.data () + pos * c.hs ();
}

absl::Status
RowMixer::grow_ (Tensor &t, int rows, int width, GPUDevice *dev, DType dtype)
{
  if ((int)t.width () == width && (int)t.height () >= rows && t.dtype () == dtype)
    return absl::OkStatus ();
  t = Tensor (1, rows, width, dev, dtype);
  return t.create ();
}

absl::Status
RowMixer::attend_rows_ (const void *q, int qtype, size_t qs, int run, int groups, int dim, int S, size_t offset,
                        void *out, int otype, size_t os)
{
  const size_t need = vkl_attn_rows_scratch_bytes (type_ (), p_.heads, groups, dim, S);
  if (scratch_.bytes () < need)
    {
      scratch_ = Tensor (1, 1, (int)need, dev_, INT8);
      VKLLAMA_STATUS_OK (scratch_.create ());
      if (int e = vkl_memset (scratch_.data (), 0, need, dev_->stream ()))
        return launch_status ("clearing attention scratch", e);
    }
  Tensor &c = caches_[(size_t)run];
  return launch_status ("attention over rows",
                        vkl_attn_rows (q, qtype, qs, c.data (), type_ (), c.width (), p_.heads, groups, dim, S,
                                       (uint32_t)offset, p_.scale, p_.temp_coef, p_.temp_every, out, otype, os,
                                       scratch_.data (), dev_->stream ()));
}
}
