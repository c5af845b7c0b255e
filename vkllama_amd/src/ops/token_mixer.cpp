#include "src/ops/token_mixer.h"
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
TokenMixer::init () noexcept
{
  if (p_.dtype != BF16 && p_.dtype != FP32)
    return absl::InvalidArgumentError ("token mixer: only bf16 and fp32 activations are supported.");
  if (p_.heads <= 0 || p_.kv_heads <= 0 || p_.heads % p_.kv_heads || p_.dim <= 0 || p_.vdim <= 0 || p_.maxlen <= 0
      || p_.runs <= 0 || p_.temp_every <= 0)
    return absl::InvalidArgumentError (
        absl::StrFormat ("token mixer: sizes do not fit: %d heads, %d key/value heads, head sizes %d and %d", p_.heads,
                         p_.kv_heads, p_.dim, p_.vdim));
  return absl::OkStatus ();
}

absl::Status
TokenMixer::pack_out (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const
{
  auto o = w.matrix (prefix + "o", (size_t)p_.width, (size_t)p_.heads * p_.vdim);
  VKLLAMA_STATUS_OK (o);
  m.put_head_columns (*o, p_.heads, p_.vdim, vdim_);
  return absl::OkStatus ();
}

absl::Status
TokenMixer::grow_ (Tensor &t, int rows, int width, GPUDevice *dev, DType dtype)
{
  if ((int)t.width () == width && (int)t.height () >= rows && t.dtype () == dtype)
    return absl::OkStatus ();
  t = Tensor (1, rows, width, dev, dtype);
  return t.create ();
}

absl::Status
TokenMixer::grow_zeroed_ (Tensor &t, int rows, int width, DType dtype)
{
  if ((int)t.width () == width && (int)t.height () >= rows && t.dtype () == dtype)
    return absl::OkStatus ();
  t = Tensor (1, rows, width, dev_, dtype);
  VKLLAMA_STATUS_OK (t.create ());
  if (int e = vkl_memset (t.data (), 0, t.bytes (), dev_->stream ()))
    return launch_status ("clearing a buffer", e);
  return absl::OkStatus ();
}
}
