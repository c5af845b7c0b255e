// TokenMixer: the part of a decoder layer that mixes tokens.  The layer multiplies
// its normed input with ONE matrix; a mixer says which output rows of that matrix
// it needs and where they go, mixes, and keeps what later tokens need - cached rows
// or a recurrent state - one set per layer run: a layer that runs several times has
// several.  Not part of the reference.
#ifndef __VKLLAMA_TOKEN_MIXER_H__
#define __VKLLAMA_TOKEN_MIXER_H__
#include "src/ops/op.h"
#include "vkl_stack.h"
#include <string>
#include <vector>

// Takes the value of an absl::StatusOr or returns its status.
#define VKL_TAKE(dst, expr)                                                   \
  do                                                                          \
    {                                                                         \
      auto v__ = (expr);                                                      \
      if (!v__.ok ())                                                         \
        return v__.status ();                                                 \
      dst = *v__;                                                             \
    }                                                                         \
  while (0)

namespace vkllama
{
class WeightSource;

// sizes as the configuration gives them; a mixer reads those it has
struct MixerParams
{
  int width = 0;    // of the layer input
  int heads = 0, kv_heads = 1;
  int dim = 0, vdim = 0;
  float scale = 1.f;
  float eps = 0.f;  // of norms inside the mixer
  int maxlen = 0;
  int runs = 1;     // caches
  DType dtype = BF16; // stored activations and caches: BF16 or FP32

  int kv_rank = 0;  // latent attention
  float temp_coef = 0.f; // queries grow by 1 + coef ln (floor ((p + 1) / every) + 1)
  int temp_every = 1;

  std::vector<double> freq; // rotation: a frequency per pair, pairs are the halves of the first 2 * size () values
  int chunk = 0;    // positions see their own chunk of this many only (0: everything before them)
  bool sink = false; // the softmax has a score of 0 without a value
  bool v_mix = false; // values are mixed with those of the first such layer

  int taps = 0;     // short convolutions
  std::vector<double> decay; // a factor per head
};

// up to this many tokens a pass takes the kernels written for few rows
constexpr int kFewRows = 16;

inline int
round_up (int n, int to)
{
  return (n + to - 1) / to * to;
}

// A bf16 matrix assembled on the host before it is uploaded; zero where nothing
// is put.
struct PackedMatrix
{
  int rows = 0, cols = 0;
  std::vector<uint16_t> data;
  PackedMatrix (int r, int c) : rows (r), cols (c), data ((size_t)r * c, 0) {}
  // n rows of a [.., src_cols] matrix to row r0, column c0
  void put (const uint16_t *src, int n, int src_cols, int r0, int c0 = 0);
  // head by head: H heads of `n` rows each, to heads of `np` rows
  void put_heads (const uint16_t *src, int H, int n, int np, int src_cols, int r0);
  // columns head by head: [rows, H*n] to heads of np columns
  void put_head_columns (const uint16_t *src, int H, int n, int np);
  absl::StatusOr<Tensor> upload (GPUDevice *dev, Command *command) const;
};
absl::StatusOr<Tensor> upload_vector (GPUDevice *dev, Command *command, const std::vector<float> &v, int padded);

class TokenMixer : public Op
{
public:
  TokenMixer (GPUDevice *dev, Command *command, const MixerParams &p) : Op (dev, command), p_ (p) {}
  // takes its weights (tensor names <prefix>q, ...)
  virtual absl::Status load (const WeightSource &w, const std::string &prefix) = 0;
  absl::Status init () noexcept override;
  uint64_t time () noexcept override { return timer_.micros (); }

  // rows of the layer's input matrix this mixer needs (a multiple of 8), and
  // their contents from row 0 on
  virtual int in_rows () const = 0;
  virtual absl::Status pack_in (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const = 0;
  // columns of the layer's output matrix the heads fill
  int out_cols () const { return p_.heads * vdim_; }
  absl::Status pack_out (const WeightSource &w, const std::string &prefix, PackedMatrix &m) const;

  // the destinations of those rows for S tokens at `offset` of run `run`
  virtual absl::StatusOr<std::vector<vkl_out_seg> > segments (int S, size_t offset, int run) = 0;
  // after the product: the heads' outputs to out [S, out_cols], row stride os
  virtual absl::Status mix (int S, size_t offset, int run, void *out, size_t os) = 0;
  // this mixer's part of the one-token step's layer table
  virtual void describe (vkl_stack_layer &l, int run) = 0;
  // bytes of the cache a position occupies
  virtual size_t row_bytes () const { return 0; }
  // bytes of a state that a token reads and writes
  virtual size_t state_bytes () const { return 0; }
  // the cached rows a token at position pos reads
  virtual size_t rows_read (size_t pos) const { return pos + 1; }
  // bytes of weights the one-token step reads in here
  virtual size_t weight_bytes () const { return 0; }

protected:
  int type_ () const { return p_.dtype == FP32 ? VKL_TYPE_F32 : VKL_TYPE_BF16; }
  // a buffer of at least that many values, kept between calls
  static absl::Status grow_ (Tensor &t, int rows, int width, GPUDevice *dev, DType dtype);
  // the same, zeroed when it is made
  absl::Status grow_zeroed_ (Tensor &t, int rows, int width, DType dtype);
  MixerParams p_;
  int dim_ = 0, vdim_ = 0; // head sizes, padded
};
}
#endif
