// Linear recurrences of decoder stacks (include/vkl_stack.h): the gated delta
// rule with a decay per key channel, and sums that decay by a factor per head.
// Per head a state M [dim, vdim]:
//   delta:  M <- diag (g_t) M,  u_t = beta_t (v_t - M^T k_t),  M <- M + k_t u_t^T
//   decay:  M <- c M + k_t v_t^T                      and in both  o_t = M^T q_t
// State and arithmetic are fp32 throughout.  Three forms:
//
// TOKENS: one wave per (head, 16 value columns) walks the tokens, the state in
// registers: lane l holds column l % 16 and rows 16 j + 4 (l / 16) + 0..3.
//
// CHUNKS: 64 tokens at a time as products.  With D_i the product of the decays of
// a chunk's tokens up to i and M0 the state before it,
//   u = T (diag (beta) V - diag (beta) (K D) M0),  T = (1 + A)^-1,
//   A_ij = beta_i sum_d k_i k_j D_i / D_j  (j < i),
//   o = (Q D) M0 + P u,  P_ij = sum_d q_i k_j D_i / D_j  (j <= i),
//   M = diag (D_64) M0 + (K D_64 / D)^T u
// (decay: the same with u = V).  A first launch, all chunks at once, computes what
// does not depend on the state (P, Q D, K D_64 / D, D_64, and for the delta rule T
// applied to both parts of u); a second walks the chunks, a workgroup per (head,
// 16 value columns).  The quotients D_i / D_j are formed from logarithms summed
// within blocks of 16 tokens, relative to the edge of a block, so that no exponent
// is positive; inside a block, where that is impossible, the factors are split at
// the block's start as long as the block decays by less than 2^-58, and formed
// pair by pair otherwise.
// Products run on v_mfma_f32_16x16x4_f32.  Its k index may be permuted: operands
// hold k = 16 b + 4 (lane / 16) + e in step (b, e), so that a result block, of which
// a lane holds rows 4 (lane / 16) + 0..3, is the right operand of the next product as
// it lies.
//
// STEP: one token in the one-token step, a workgroup per head, with everything
// between the projections: convolutions, unit norms, decays, the output's norm
// and gate.
#include "../../include/vkl_stack.h"
#include "vkl_stack_dev.h"
#include <algorithm>

namespace vkl
{
namespace
{
typedef float f4 __attribute__ ((ext_vector_type (4)));
constexpr int kChunk = 64, kBlocks = kChunk / 16;

__device__ __forceinline__ f4
mfma4 (float a, float b, f4 c)
{
  return __builtin_amdgcn_mfma_f32_16x16x4f32 (a, b, c, 0, 0, 0);
}

__device__ __forceinline__ f4
ldf4 (const float *p)
{
  return __builtin_bit_cast (f4, ldg4 (p));
}

__device__ __forceinline__ void
stf4 (float *p, f4 v)
{
  stg ((vkl_u32x4 *)p, __builtin_bit_cast (vkl_u32x4, v));
}

// Rows in one of the two formats: T is float, or uint16_t for bf16.  (The format is a
// template parameter wherever many loads are in flight: a branch per load would
// wait for each.)
template <typename T>
__device__ __forceinline__ f4
load4 (const void *p, size_t i)
{
  if constexpr (sizeof (T) == 4)
    return ldf4 ((const float *)p + i);
  const unsigned long long w = ldg ((const unsigned long long *)((const uint16_t *)p + i));
  const uint32_t lo = (uint32_t)w, hi = (uint32_t)(w >> 32);
  return f4{ __uint_as_float (lo << 16), __uint_as_float (lo & 0xffff0000u), __uint_as_float (hi << 16),
             __uint_as_float (hi & 0xffff0000u) };
}

__device__ __forceinline__ float
value_of (float v)
{
  return v;
}

__device__ __forceinline__ float
value_of (uint16_t v)
{
  return bf2f (v);
}

template <typename T>
__device__ __forceinline__ float
load1 (const void *p, size_t i)
{
  return value_of (ldg ((const T *)p + i));
}

template <typename T>
__device__ __forceinline__ void
store4 (void *p, size_t i, f4 v)
{
  if constexpr (sizeof (T) == 4)
    stf4 ((float *)p + i, v);
  else
    stg ((unsigned long long *)((uint16_t *)p + i),
         (unsigned long long)f2bf (v[0]) | ((unsigned long long)f2bf (v[1]) << 16) | ((unsigned long long)f2bf (v[2]) << 32)
             | ((unsigned long long)f2bf (v[3]) << 48));
}

template <typename T>
__device__ __forceinline__ void
store8 (void *p, size_t i, const float (&v)[8])
{
  if constexpr (sizeof (T) == 4)
    {
      stf4 ((float *)p + i, f4{ v[0], v[1], v[2], v[3] }), stf4 ((float *)p + i + 4, f4{ v[4], v[5], v[6], v[7] });
      return;
    }
  vkl_u32x4 w;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    w[e] = f2bf (v[2 * e]) | ((uint32_t)f2bf (v[2 * e + 1]) << 16);
  stg ((vkl_u32x4 *)((uint16_t *)p + i), w);
}

// calls f with a value of the format's type
template <typename F>
int
with_format (int type, F f)
{
  return type == VKL_TYPE_F32 ? f (float ()) : f (uint16_t ());
}

__device__ __forceinline__ float
softplus (float z)
{
  return fmaxf (z, 0.f) + log1pf (expf (-fabsf (z)));
}

// the logarithm of a decay; a factor of zero has a finite one
__device__ __forceinline__ float
log_decay_of (float rate, float z)
{
  return fmaxf (-rate * softplus (z), -1.0e4f);
}

// In the chunked form logarithms are to base 2: their powers are one instruction.
constexpr float kLog2e = 1.44269504088896340736f;

__device__ __forceinline__ float
power2 (float x)
{
  return __builtin_amdgcn_exp2f (x);
}

// 1 / (1 + e^-x) on the hardware's power and reciprocal, good to a few units of the last
// place: where every value of a large tensor takes one
__device__ __forceinline__ float
quick_sigmoid (float x)
{
  return __builtin_amdgcn_rcpf (1.0f + power2 (-kLog2e * x));
}

// log2_decay_of: kLog2e * log_decay_of, with hardware powers and logarithms.  ln (1 + x)
// comes from its series where 1 + x would round x away.
__device__ __forceinline__ float
log2_decay_of (float rate, float z)
{
  const float x = power2 (-kLog2e * fabsf (z));
  float s = __builtin_fmaf (x, -1.0f / 8, 1.0f / 7);
  s = __builtin_fmaf (x, s, -1.0f / 6);
  s = __builtin_fmaf (x, s, 1.0f / 5);
  s = __builtin_fmaf (x, s, -1.0f / 4);
  s = __builtin_fmaf (x, s, 1.0f / 3);
  s = __builtin_fmaf (x, s, -1.0f / 2);
  s = __builtin_fmaf (x, s, 1.0f) * x * kLog2e;
  const float l = x < 0.1f ? s : __builtin_amdgcn_logf (1.0f + x);
  return fmaxf (-rate * (kLog2e * fmaxf (z, 0.f) + l), -1.4427e4f);
}

// sum over the lanes that hold the same column (four groups of 16)
__device__ __forceinline__ float
rows_sum (float v)
{
  v += __shfl_xor (v, 16, 64);
  v += __shfl_xor (v, 32, 64);
  return v;
}

// ---------------------------------------------------------------------------
// short convolution
// ---------------------------------------------------------------------------
struct ConvArgs
{
  const void *x;
  int type;
  size_t xs;
  const float *w;
  int n, taps;
  float *ring;
  uint32_t pos0;
  int S;
  void *out;
  size_t os;
};

// the input of eight channels at token s of the pass (negative: of the tokens before it)
template <typename T>
__device__ __forceinline__ void
conv_input (const ConvArgs &a, int s, int c, f4 (&x)[2])
{
  x[0] = x[1] = f4{ 0.f, 0.f, 0.f, 0.f };
  if (s >= 0)
    {
      const size_t at = (size_t)s * a.xs + c;
      x[0] = load4<T> (a.x, at), x[1] = load4<T> (a.x, at + 4);
    }
  else if ((uint32_t)-s <= a.pos0)
    {
      const float *r = a.ring + (size_t)((a.pos0 - (uint32_t)-s) % (uint32_t)a.taps) * a.n + c;
      x[0] = ldf4 (r), x[1] = ldf4 (r + 4);
    }
}

template <typename T>
__device__ __forceinline__ void
conv_output (const ConvArgs &a, int s, int c, const f4 (&y)[2])
{
  float z[8];
#pragma unroll
  for (int e = 0; e < 8; ++e)
    z[e] = y[e / 4][e % 4] * quick_sigmoid (y[e / 4][e % 4]);
  store8<T> (a.out, (size_t)s * a.os + c, z);
}

constexpr int kConvRun = 4; // tokens of a thread

// eight channels of a run of tokens per thread.  TAPS: the inputs of the window and
// the weights stay in registers; 0: any number of taps
template <int TAPS, typename T>
__global__ __launch_bounds__ (256) void
short_conv_kernel (const ConvArgs a)
{
  const int n8 = a.n / 8;
  const size_t it = (size_t)blockIdx.x * 256 + threadIdx.x;
  const int s0 = (int)(it / n8) * kConvRun, c = (int)(it % n8) * 8;
  if (s0 >= a.S)
    return;
  if constexpr (TAPS > 0)
    {
      f4 w[TAPS][2], x[kConvRun + TAPS - 1][2];
#pragma unroll
      for (int j = 0; j < TAPS; ++j)
        w[j][0] = ldf4 (a.w + (size_t)j * a.n + c), w[j][1] = ldf4 (a.w + (size_t)j * a.n + c + 4);
#pragma unroll
      for (int j = 0; j < kConvRun + TAPS - 1; ++j)
        {
          const size_t at = (size_t)max (min (s0 + j - (TAPS - 1), a.S - 1), 0) * a.xs + c;
          x[j][0] = load4<T> (a.x, at), x[j][1] = load4<T> (a.x, at + 4);
        }
      if (s0 < TAPS - 1) // (the first run reaches back before the pass)
#pragma unroll
        for (int j = 0; j < TAPS - 1; ++j)
          if (s0 + j < TAPS - 1)
            conv_input<T> (a, s0 + j - (TAPS - 1), c, x[j]);
#pragma unroll
      for (int t = 0; t < kConvRun; ++t)
        {
          f4 y[2] = { { 0.f, 0.f, 0.f, 0.f }, { 0.f, 0.f, 0.f, 0.f } };
#pragma unroll
          for (int j = 0; j < TAPS; ++j)
#pragma unroll
            for (int h = 0; h < 2; ++h)
#pragma unroll
              for (int e = 0; e < 4; ++e)
                y[h][e] = __builtin_fmaf (w[j][h][e], x[t + j][h][e], y[h][e]);
          if (s0 + t < a.S)
            conv_output<T> (a, s0 + t, c, y);
        }
      return;
    }
  for (int s = s0; s < min (s0 + kConvRun, a.S); ++s)
    {
      f4 y[2] = { { 0.f, 0.f, 0.f, 0.f }, { 0.f, 0.f, 0.f, 0.f } };
      for (int j = 0; j < a.taps; ++j)
        {
          f4 x[2];
          conv_input<T> (a, s - (a.taps - 1 - j), c, x);
          const f4 w[2] = { ldf4 (a.w + (size_t)j * a.n + c), ldf4 (a.w + (size_t)j * a.n + c + 4) };
#pragma unroll
          for (int h = 0; h < 2; ++h)
#pragma unroll
            for (int e = 0; e < 4; ++e)
              y[h][e] = __builtin_fmaf (w[h][e], x[h][e], y[h][e]);
        }
      conv_output<T> (a, s, c, y);
    }
}

// the last inputs into the ring, in a launch of their own: the one above reads it
__global__ __launch_bounds__ (256) void
short_conv_keep_kernel (const ConvArgs a)
{
  const int keep = min (a.S, a.taps);
  const size_t it = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (it >= (size_t)keep * a.n)
    return;
  const int r = (int)(it / a.n), c = (int)(it - (size_t)r * a.n), s = a.S - keep + r;
  stg (a.ring + (size_t)((a.pos0 + (uint32_t)s) % (uint32_t)a.taps) * a.n + c, load_elem (a.x, a.type, (size_t)s * a.xs + c));
}

// ---------------------------------------------------------------------------
// token by token
// ---------------------------------------------------------------------------
struct RecurArgs
{
  vkl_recurrence_args r;
  int S;
  bool fresh; // the state is zero
};

template <int DJ, bool DELTA, typename T>
__global__ __launch_bounds__ (64) void
recur_tokens_kernel (const RecurArgs a)
{
  const vkl_recurrence_args &r = a.r;
  const int h = blockIdx.x % r.H, vb = blockIdx.x / r.H, lane = threadIdx.x;
  const int col = vb * 16 + (lane & 15), row = 4 * (lane >> 4);
  float *st = r.state + (size_t)h * r.dim * r.vdim + col;
  f4 m[DJ];
#pragma unroll
  for (int j = 0; j < DJ; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      m[j][e] = a.fresh ? 0.f : ldg (st + (size_t)(16 * j + row + e) * r.vdim);
  const size_t qo = (size_t)(h / r.rep) * r.dim + row, vo = (size_t)h * r.vdim + col;
  float rate = 0.f, decay = 1.f;
  if (DELTA)
    rate = ldg (r.rate + h);
  else
    decay = expf (fmaxf (ldg (r.log_decay + h), -1.0e4f));
  for (int s = 0; s < a.S; ++s)
    {
      f4 q[DJ], k[DJ], g[DJ];
#pragma unroll
      for (int j = 0; j < DJ; ++j)
        {
          q[j] = load4<T> (r.q, (size_t)s * r.qs + qo + 16 * j);
          k[j] = load4<T> (r.k, (size_t)s * r.ks + qo + 16 * j);
          if (DELTA)
            g[j] = ldf4 (r.z + (size_t)s * r.zs + (size_t)h * r.dim + 16 * j + row);
        }
      const float v = load1<T> (r.v, (size_t)s * r.vs + vo);
      float o = 0.f;
      if (DELTA)
        {
          float qq = 0.f, kk = 0.f, mk = 0.f;
#pragma unroll
          for (int j = 0; j < DJ; ++j)
            {
              const f4 bias = ldf4 (r.dt_bias + (size_t)h * r.dim + 16 * j + row);
#pragma unroll
              for (int e = 0; e < 4; ++e)
                {
                  qq = __builtin_fmaf (q[j][e], q[j][e], qq), kk = __builtin_fmaf (k[j][e], k[j][e], kk);
                  m[j][e] *= expf (log_decay_of (rate, g[j][e] + bias[e]));
                }
            }
          const float fq = r.qscale / sqrtf (rows_sum (qq) + r.unit_eps), fk = 1.0f / sqrtf (rows_sum (kk) + r.unit_eps);
#pragma unroll
          for (int j = 0; j < DJ; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e)
              {
                k[j][e] *= fk;
                mk = __builtin_fmaf (m[j][e], k[j][e], mk);
              }
          const float u = sigmoid (ldg (r.b + (size_t)s * r.bs + h)) * (v - rows_sum (mk));
#pragma unroll
          for (int j = 0; j < DJ; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e)
              {
                m[j][e] = __builtin_fmaf (k[j][e], u, m[j][e]);
                o = __builtin_fmaf (m[j][e], q[j][e], o);
              }
          o = rows_sum (o) * fq;
        }
      else
        {
#pragma unroll
          for (int j = 0; j < DJ; ++j)
#pragma unroll
            for (int e = 0; e < 4; ++e)
              {
                m[j][e] = __builtin_fmaf (k[j][e], v, decay * m[j][e]);
                o = __builtin_fmaf (m[j][e], q[j][e], o);
              }
          o = rows_sum (o) * r.qscale;
        }
      if (lane < 16)
        stg (r.out + (size_t)s * r.os + vo, o);
    }
#pragma unroll
  for (int j = 0; j < DJ; ++j)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      stg (st + (size_t)(16 * j + row + e) * r.vdim, m[j][e]);
}

// ---------------------------------------------------------------------------
// chunks: what does not depend on the state
// ---------------------------------------------------------------------------
constexpr int kPrepThreads = 512;

// floats of scratch per (chunk, head)
__host__ __device__ inline size_t
chunk_floats (int dim, int vdim)
{
  return (size_t)3 * kChunk * dim + kChunk * kChunk + (size_t)kChunk * vdim + dim;
}

// Operands lie as the second launch's lanes load them: a block of 16 rows and 16 columns
// (of the product's inner index) is 64 lanes of four values, lane = row % 16 +
// 16 (column / 4) - or, for u, as a result lies: lane = column % 16 + 16 (row / 4).
struct ChunkView
{
  float *w, *qd, *kt, *p, *u, *dec;
};

__device__ __forceinline__ ChunkView
chunk_view (float *ws, int dim, int vdim)
{
  ChunkView c;
  c.w = ws;                            // [4 token blocks][dim / 16]
  c.qd = c.w + (size_t)kChunk * dim;   // the same
  c.kt = c.qd + (size_t)kChunk * dim;  // [dim / 16][4 token blocks]
  c.p = c.kt + (size_t)kChunk * dim;   // [4][4]
  c.u = c.p + kChunk * kChunk;         // [4][vdim / 16]
  c.dec = c.u + (size_t)kChunk * vdim; // [dim]
  return c;
}

constexpr int kLdA = kChunk + 4, kLdT = 20;

inline size_t
prep_lds_bytes (int dim)
{
  return ((size_t)3 * kChunk * (dim + 4) + kChunk * kLdA + (size_t)kBlocks * dim + kChunk + kChunk * kLdT)
         * sizeof (float);
}

typedef __bf16 bf8 __attribute__ ((ext_vector_type (8)));

// x W^T for the 16 columns of W rows w0 .. +15 and kChunk rows of x from row s0 on (n of
// them exist), K a multiple of 64: acc[m][e] is row 16 m + 4 (lane / 16) + e, column
// lane % 16
template <typename T>
__device__ __forceinline__ void
low_rank_tile (const void *x, size_t xs, int s0, int n, const uint16_t *w, int K, int lane,
               f4 (&acc)[kBlocks])
{
  const int lo = lane & 15, q = lane >> 4;
  size_t row[kBlocks];
#pragma unroll
  for (int m = 0; m < kBlocks; ++m)
    {
      acc[m] = f4{ 0.f, 0.f, 0.f, 0.f };
      row[m] = (size_t)(s0 + min (16 * m + lo, n - 1)) * xs;
    }
  const uint16_t *wr = w + (size_t)lo * K;
  if constexpr (sizeof (T) == 2)
    {
      for (int k0 = 0; k0 < K; k0 += 64)
#pragma unroll
        for (int k = k0 + 8 * q, u = 0; u < 2; ++u, k += 32)
          {
            const bf8 b = __builtin_bit_cast (bf8, ldg4 (wr + k));
#pragma unroll
            for (int m = 0; m < kBlocks; ++m)
              acc[m] = __builtin_amdgcn_mfma_f32_16x16x32_bf16 (
                  __builtin_bit_cast (bf8, ldg4 ((const uint16_t *)x + row[m] + k)), b, acc[m], 0, 0, 0);
          }
      return;
    }
  for (int k = 4 * q; k < K; k += 16)
    {
      const f4 b = load4<uint16_t> (wr, (size_t)k);
#pragma unroll
      for (int m = 0; m < kBlocks; ++m)
        {
          const f4 v = ldf4 ((const float *)x + row[m] + k);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            acc[m] = mfma4 (v[e], b[e], acc[m]);
        }
    }
}

template <bool DELTA, typename T>
__global__ __launch_bounds__ (kPrepThreads) void
chunk_prep_kernel (const RecurArgs a, float *ws)
{
  extern __shared__ __align__ (16) float lds_prep[];
  const vkl_recurrence_args &r = a.r;
  const int D = r.dim, LD = D + 4;
  float *ks = lds_prep;           // [64][LD]: unit keys
  float *qs = ks + kChunk * LD;   // scaled queries
  float *ls = qs + kChunk * LD;   // logarithms, summed from the start of a block of 16
  float *A = ls + kChunk * LD;    // [64][kLdA]
  float *es = A + kChunk * kLdA;  // [4][D]: a block's sum
  float *beta = es + kBlocks * D; // [64]
  float *Ti = beta + kChunk;      // [4][16][kLdT]: (1 + A)^-1 of the blocks on the diagonal
  __shared__ uint32_t steep;
  const int h = blockIdx.x % r.H, c = blockIdx.x / r.H, s0 = c * kChunk;
  const int n = min (kChunk, a.S - s0); // tokens; the rest of the chunk changes nothing
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lo = lane & 15, hi = 4 * (lane >> 4);
  const ChunkView v = chunk_view (ws + ((size_t)c * r.H + h) * chunk_floats (D, r.vdim), D, r.vdim);
  if (tid == 0)
    steep = 0;
  const size_t qo = (size_t)(h / r.rep) * D;
  const float rate = DELTA ? ldg (r.rate + h) : 0.f;
  const float ld = DELTA ? 0.f : kLog2e * fmaxf (ldg (r.log_decay + h), -1.0e4f);
  {
    // queries and keys: 16 lanes per token, eight channels each
    constexpr int PASS = kChunk / (kPrepThreads / 16);
    const int d = 8 * lo, dc = min (d, D - 8);
    f4 x[PASS][2][2], z[PASS][2];
    float bv[PASS];
#pragma unroll
    for (int p = 0; p < PASS; ++p)
      {
        const int i = (p * 8 + wave) * 4 + (lane >> 4);
        const size_t s = (size_t)(s0 + min (i, n - 1));
#pragma unroll
        for (int e = 0; e < 2; ++e)
          {
            x[p][0][e] = load4<T> (r.q, s * r.qs + qo + dc + 4 * e);
            x[p][1][e] = load4<T> (r.k, s * r.ks + qo + dc + 4 * e);
            if (DELTA && !r.a1)
              z[p][e] = ldf4 (r.z + s * r.zs + (size_t)h * D + dc + 4 * e);
          }
        if (DELTA)
          bv[p] = ldg (r.b + s * r.bs + h);
      }
    if constexpr (DELTA)
      if (r.a1 && 16 * wave < D)
        {
          f4 acc[kBlocks];
          low_rank_tile<T> (r.a1, r.as, s0, n, (const uint16_t *)r.w_a2 + ((size_t)h * D + 16 * wave) * r.r_a, r.r_a,
                         lane, acc);
          const float bias = ldg (r.dt_bias + (size_t)h * D + 16 * wave + lo);
#pragma unroll
          for (int m = 0; m < kBlocks; ++m)
#pragma unroll
            for (int e = 0; e < 4; ++e)
              {
                const int i = 16 * m + hi + e;
                ls[i * LD + 16 * wave + lo] = i < n ? log2_decay_of (rate, acc[m][e] + bias) : 0.f;
              }
        }
#pragma unroll
    for (int p = 0; p < PASS; ++p)
      {
        const int i = (p * 8 + wave) * 4 + (lane >> 4);
        const bool in = i < n;
        float qq = 0.f, kk = 0.f;
#pragma unroll
        for (int e = 0; e < 8; ++e)
          {
            const float qv = in && d < D ? x[p][0][e >> 2][e & 3] : 0.f, kv = in && d < D ? x[p][1][e >> 2][e & 3] : 0.f;
            x[p][0][e >> 2][e & 3] = qv, x[p][1][e >> 2][e & 3] = kv;
            qq = __builtin_fmaf (qv, qv, qq), kk = __builtin_fmaf (kv, kv, kk);
          }
        float fq = r.qscale, fk = 1.f;
        if (DELTA)
          {
            fq = r.qscale / sqrtf (row_sum<16> (qq) + r.unit_eps), fk = 1.0f / sqrtf (row_sum<16> (kk) + r.unit_eps);
            if (lo == 0)
              beta[i] = in ? sigmoid (bv[p]) : 0.f;
          }
        if (d >= D)
          continue;
#pragma unroll
        for (int e = 0; e < 2; ++e)
          {
            *(f4 *)(qs + i * LD + d + 4 * e) = x[p][0][e] * fq;
            *(f4 *)(ks + i * LD + d + 4 * e) = x[p][1][e] * fk;
            if (DELTA && r.a1)
              continue;
            f4 l;
#pragma unroll
            for (int g = 0; g < 4; ++g)
              {
                if (DELTA)
                  l[g] = log2_decay_of (rate, z[p][e][g] + ldg (r.dt_bias + (size_t)h * D + d + 4 * e + g));
                else
                  l[g] = ld;
                l[g] = in ? l[g] : 0.f;
              }
            *(f4 *)(ls + i * LD + d + 4 * e) = l;
          }
      }
  }
  __syncthreads ();
  for (int it = tid; it < kBlocks * D; it += kPrepThreads)
    {
      const int b = it / D, d = it - b * D;
      float x[16], l = 0.f;
#pragma unroll
      for (int i = 0; i < 16; ++i)
        x[i] = ls[(16 * b + i) * LD + d];
#pragma unroll
      for (int i = 0; i < 16; ++i)
        {
          l += x[i];
          ls[(16 * b + i) * LD + d] = l;
        }
      es[it] = l;
      if (l < -58.f)
        atomicOr (&steep, 1u << b);
    }
  __syncthreads ();

  // (the values of this wave's first columns: on their way while P is formed)
  T vr[kBlocks][4];
  if constexpr (DELTA)
    {
      const int col = 16 * min (wave, r.vdim / 16 - 1) + lo;
#pragma unroll
      for (int b = 0; b < kBlocks; ++b)
#pragma unroll
        for (int e = 0; e < 4; ++e)
          vr[b][e] = ldg ((const T *)r.v + (size_t)(s0 + min (16 * b + hi + e, n - 1)) * r.vs + (size_t)h * r.vdim + col);
    }
  // P, and for the delta rule A, in blocks (bi, bj <= bi), transposed in the registers:
  // a lane holds row lo, columns hi .. hi + 3.  Waves 0 .. 3 take the diagonal and
  // invert it, the others the blocks below it.
  const int DB = D / 16;
  auto block = [&] (int bi, int bj) {
    const int i = 16 * bi + lo;
    f4 sp = { 0.f, 0.f, 0.f, 0.f }, sa = sp;
    if (bi == bj && ((steep >> bi) & 1u))
      // pair by pair
      for (int d = 0; d < D; ++d)
        {
          const float q = qs[i * LD + d], k = ks[i * LD + d], l = ls[i * LD + d];
#pragma unroll
          for (int e = 0; e < 4; ++e)
            {
              const int j = 16 * bj + hi + e;
              const float f = ks[j * LD + d] * power2 (fminf (l - ls[j * LD + d], 0.f));
              sp[e] = __builtin_fmaf (q, f, sp[e]);
              if (DELTA)
                sa[e] = __builtin_fmaf (k, f, sa[e]);
            }
        }
    else
      for (int d0 = hi; d0 < D; d0 += 16)
        {
          const f4 li = *(const f4 *)(ls + i * LD + d0), lj = *(const f4 *)(ls + (16 * bj + lo) * LD + d0);
          const f4 qi = *(const f4 *)(qs + i * LD + d0), kj = *(const f4 *)(ks + (16 * bj + lo) * LD + d0);
          f4 mid = { 0.f, 0.f, 0.f, 0.f };
          if (bj < bi)
            mid = *(const f4 *)(es + bj * D + d0);
          for (int b = bj + 1; b < bi; ++b)
            mid += *(const f4 *)(es + b * D + d0);
          f4 ki = { 0.f, 0.f, 0.f, 0.f };
          if (DELTA)
            ki = *(const f4 *)(ks + i * LD + d0);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            {
              const float fi = power2 (li[e]), x = kj[e] * power2 (mid[e] - lj[e]);
              sp = mfma4 (x, qi[e] * fi, sp);
              if (DELTA)
                sa = mfma4 (x, ki[e] * fi, sa);
            }
        }
    const float bi_ = DELTA ? beta[i] : 0.f;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      {
        const int j = 16 * bj + hi + e;
        sp[e] = j <= i ? sp[e] : 0.f;
        if (DELTA)
          sa[e] = j < i ? sa[e] * bi_ : 0.f;
      }
    stf4 (v.p + ((size_t)(bi * kBlocks + bj) * 64 + lane) * 4, sp);
    if (DELTA)
      *(f4 *)(A + i * kLdA + 16 * bj + hi) = sa;
  };
  if (wave < kBlocks)
    {
      block (wave, wave);
      if constexpr (DELTA)
        {
          // column lo of the inverse (the lane groups do the same)
          __builtin_amdgcn_fence (__ATOMIC_RELEASE, "wavefront");
          __builtin_amdgcn_wave_barrier ();
          const float *Ab = A + 16 * wave * kLdA + 16 * wave;
          float x[16];
          f4 rows[16][4];
#pragma unroll
          for (int i = 1; i < 16; ++i)
#pragma unroll
            for (int j = 0; j < i; j += 4)
              rows[i][j / 4] = *(const f4 *)(Ab + i * kLdA + j);
#pragma unroll
          for (int i = 0; i < 16; ++i)
            {
              float y = i == lo ? 1.f : 0.f;
#pragma unroll
              for (int j = 0; j < i; ++j)
                y = __builtin_fmaf (-rows[i][j / 4][j % 4], x[j], y);
              x[i] = y;
              Ti[(16 * wave + i) * kLdT + lo] = y;
            }
        }
    }
  else if (wave < 6)
    block (wave - 3, 0), block (3, wave - 4);
  else
    block (wave == 6 ? 3 : 2, wave == 6 ? 2 : 1);
  // keys with the decay to the end of the chunk
  for (int it = wave; it < DB * kBlocks; it += kPrepThreads / 64)
    {
      const int b = it % kBlocks, d = it / kBlocks * 16 + lo, j = 16 * b + hi;
      float end = es[b * D + d];
      for (int k = b + 1; k < kBlocks; ++k)
        end += es[k * D + d];
      f4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        o[e] = ks[(j + e) * LD + d] * power2 (end - ls[(j + e) * LD + d]);
      stf4 (v.kt + ((size_t)it * 64 + lane) * 4, o);
    }
  // queries with the decay since its start
  for (int it = wave; it < kBlocks * DB; it += kPrepThreads / 64)
    {
      const int b = it / DB, d = it % DB * 16 + hi, i = 16 * b + lo;
      f4 l = *(const f4 *)(ls + i * LD + d), o = *(const f4 *)(qs + i * LD + d);
      for (int k = 0; k < b; ++k)
        l += *(const f4 *)(es + k * D + d);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        o[e] *= power2 (l[e]);
      stf4 (v.qd + ((size_t)it * 64 + lane) * 4, o);
    }
  for (int d = tid; d < D; d += kPrepThreads)
    {
      float l = 0.f;
      for (int b = 0; b < kBlocks; ++b)
        l += es[b * D + d];
      stg (v.dec + d, power2 (l));
    }
  if constexpr (DELTA)
    {
      __syncthreads ();
      // (1 + A) X = [diag (beta) V | diag (beta) K D], 16 columns of X per wave, block row
      // by block row: X_b = T_b (R_b - sum_{b' < b} A_bb' X_b').  The queries' place in LDS
      // takes W, which leaves it in the other order.
      const int VB = r.vdim / 16;
      for (int g = wave; g < VB + DB; g += kPrepThreads / 64)
        {
          const bool val = g < VB;
          const int col = 16 * (val ? g : g - VB) + lo;
          f4 x[kBlocks];
          if (val && g == wave)
            {
#pragma unroll
              for (int b = 0; b < kBlocks; ++b)
#pragma unroll
                for (int e = 0; e < 4; ++e)
                  x[b][e] = value_of (vr[b][e]);
            }
          else if (val)
            {
#pragma unroll
              for (int b = 0; b < kBlocks; ++b)
#pragma unroll
                for (int e = 0; e < 4; ++e)
                  x[b][e] = load1<T> (r.v, (size_t)(s0 + min (16 * b + hi + e, n - 1)) * r.vs + (size_t)h * r.vdim + col);
            }
          else
            {
              float before = 0.f;
#pragma unroll
              for (int b = 0; b < kBlocks; ++b)
                {
#pragma unroll
                  for (int e = 0; e < 4; ++e)
                    {
                      const int i = 16 * b + hi + e;
                      x[b][e] = ks[i * LD + col] * power2 (ls[i * LD + col] + before);
                    }
                  before += es[b * D + col];
                }
            }
#pragma unroll
          for (int b = 0; b < kBlocks; ++b)
            x[b] *= *(const f4 *)(beta + 16 * b + hi);
#pragma unroll
          for (int b = 0; b < kBlocks; ++b)
            {
              f4 acc = x[b];
#pragma unroll
              for (int k = 0; k < b; ++k)
                {
                  const f4 m = *(const f4 *)(A + (16 * b + lo) * kLdA + 16 * k + hi);
#pragma unroll
                  for (int e = 0; e < 4; ++e)
                    acc = mfma4 (-m[e], x[k][e], acc);
                }
              const f4 m = *(const f4 *)(Ti + (16 * b + lo) * kLdT + hi);
              f4 y = { 0.f, 0.f, 0.f, 0.f };
#pragma unroll
              for (int e = 0; e < 4; ++e)
                y = mfma4 (m[e], acc[e], y);
              x[b] = y;
              if (val)
                stf4 (v.u + ((size_t)(b * VB + g) * 64 + lane) * 4, y);
              else
#pragma unroll
                for (int e = 0; e < 4; ++e)
                  qs[(16 * b + hi + e) * LD + col] = y[e];
            }
        }
      __syncthreads ();
      for (int it = wave; it < kBlocks * DB; it += kPrepThreads / 64)
        stf4 (v.w + ((size_t)it * 64 + lane) * 4, *(const f4 *)(qs + (16 * (it / DB) + lo) * LD + it % DB * 16 + hi));
    }
}

// ---------------------------------------------------------------------------
// chunks: along the state
// ---------------------------------------------------------------------------
// wave w: tokens 16 w .. +15 of a chunk, and blocks w, w + 4 of the state's rows
// (one workgroup per compute unit: the next chunk's operands travel in registers)
template <int DB, bool DELTA, typename T>
__global__ __launch_bounds__ (256) __attribute__ ((amdgpu_waves_per_eu (1, 1))) void
chunk_scan_kernel (const RecurArgs a, const float *ws)
{
  constexpr int KB = (DB + 3) / 4, D = 16 * DB;
  __shared__ f4 ms[DB][64], us[kBlocks][64];
  const vkl_recurrence_args &r = a.r;
  const int h = blockIdx.x % r.H, vb = blockIdx.x / r.H;
  const int lane = threadIdx.x & 63, wave = __builtin_amdgcn_readfirstlane (threadIdx.x >> 6);
  const int lo = lane & 15, hi = 4 * (lane >> 4), col = vb * 16 + lo;
  float *st = r.state + (size_t)h * D * r.vdim + col;
#pragma unroll
  for (int i = 0; i < KB; ++i)
    {
      const int b = wave + 4 * i;
      if (b >= DB)
        continue;
      f4 m;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        m[e] = a.fresh ? 0.f : ldg (st + (size_t)(16 * b + hi + e) * r.vdim);
      ms[b][lane] = m;
    }
  const int chunks = (a.S + kChunk - 1) / kChunk;
  const size_t per = chunk_floats (D, r.vdim);
  struct Operands
  {
    f4 w[DELTA ? DB : 1], q[DB], p[kBlocks], k[KB][kBlocks], u, dec[KB];
    T v[4]; // u, as the values lie (decaying sums)
  };
  auto fetch = [&] (int c, Operands &o) {
    const float *base = ws + ((size_t)c * r.H + h) * per;
    const ChunkView v = chunk_view (const_cast<float *> (base), D, r.vdim);
    auto at = [&] (const float *m, int blk) { return ldf4 (m + ((size_t)blk * 64 + lane) * 4); };
#pragma unroll
    for (int b = 0; b < DB; ++b)
      {
        o.q[b] = at (v.qd, wave * DB + b);
        if constexpr (DELTA)
          o.w[b] = at (v.w, wave * DB + b);
      }
#pragma unroll
    for (int b = 0; b < kBlocks; ++b)
      // (blocks right of the diagonal do not exist)
      o.p[b] = at (v.p, wave * kBlocks + min (b, wave));
#pragma unroll
    for (int i = 0; i < KB; ++i)
      {
        const int b = min (wave + 4 * i, DB - 1);
        o.dec[i] = ldf4 (v.dec + 16 * b + hi);
#pragma unroll
        for (int j = 0; j < kBlocks; ++j)
          o.k[i][j] = at (v.kt, b * kBlocks + j);
      }
    if constexpr (DELTA)
      o.u = at (v.u, wave * (r.vdim / 16) + vb);
    else
#pragma unroll
      for (int e = 0; e < 4; ++e)
        {
          // (tokens past the end have keys of zero)
          const int s = min (c * kChunk + 16 * wave + hi + e, a.S - 1);
          o.v[e] = ldg ((const T *)r.v + (size_t)s * r.vs + (size_t)h * r.vdim + col);
        }
  };
  auto chunk = [&] (int c, const Operands &o) {
    f4 m[DB], u[kBlocks];
#pragma unroll
    for (int b = 0; b < DB; ++b)
      m[b] = ms[b][lane];
    __builtin_amdgcn_sched_barrier (0);
    f4 acc = { 0.f, 0.f, 0.f, 0.f }, sub = acc, acc2 = acc, sub2 = acc;
    if constexpr (!DELTA)
      {
#pragma unroll
        for (int e = 0; e < 4; ++e)
          u[0][e] = value_of (o.v[e]);
        us[wave][lane] = u[0];
      }
    else
      {
#pragma unroll
        for (int b = 0; b < DB; ++b)
#pragma unroll
          for (int e = 0; e < 4; e += 2)
            {
              sub = mfma4 (o.w[b][e], m[b][e], sub);
              sub2 = mfma4 (o.w[b][e + 1], m[b][e + 1], sub2);
            }
        us[wave][lane] = o.u - (sub + sub2);
      }
    // (what needs u of the other waves comes after this product)
#pragma unroll
    for (int b = 0; b < DB; ++b)
#pragma unroll
      for (int e = 0; e < 4; e += 2)
        {
          acc = mfma4 (o.q[b][e], m[b][e], acc);
          acc2 = mfma4 (o.q[b][e + 1], m[b][e + 1], acc2);
        }
    __syncthreads ();
#pragma unroll
    for (int b = 0; b < kBlocks; ++b)
      u[b] = us[b][lane];
#pragma unroll
    for (int i = 0; i < KB; ++i)
      m[i] = o.dec[i] * ms[min (wave + 4 * i, DB - 1)][lane];
    __builtin_amdgcn_sched_barrier (0);
#pragma unroll
    for (int j = 0; j < kBlocks; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e)
#pragma unroll
        for (int i = 0; i < KB; ++i)
          m[i] = mfma4 (o.k[i][j][e], u[j][e], m[i]);
#pragma unroll
    for (int i = 0; i < KB; ++i)
      if (wave + 4 * i < DB)
        ms[wave + 4 * i][lane] = m[i];
#pragma unroll
    for (int b = 0; b < kBlocks; ++b)
      if (b <= wave)
#pragma unroll
        for (int e = 0; e < 4; e += 2)
          {
            acc = mfma4 (o.p[b][e], u[b][e], acc);
            acc2 = mfma4 (o.p[b][e + 1], u[b][e + 1], acc2);
          }
    acc += acc2;
    float *out = r.out + (size_t)(c * kChunk + 16 * wave + hi) * r.os + (size_t)h * r.vdim + col;
    if (c * kChunk + kChunk <= a.S)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        stg (out + (size_t)e * r.os, acc[e]);
    else
#pragma unroll
      for (int e = 0; e < 4; ++e)
        if (c * kChunk + 16 * wave + hi + e < a.S)
          stg (out + (size_t)e * r.os, acc[e]);
    __syncthreads ();
  };
  Operands x, y;
  fetch (0, x);
  __syncthreads ();
  for (int c = 0; c < chunks; c += 2)
    {
      fetch (min (c + 1, chunks - 1), y);
      __builtin_amdgcn_sched_barrier (0);
      chunk (c, x);
      if (c + 1 >= chunks)
        break;
      fetch (min (c + 2, chunks - 1), x);
      __builtin_amdgcn_sched_barrier (0);
      chunk (c + 1, y);
    }
#pragma unroll
  for (int i = 0; i < KB; ++i)
    {
      const int b = wave + 4 * i;
      if (b >= DB)
        continue;
      const f4 m = ms[b][lane];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        stg (st + (size_t)(16 * b + hi + e) * r.vdim, m[e]);
    }
}

template <bool DELTA, typename T>
int
launch_tokens (const RecurArgs &a, hipStream_t s)
{
  const dim3 grid ((unsigned)(a.r.H * (a.r.vdim / 16))), block (64);
  switch (a.r.dim / 32)
    {
    case 1: recur_tokens_kernel<2, DELTA, T><<<grid, block, 0, s>>> (a); break;
    case 2: recur_tokens_kernel<4, DELTA, T><<<grid, block, 0, s>>> (a); break;
    case 3: recur_tokens_kernel<6, DELTA, T><<<grid, block, 0, s>>> (a); break;
    case 4: recur_tokens_kernel<8, DELTA, T><<<grid, block, 0, s>>> (a); break;
    case 5: recur_tokens_kernel<10, DELTA, T><<<grid, block, 0, s>>> (a); break;
    case 6: recur_tokens_kernel<12, DELTA, T><<<grid, block, 0, s>>> (a); break;
    case 7: recur_tokens_kernel<14, DELTA, T><<<grid, block, 0, s>>> (a); break;
    default: recur_tokens_kernel<16, DELTA, T><<<grid, block, 0, s>>> (a); break;
    }
  return (int)hipGetLastError ();
}

template <bool DELTA, typename T>
int
launch_chunks (const RecurArgs &a, float *ws, hipStream_t s)
{
  static LdsLimit limit;
  const size_t lds = prep_lds_bytes (a.r.dim);
  const auto prep = chunk_prep_kernel<DELTA, T>;
  if (int e = limit.raise ((const void *)prep, lds))
    return e;
  const int chunks = (a.S + kChunk - 1) / kChunk;
  prep<<<dim3 ((unsigned)(chunks * a.r.H)), dim3 (kPrepThreads), lds, s>>> (a, ws);
  if (hipError_t e = hipGetLastError ())
    return (int)e;
  const dim3 grid ((unsigned)(a.r.H * (a.r.vdim / 16))), block (256);
  switch (a.r.dim / 32)
    {
    case 1: chunk_scan_kernel<2, DELTA, T><<<grid, block, 0, s>>> (a, ws); break;
    case 2: chunk_scan_kernel<4, DELTA, T><<<grid, block, 0, s>>> (a, ws); break;
    case 3: chunk_scan_kernel<6, DELTA, T><<<grid, block, 0, s>>> (a, ws); break;
    default: chunk_scan_kernel<8, DELTA, T><<<grid, block, 0, s>>> (a, ws); break;
    }
  return (int)hipGetLastError ();
}

// ---------------------------------------------------------------------------
// norm and gate of what a recurrence puts out
// ---------------------------------------------------------------------------
struct GatedNormArgs
{
  const float *x;
  size_t xs;
  int groups, gw, n;
  const float *w;
  float eps;
  const void *gate;
  size_t gs;
  int type;
  void *out;
  size_t os;
  int S;
};

// WIDE: a workgroup per row that is one group; else a wave per group
template <bool WIDE, typename T>
__global__ __launch_bounds__ (256) void
gated_norm_kernel (const GatedNormArgs a)
{
  __shared__ float red[8];
  constexpr int N = WIDE ? 256 : 64;
  const int t = WIDE ? threadIdx.x : (threadIdx.x & 63);
  const size_t it = WIDE ? blockIdx.x : (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (!WIDE && it >= (size_t)a.S * a.groups)
    return;
  const size_t s = it / a.groups, g0 = (it - s * a.groups) * (size_t)a.gw;
  const float *x = a.x + s * a.xs + g0;
  float ss = 0.f;
  for (int c = t * 4; c < a.gw; c += N * 4)
    {
      const f4 v = ldf4 (x + c);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        ss = __builtin_fmaf (v[e], v[e], ss);
    }
  ss = WIDE ? group_sum (ss, red) : wave_sum (ss);
  const float alpha = 1.0f / sqrtf (ss / (float)a.n + a.eps);
  for (int c = t * 4; c < a.gw; c += N * 4)
    {
      const f4 v = ldf4 (x + c), w = ldf4 (a.w + c), g = load4<T> (a.gate, s * a.gs + g0 + c);
      f4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        o[e] = v[e] * alpha * w[e] * quick_sigmoid (g[e]);
      store4<T> (a.out, s * a.os + g0 + c, o);
    }
}

// The same per head with gates x W^T of low rank: a wave takes 16 tokens of a head, a
// workgroup 64.
struct LowRankNormArgs
{
  const float *x;
  size_t xs;
  int H, vdim, n;
  const float *w;
  float eps;
  const void *g1;
  size_t gs;
  const uint16_t *g2;
  int r, type, S;
  void *out;
  size_t os;
};

template <int VB, typename T>
__global__ __launch_bounds__ (256) void
low_rank_norm_kernel (const LowRankNormArgs a)
{
  const int lane = threadIdx.x & 63, lo = lane & 15, q = lane >> 4;
  const int h = blockIdx.x % a.H, s0 = (blockIdx.x / a.H) * 64 + (threadIdx.x >> 6) * 16;
  if (s0 >= a.S)
    return;
  // Columns are dealt to the result blocks so that a lane holds eight neighbours of token
  // lo: row m of block b is column 32 (b / 2) + 8 (m / 4) + 4 (b % 2) + m % 4.
  const size_t s = (size_t)min (s0 + lo, a.S - 1);
  const float *x = a.x + s * a.xs + (size_t)h * a.vdim + 8 * q;
  f4 o[VB], g[VB];
  float ss = 0.f;
#pragma unroll
  for (int b = 0; b < VB; ++b)
    {
      g[b] = f4{ 0.f, 0.f, 0.f, 0.f };
      o[b] = ldf4 (x + 32 * (b / 2) + 4 * (b % 2));
    }
  const uint16_t *w = a.g2 + ((size_t)h * a.vdim + 8 * (lo / 4) + lo % 4) * a.r;
  auto row = [&] (int b) { return (size_t)(32 * (b / 2) + 4 * (b % 2)) * a.r; };
  if constexpr (sizeof (T) == 2)
    for (int k0 = 0; k0 < a.r; k0 += 64)
      {
        bf8 v[2], y[2][VB];
#pragma unroll
        for (int u = 0; u < 2; ++u)
          {
            const int k = k0 + 32 * u + 8 * q;
            v[u] = __builtin_bit_cast (bf8, ldg4 ((const uint16_t *)a.g1 + s * a.gs + k));
#pragma unroll
            for (int b = 0; b < VB; ++b)
              y[u][b] = __builtin_bit_cast (bf8, ldg4 (w + row (b) + k));
          }
#pragma unroll
        for (int u = 0; u < 2; ++u)
#pragma unroll
          for (int b = 0; b < VB; ++b)
            g[b] = __builtin_amdgcn_mfma_f32_16x16x32_bf16 (y[u][b], v[u], g[b], 0, 0, 0);
      }
  else
    for (int k = 4 * q; k < a.r; k += 16)
      {
        const f4 v = ldf4 ((const float *)a.g1 + s * a.gs + k);
#pragma unroll
        for (int b = 0; b < VB; ++b)
          {
            const f4 y = load4<uint16_t> (w, row (b) + k);
#pragma unroll
            for (int e = 0; e < 4; ++e)
              g[b] = mfma4 (y[e], v[e], g[b]);
          }
      }
#pragma unroll
  for (int b = 0; b < VB; ++b)
#pragma unroll
    for (int e = 0; e < 4; ++e)
      ss = __builtin_fmaf (o[b][e], o[b][e], ss);
  const float alpha = 1.0f / sqrtf (rows_sum (ss) / (float)a.n + a.eps);
  if (s0 + lo >= a.S)
    return;
#pragma unroll
  for (int b = 0; b < VB; b += 2)
    {
      float y[8];
#pragma unroll
      for (int i = 0; i < 8; ++i)
        {
          const f4 &v = o[b + i / 4], &z = g[b + i / 4];
          y[i] = v[i % 4] * alpha * ldg (a.w + 16 * b + 8 * q + i) * quick_sigmoid (z[i % 4]);
        }
      store8<T> (a.out, s * a.os + (size_t)h * a.vdim + 16 * b + 8 * q, y);
    }
}

// ---------------------------------------------------------------------------
// one token
// ---------------------------------------------------------------------------
constexpr int kStepThreads = 512, kStepWaves = 8;

// y[i] = w[i, :] x for the rows i of one head.  Rows of 64 or 128 values are dealt out
// in 16-byte chunks, so that the first of them are requested long before x is
// there; other lengths take eight lanes per row.
constexpr int kAhead = 4; // chunks of a thread

struct HeadRows
{
  const uint16_t *w;
  int rows, K;
  uint4 ahead[kAhead];

  __device__ __forceinline__ bool
  dealt () const
  {
    return K == 64 || K == 128;
  }
  __device__ __forceinline__ int
  shift () const
  {
    return K == 64 ? 3 : 4;
  }
  __device__ __forceinline__ void
  request ()
  {
    if (dealt ())
#pragma unroll
      for (int u = 0; u < kAhead; ++u)
        ahead[u] = ldg4 (w + (size_t)min ((int)threadIdx.x + u * kStepThreads, (rows << shift ()) - 1) * 8);
  }
  static __device__ __forceinline__ float
  dot8 (const uint4 v, const float *x)
  {
    float f[8], acc = 0.f;
    widen8 (v, f);
    const f4 x0 = *(const f4 *)x, x1 = *(const f4 *)(x + 4);
#pragma unroll
    for (int e = 0; e < 4; ++e)
      acc = __builtin_fmaf (f[e], x0[e], acc), acc = __builtin_fmaf (f[4 + e], x1[e], acc);
    return acc;
  }
  template <typename F>
  __device__ __forceinline__ void
  run (const float *x, F put) const
  {
    if (dealt ())
      {
        const int sh = shift (), all = rows << sh, mask = (1 << sh) - 1;
        auto part = [&] (int c, const uint4 v) {
          float y = row_sum<8> (dot8 (v, x + (c & mask) * 8));
          if (sh == 4)
            y += dpp_get<0x140> (y);
          if ((c & mask) == 0 && c < all)
            put (c >> sh, y);
        };
#pragma unroll
        for (int u = 0; u < kAhead; ++u)
          part ((int)threadIdx.x + u * kStepThreads, ahead[u]);
#pragma unroll 1
        for (int c = (int)threadIdx.x + kAhead * kStepThreads; c < all; c += kStepThreads)
          part (c, ldg4 (w + (size_t)c * 8));
        return;
      }
    const int sub = threadIdx.x & 7;
#pragma unroll 1
    for (int i0 = 0; i0 < rows; i0 += kStepThreads / 8)
      {
        const int i = i0 + (int)(threadIdx.x >> 3), ic = min (i, rows - 1);
        float acc = 0.f;
#pragma unroll 1
        for (int k = sub * 8; k < K; k += 64)
          acc += dot8 (ldg4 (w + (size_t)ic * K + k), x + k);
        acc = row_sum<8> (acc);
        if (sub == 0 && i < rows)
          put (i, acc);
      }
  }
};

// DJ: dim / 16.  A wave takes blocks of 16 value columns in turn.  What the launch
// reads is requested at its start, in one round trip.
template <int DJ, bool DELTA>
__global__ __launch_bounds__ (kStepThreads) void
recur_step_kernel (const RecurStepArgs a)
{
  constexpr int D = 16 * DJ, MV = 256, TAPS = 4; // taps requested ahead
  __shared__ __align__ (16) float q[D], k[D], g[D], v[MV], o[MV], z[MV], bias[D];
  extern __shared__ __align__ (16) float lds_step[]; // a1 | g1
  __shared__ float red[kStepWaves];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lo = lane & 15, hi = 4 * (lane >> 4);
  const uint32_t pos = a.pos.get ();
  float *st = a.state + (size_t)h * D * a.vdim;
  const uint32_t cell = (uint32_t)(hi * a.vdim + lo); // a lane's place in a block of the state
  f4 m[DJ];
  auto fetch = [&] (int vb) {
#pragma unroll
    for (int j = 0; j < DJ; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        m[j][e] = ldg (st + ((16 * j + e) * a.vdim + 16 * vb) + cell);
  };
  const int G = a.H / a.rep, hq = h / a.rep;
  const int nqk = G * D, n = 2 * nqk + a.H * a.vdim;
  // q, k, v of the head: a channel per thread, where there are more than threads in turns
  auto channel = [&] (int c) {
    return c < D ? hq * D + c : c < 2 * D ? nqk + hq * D + c - D : 2 * nqk + h * a.vdim + c - 2 * D;
  };
  auto request = [&] (int c, float &now, float (&w)[TAPS], float (&x)[TAPS]) {
    const int ch = channel (min (c, 2 * D + a.vdim - 1));
    now = ldg (a.qkv + ch);
    if (DELTA)
#pragma unroll
      for (int b = 0; b < TAPS; ++b)
        {
          w[b] = ldg (a.conv + (size_t)max (a.taps - 1 - b, 0) * n + ch);
          x[b] = ldg (a.ring + (size_t)((pos - (uint32_t)min (b, (int)pos)) % (uint32_t)a.taps) * n + ch);
        }
  };
  auto finish = [&] (int c, float now, const float (&w)[TAPS], const float (&x)[TAPS]) {
    float y = now;
    if (DELTA)
      {
        const int ch = channel (c);
        y = w[0] * now;
#pragma unroll
        for (int b = 1; b < TAPS; ++b)
          if (b < a.taps && (uint32_t)b <= pos)
            y = __builtin_fmaf (w[b], x[b], y);
#pragma unroll 1
        for (int b = TAPS; b < a.taps && (uint32_t)b <= pos; ++b)
          y = __builtin_fmaf (ldg (a.conv + (size_t)(a.taps - 1 - b) * n + ch),
                              ldg (a.ring + (size_t)((pos - (uint32_t)b) % (uint32_t)a.taps) * n + ch), y);
        y = silu (y);
        // (the row of this position is none that the step uses; heads that share a
        // query and key leave it to the first of them)
        if (c >= 2 * D || h % a.rep == 0)
          stg (a.ring + (size_t)(pos % (uint32_t)a.taps) * n + ch, now);
      }
    if (c < D)
      q[c] = y;
    else if (c < 2 * D)
      k[c - D] = y;
    else
      v[c - 2 * D] = y;
  };
  float now, cw[TAPS], cx[TAPS];
  request (tid, now, cw, cx);
  const int blocks = a.vdim / 16;
  float a1v = 0.f, g1v = 0.f, bv = 0.f, rate = 0.f, bias_v = 0.f, gn = 0.f;
  HeadRows decays, gates;
  if constexpr (DELTA)
    {
      a1v = ldg (a.a1 + min (tid, a.r_a - 1)), g1v = ldg (a.g1 + min (tid, a.r_g - 1));
      bv = ldg (a.b + h), rate = ldg (a.rate + h);
      bias_v = ldg (a.dt_bias + (size_t)h * D + min (tid, D - 1));
      gn = ldg (a.gnorm + min (tid, a.vdim - 1));
      decays.w = a.w_a2 + (size_t)h * D * a.r_a, decays.rows = D, decays.K = a.r_a;
      gates.w = a.w_g2 + (size_t)h * a.vdim * a.r_g, gates.rows = a.vdim, gates.K = a.r_g;
      decays.request (), gates.request ();
    }
  fetch (min (wave, blocks - 1));
  __builtin_amdgcn_sched_barrier (0);
  if (tid < 2 * D + a.vdim)
    finish (tid, now, cw, cx);
#pragma unroll 1
  for (int c = tid + kStepThreads; c < 2 * D + a.vdim; c += kStepThreads)
    {
      request (c, now, cw, cx);
      finish (c, now, cw, cx);
    }
  float decay = 1.f, beta = 0.f, fq = a.qscale, fk = 1.f;
  if (DELTA)
    {
      float *a1 = lds_step, *g1 = lds_step + a.r_a;
      if (tid < a.r_a)
        a1[tid] = a1v;
      if (tid < a.r_g)
        g1[tid] = g1v;
      if (tid < D)
        bias[tid] = bias_v;
#pragma unroll 1
      for (int i = tid + kStepThreads; i < a.r_a; i += kStepThreads)
        a1[i] = ldg (a.a1 + i);
#pragma unroll 1
      for (int i = tid + kStepThreads; i < a.r_g; i += kStepThreads)
        g1[i] = ldg (a.g1 + i);
      beta = sigmoid (bv);
      __syncthreads ();
      decays.run (a1, [&] (int i, float y) { g[i] = expf (log_decay_of (rate, y + bias[i])); });
      gates.run (g1, [&] (int i, float y) { z[i] = sigmoid (y); });
      float qq = 0.f, kk = 0.f;
      for (int d = lane; d < D; d += 64)
        qq = __builtin_fmaf (q[d], q[d], qq), kk = __builtin_fmaf (k[d], k[d], kk);
      fq = a.qscale / sqrtf (wave_sum (qq) + a.unit_eps), fk = 1.0f / sqrtf (wave_sum (kk) + a.unit_eps);
    }
  else
    decay = expf (fmaxf (ldg (a.log_decay + h), -1.0e4f));
  __syncthreads ();
  for (int vb = wave; vb < blocks; vb += kStepWaves)
    {
      if (vb != wave)
        fetch (vb);
      const int col = 16 * vb + lo;
      float u = v[col], out = 0.f;
      if (DELTA)
        {
          float mk = 0.f;
#pragma unroll
          for (int j = 0; j < DJ; ++j)
            {
              const f4 gj = *(const f4 *)(g + 16 * j + hi), kj = *(const f4 *)(k + 16 * j + hi);
#pragma unroll
              for (int e = 0; e < 4; ++e)
                {
                  m[j][e] = pos ? m[j][e] * gj[e] : 0.f;
                  mk = __builtin_fmaf (m[j][e], kj[e] * fk, mk);
                }
            }
          u = beta * (u - rows_sum (mk));
        }
#pragma unroll
      for (int j = 0; j < DJ; ++j)
        {
          const f4 kj = *(const f4 *)(k + 16 * j + hi), qj = *(const f4 *)(q + 16 * j + hi);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            {
              if (!DELTA)
                m[j][e] = pos ? m[j][e] * decay : 0.f;
              m[j][e] = __builtin_fmaf (kj[e] * fk, u, m[j][e]);
              out = __builtin_fmaf (m[j][e], qj[e], out);
              stg (st + ((16 * j + e) * a.vdim + 16 * vb) + cell, m[j][e]);
            }
        }
      out = rows_sum (out) * fq;
      if (lane < 16)
        {
          if (DELTA)
            o[col] = out;
          else
            stg (a.out + (size_t)h * a.vdim + col, out);
        }
    }
  if (!DELTA)
    {
      if (h == 0 && tid < a.out_pad)
        stg (a.out + (size_t)a.H * a.vdim + tid, 0.f);
      return;
    }
  __syncthreads ();
  float ss = 0.f;
  for (int c = tid; c < a.vdim; c += kStepThreads)
    ss = __builtin_fmaf (o[c], o[c], ss);
  const float alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.vn + a.eps);
  if (tid < a.vdim)
    stg (a.out + (size_t)h * a.vdim + tid, o[tid] * alpha * gn * z[tid]);
}

template <bool DELTA>
int
launch_step (const RecurStepArgs &a, hipStream_t s)
{
  const dim3 grid ((unsigned)a.H), block (kStepThreads);
  const size_t lds = DELTA ? (size_t)(a.r_a + a.r_g) * sizeof (float) : 0;
  if (lds > (size_t)48 << 10)
    return (int)hipErrorInvalidValue;
  switch (a.dim / 32)
    {
    case 1: recur_step_kernel<2, DELTA><<<grid, block, lds, s>>> (a); break;
    case 2: recur_step_kernel<4, DELTA><<<grid, block, lds, s>>> (a); break;
    case 3: recur_step_kernel<6, DELTA><<<grid, block, lds, s>>> (a); break;
    case 4: recur_step_kernel<8, DELTA><<<grid, block, lds, s>>> (a); break;
    case 5: recur_step_kernel<10, DELTA><<<grid, block, lds, s>>> (a); break;
    case 6: recur_step_kernel<12, DELTA><<<grid, block, lds, s>>> (a); break;
    case 7: recur_step_kernel<14, DELTA><<<grid, block, lds, s>>> (a); break;
    default: recur_step_kernel<16, DELTA><<<grid, block, lds, s>>> (a); break;
    }
  return (int)hipGetLastError ();
}

// below this many tokens the walk along the tokens is shorter
constexpr int kChunkMin = 24;
} // namespace

bool
recur_supported (int H, int rep, int dim, int vdim)
{
  return H > 0 && rep > 0 && (H % rep) == 0 && dim > 0 && (dim % 32) == 0 && dim <= 256 && vdim > 0 && (vdim % 32) == 0
         && vdim <= 256;
}

int
delta_step_launch (const RecurStepArgs &a, hipStream_t s)
{
  return launch_step<true> (a, s);
}

int
decay_step_launch (const RecurStepArgs &a, hipStream_t s)
{
  return launch_step<false> (a, s);
}
} // namespace vkl

using namespace vkl;

extern "C" int
vkl_short_conv_silu (const void *x, int type, size_t xs, const float *w, int n, int taps, float *ring, uint32_t pos0,
                     int S, void *out, size_t os, void *stream)
{
  VKL_CHECK_ARG (x && w && ring && out && x != out && n > 0 && (n % 8) == 0 && taps >= 1 && taps <= 16 && S > 0);
  VKL_CHECK_ARG ((type == VKL_TYPE_F32 || type == VKL_TYPE_BF16) && xs >= (size_t)n && os >= (size_t)n && (xs % 8) == 0
                 && (os % 8) == 0);
  VKL_CHECK_ARG (((uintptr_t)x % 16) == 0 && ((uintptr_t)out % 16) == 0 && ((uintptr_t)w % 16) == 0
                 && ((uintptr_t)ring % 16) == 0);
  const ConvArgs a = { x, type, xs, w, n, taps, ring, pos0, S, out, os };
  hipStream_t s = (hipStream_t)stream;
  const size_t items = (size_t)((S + kConvRun - 1) / kConvRun) * (n / 8), keep = (size_t)std::min (S, taps) * n;
  const dim3 grid ((unsigned)((items + 255) / 256)), block (256);
  with_format (type, [&] (auto t) {
    typedef decltype (t) T;
    switch (taps)
      {
      case 2: short_conv_kernel<2, T><<<grid, block, 0, s>>> (a); break;
      case 3: short_conv_kernel<3, T><<<grid, block, 0, s>>> (a); break;
      case 4: short_conv_kernel<4, T><<<grid, block, 0, s>>> (a); break;
      default: short_conv_kernel<0, T><<<grid, block, 0, s>>> (a); break;
      }
    return 0;
  });
  short_conv_keep_kernel<<<dim3 ((unsigned)((keep + 255) / 256)), dim3 (256), 0, s>>> (a);
  return vkl_launch_status ();
}

extern "C" size_t
vkl_recurrence_scratch_bytes (const vkl_recurrence_args *a, int S)
{
  if (!a || S <= 0 || !recur_supported (a->H, a->rep, a->dim, a->vdim) || a->dim > 128)
    return 0;
  return (size_t)((S + kChunk - 1) / kChunk) * a->H * chunk_floats (a->dim, a->vdim) * sizeof (float);
}

extern "C" int
vkl_recurrence_chunked (const vkl_recurrence_args *a, int S)
{
  return a && S >= kChunkMin && recur_supported (a->H, a->rep, a->dim, a->vdim) && a->dim <= 128;
}

extern "C" int
vkl_recurrence (const vkl_recurrence_args *r, int S, uint32_t pos0, int form, void *scratch, size_t scratch_bytes,
                void *stream)
{
  VKL_CHECK_ARG (r && S > 0 && recur_supported (r->H, r->rep, r->dim, r->vdim));
  const size_t nqk = (size_t)(r->H / r->rep) * r->dim, nv = (size_t)r->H * r->vdim;
  VKL_CHECK_ARG (r->q && r->k && r->v && r->state && r->out && r->qs >= nqk && r->ks >= nqk && r->vs >= nv && r->os >= nv);
  VKL_CHECK_ARG ((r->type == VKL_TYPE_F32 || r->type == VKL_TYPE_BF16) && (r->qs % 8) == 0 && (r->ks % 8) == 0
                 && ((uintptr_t)r->q % 16) == 0 && ((uintptr_t)r->k % 16) == 0);
  const bool delta = r->b != nullptr;
  if (delta)
    {
      VKL_CHECK_ARG (r->dt_bias && r->rate && (r->z || r->a1) && ((uintptr_t)r->dt_bias % 16) == 0 && r->bs >= (size_t)r->H);
      VKL_CHECK_ARG (!r->z || (r->zs >= (size_t)r->H * r->dim && (r->zs % 4) == 0 && ((uintptr_t)r->z % 16) == 0));
      VKL_CHECK_ARG (!r->a1 || (r->w_a2 && r->r_a > 0 && (r->r_a % 64) == 0 && r->as >= (size_t)r->r_a && (r->as % 8) == 0
                                && ((uintptr_t)r->a1 % 16) == 0 && ((uintptr_t)r->w_a2 % 16) == 0));
    }
  else
    VKL_CHECK_ARG (r->log_decay);
  VKL_CHECK_ARG (form >= VKL_RECUR_AUTO && form <= VKL_RECUR_CHUNKS && (form != VKL_RECUR_CHUNKS || r->dim <= 128));
  hipStream_t s = (hipStream_t)stream;
  RecurArgs a = { *r, S, pos0 == 0 };
  const size_t one = (size_t)r->H * chunk_floats (r->dim, r->vdim) * sizeof (float);
  if (form == VKL_RECUR_TOKENS || (form == VKL_RECUR_AUTO && !vkl_recurrence_chunked (r, S)))
    VKL_CHECK_ARG (!delta || r->z);
  if (form == VKL_RECUR_TOKENS || (form == VKL_RECUR_AUTO && !vkl_recurrence_chunked (r, S)))
    return with_format (r->type, [&] (auto t) {
      return delta ? launch_tokens<true, decltype (t)> (a, s) : launch_tokens<false, decltype (t)> (a, s);
    });
  VKL_CHECK_ARG (scratch && scratch_bytes >= one && ((uintptr_t)scratch % 16) == 0 && (r->vs % 8) == 0);
  const int piece = (int)std::min<size_t> (scratch_bytes / one, (size_t)1 << 20) * kChunk;
  const size_t es = r->type == VKL_TYPE_F32 ? 4 : 2;
  for (int at = 0; at < S; at += piece)
    {
      RecurArgs p = a;
      p.S = std::min (piece, S - at);
      p.fresh = a.fresh && at == 0;
      p.r.q = (const uint8_t *)r->q + (size_t)at * r->qs * es;
      p.r.k = (const uint8_t *)r->k + (size_t)at * r->ks * es;
      p.r.v = (const uint8_t *)r->v + (size_t)at * r->vs * es;
      p.r.out = r->out + (size_t)at * r->os;
      if (delta)
        p.r.b = r->b + (size_t)at * r->bs;
      if (r->z)
        p.r.z = r->z + (size_t)at * r->zs;
      if (r->a1)
        p.r.a1 = (const uint8_t *)r->a1 + (size_t)at * r->as * es;
      if (int e = with_format (r->type, [&] (auto t) {
            return delta ? launch_chunks<true, decltype (t)> (p, (float *)scratch, s)
                         : launch_chunks<false, decltype (t)> (p, (float *)scratch, s);
          }))
        return e;
    }
  return 0;
}

extern "C" int
vkl_low_rank_gated_norm (const float *x, size_t xs, int H, int vdim, int n, const float *w, float eps, const void *g1,
                         size_t gs, const void *g2, int r, int type, int S, void *out, size_t os, void *stream)
{
  VKL_CHECK_ARG (x && w && g1 && g2 && out && H > 0 && vdim > 0 && (vdim % 32) == 0 && vdim <= 256 && n > 0 && n <= vdim);
  VKL_CHECK_ARG (S > 0 && r > 0 && (r % 64) == 0 && gs >= (size_t)r && (gs % 8) == 0 && xs >= (size_t)H * vdim
                 && os >= (size_t)H * vdim);
  VKL_CHECK_ARG ((type == VKL_TYPE_F32 || type == VKL_TYPE_BF16) && ((uintptr_t)g1 % 16) == 0 && ((uintptr_t)g2 % 16) == 0
                 && ((uintptr_t)x % 16) == 0 && ((uintptr_t)w % 16) == 0 && ((uintptr_t)out % 16) == 0 && (xs % 4) == 0
                 && (os % 8) == 0);
  const LowRankNormArgs a = { x, xs, H, vdim, n, w, eps, g1, gs, (const uint16_t *)g2, r, type, S, out, os };
  const dim3 grid ((unsigned)((S + 63) / 64 * H)), block (256);
  hipStream_t s = (hipStream_t)stream;
  with_format (type, [&] (auto t) {
    typedef decltype (t) T;
    switch (vdim / 32)
      {
      case 1: low_rank_norm_kernel<2, T><<<grid, block, 0, s>>> (a); break;
      case 2: low_rank_norm_kernel<4, T><<<grid, block, 0, s>>> (a); break;
      case 3: low_rank_norm_kernel<6, T><<<grid, block, 0, s>>> (a); break;
      case 4: low_rank_norm_kernel<8, T><<<grid, block, 0, s>>> (a); break;
      case 5: low_rank_norm_kernel<10, T><<<grid, block, 0, s>>> (a); break;
      case 6: low_rank_norm_kernel<12, T><<<grid, block, 0, s>>> (a); break;
      case 7: low_rank_norm_kernel<14, T><<<grid, block, 0, s>>> (a); break;
      default: low_rank_norm_kernel<16, T><<<grid, block, 0, s>>> (a); break;
      }
    return 0;
  });
  return vkl_launch_status ();
}

extern "C" int
vkl_gated_norm (const float *x, size_t xs, int groups, int gw, int n, const float *w, float eps, const void *gate,
                size_t gs, int type, int S, void *out, size_t os, void *stream)
{
  VKL_CHECK_ARG (x && w && gate && out && groups > 0 && gw > 0 && (gw % 4) == 0 && n > 0 && n <= gw && S > 0);
  const size_t need = (size_t)groups * gw;
  VKL_CHECK_ARG (xs >= need && gs >= need && os >= need && (xs % 4) == 0 && (gs % 4) == 0 && (os % 4) == 0);
  VKL_CHECK_ARG ((type == VKL_TYPE_F32 || type == VKL_TYPE_BF16) && ((uintptr_t)x % 16) == 0 && ((uintptr_t)w % 16) == 0
                 && ((uintptr_t)gate % 16) == 0 && ((uintptr_t)out % 16) == 0);
  const GatedNormArgs a = { x, xs, groups, gw, n, w, eps, gate, gs, type, out, os, S };
  hipStream_t s = (hipStream_t)stream;
  with_format (type, [&] (auto t) {
    typedef decltype (t) T;
    if (groups == 1)
      gated_norm_kernel<true, T><<<dim3 ((unsigned)S), dim3 (256), 0, s>>> (a);
    else
      gated_norm_kernel<false, T><<<dim3 ((unsigned)(((size_t)S * groups + 3) / 4)), dim3 (256), 0, s>>> (a);
    return 0;
  });
  return vkl_launch_status ();
}
