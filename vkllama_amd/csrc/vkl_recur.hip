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
// the block's start as long as the block decays by less than e^-40, and formed
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

__device__ __forceinline__ f4
load4 (const void *p, int type, size_t i)
{
  if (type == VKL_TYPE_F32)
    return ldf4 ((const float *)p + i);
  const unsigned long long w = ldg ((const unsigned long long *)((const uint16_t *)p + i));
  const uint32_t lo = (uint32_t)w, hi = (uint32_t)(w >> 32);
  return f4{ __uint_as_float (lo << 16), __uint_as_float (lo & 0xffff0000u), __uint_as_float (hi << 16),
             __uint_as_float (hi & 0xffff0000u) };
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

// eight channels of one token per thread
__global__ __launch_bounds__ (256) void
short_conv_kernel (const ConvArgs a)
{
  const int n8 = a.n / 8;
  const size_t it = (size_t)blockIdx.x * 256 + threadIdx.x;
  if (it >= (size_t)a.S * n8)
    return;
  const int s = (int)(it / n8), c = (int)(it - (size_t)s * n8) * 8;
  f4 lo = { 0.f, 0.f, 0.f, 0.f }, hi = lo;
  for (int j = 0; j < a.taps; ++j)
    {
      const int back = a.taps - 1 - j;
      f4 x0, x1;
      if (back <= s)
        {
          const size_t at = (size_t)(s - back) * a.xs + c;
          x0 = load4 (a.x, a.type, at), x1 = load4 (a.x, a.type, at + 4);
        }
      else if ((uint32_t)(back - s) <= a.pos0)
        {
          const float *r = a.ring + (size_t)((a.pos0 - (uint32_t)(back - s)) % (uint32_t)a.taps) * a.n + c;
          x0 = ldf4 (r), x1 = ldf4 (r + 4);
        }
      else
        continue;
      const f4 w0 = ldf4 (a.w + (size_t)j * a.n + c), w1 = ldf4 (a.w + (size_t)j * a.n + c + 4);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        lo[e] = __builtin_fmaf (w0[e], x0[e], lo[e]), hi[e] = __builtin_fmaf (w1[e], x1[e], hi[e]);
    }
  const size_t o = (size_t)s * a.os + c;
  if (a.type == VKL_TYPE_F32)
    {
#pragma unroll
      for (int e = 0; e < 4; ++e)
        lo[e] = silu (lo[e]), hi[e] = silu (hi[e]);
      stf4 ((float *)a.out + o, lo), stf4 ((float *)a.out + o + 4, hi);
      return;
    }
  uint32_t h[8];
#pragma unroll
  for (int e = 0; e < 4; ++e)
    h[e] = f2bf (silu (lo[e])), h[4 + e] = f2bf (silu (hi[e]));
  stg ((vkl_u32x4 *)((uint16_t *)a.out + o), vkl_u32x4{ h[0] | (h[1] << 16), h[2] | (h[3] << 16), h[4] | (h[5] << 16),
                                                        h[6] | (h[7] << 16) });
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

template <int DJ, bool DELTA>
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
          q[j] = load4 (r.q, r.type, (size_t)s * r.qs + qo + 16 * j);
          k[j] = load4 (r.k, r.type, (size_t)s * r.ks + qo + 16 * j);
          if (DELTA)
            g[j] = ldf4 (r.z + (size_t)s * r.zs + (size_t)h * r.dim + 16 * j + row);
        }
      float v = load_elem (r.v, r.type, (size_t)s * r.vs + vo), o = 0.f;
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

struct ChunkView
{
  float *w, *qd, *kt, *p, *u, *dec;
};

__device__ __forceinline__ ChunkView
chunk_view (float *ws, int dim, int vdim)
{
  ChunkView c;
  c.w = ws;                           // [64][dim]
  c.qd = c.w + (size_t)kChunk * dim;  // [64][dim]
  c.kt = c.qd + (size_t)kChunk * dim; // [dim][64]
  c.p = c.kt + (size_t)kChunk * dim;  // [64][64]
  c.u = c.p + kChunk * kChunk;        // [64][vdim]
  c.dec = c.u + (size_t)kChunk * vdim; // [dim]
  return c;
}

constexpr int kLdA = kChunk + 4;

inline size_t
prep_lds_bytes (int dim)
{
  return ((size_t)3 * kChunk * (dim + 4) + kChunk * kLdA + (size_t)kBlocks * dim + 2 * kChunk) * sizeof (float);
}

template <bool DELTA>
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
  __shared__ uint32_t steep;
  const int h = blockIdx.x % r.H, c = blockIdx.x / r.H, s0 = c * kChunk;
  const int n = min (kChunk, a.S - s0); // tokens; the rest of the chunk changes nothing
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const ChunkView v = chunk_view (ws + ((size_t)c * r.H + h) * chunk_floats (D, r.vdim), D, r.vdim);
  if (tid == 0)
    steep = 0;
  const size_t qo = (size_t)(h / r.rep) * D;
  // a wave per token: queries, keys, decays
  const float rate = DELTA ? ldg (r.rate + h) : 0.f;
  const float ld = DELTA ? 0.f : fmaxf (ldg (r.log_decay + h), -1.0e4f);
  for (int i = wave; i < kChunk; i += kPrepThreads / 64)
    {
      const bool in = i < n;
      const size_t s = (size_t)(s0 + min (i, n - 1));
      float x[2][2], qq = 0.f, kk = 0.f;
#pragma unroll
      for (int j = 0; j < 2; ++j)
        {
          const int d = lane + 64 * j, dc = min (d, D - 1);
          x[0][j] = in && d < D ? load_elem (r.q, r.type, s * r.qs + qo + dc) : 0.f;
          x[1][j] = in && d < D ? load_elem (r.k, r.type, s * r.ks + qo + dc) : 0.f;
          qq = __builtin_fmaf (x[0][j], x[0][j], qq), kk = __builtin_fmaf (x[1][j], x[1][j], kk);
        }
      float fq = r.qscale, fk = 1.f;
      if (DELTA)
        fq = r.qscale / sqrtf (wave_sum (qq) + r.unit_eps), fk = 1.0f / sqrtf (wave_sum (kk) + r.unit_eps);
#pragma unroll
      for (int j = 0; j < 2; ++j)
        {
          const int d = lane + 64 * j;
          if (d >= D)
            continue;
          qs[i * LD + d] = x[0][j] * fq, ks[i * LD + d] = x[1][j] * fk;
          float l = ld;
          if (DELTA)
            l = log_decay_of (rate, ldg (r.z + s * r.zs + (size_t)h * D + d) + ldg (r.dt_bias + (size_t)h * D + d));
          ls[i * LD + d] = in ? l : 0.f;
        }
      if (DELTA && lane == 0)
        beta[i] = in ? sigmoid (ldg (r.b + s * r.bs + h)) : 0.f;
    }
  __syncthreads ();
  for (int it = tid; it < kBlocks * D; it += kPrepThreads)
    {
      const int b = it / D, d = it - b * D;
      float l = 0.f;
      for (int i = 0; i < 16; ++i)
        {
          l += ls[(16 * b + i) * LD + d];
          ls[(16 * b + i) * LD + d] = l;
        }
      es[it] = l;
      if (l < -40.f)
        atomicOr (&steep, 1u << b);
    }
  __syncthreads ();

  // P, and for the delta rule A: pairs of blocks (bi, bj <= bi)
  const int lo = lane & 15, hi = 4 * (lane >> 4);
  for (int t = wave; t < kBlocks * (kBlocks + 1) / 2; t += kPrepThreads / 64)
    {
      const int bi = t < 1 ? 0 : t < 3 ? 1 : t < 6 ? 2 : 3, bj = t - bi * (bi + 1) / 2;
      if (bi == bj && ((steep >> bi) & 1u))
        {
          // pair by pair
          for (int pr = lane; pr < 256; pr += 64)
            {
              const int i = 16 * bi + (pr >> 4), j = 16 * bi + (pr & 15);
              float sa = 0.f, sp = 0.f;
              if (j <= i)
                for (int d = 0; d < D; ++d)
                  {
                    const float f = ks[j * LD + d] * expf (ls[i * LD + d] - ls[j * LD + d]);
                    sp = __builtin_fmaf (qs[i * LD + d], f, sp);
                    if (DELTA)
                      sa = __builtin_fmaf (ks[i * LD + d], f, sa);
                  }
              stg (v.p + i * kChunk + j, sp);
              if (DELTA)
                A[i * kLdA + j] = j < i ? sa * beta[i] : 0.f;
            }
          continue;
        }
      f4 accp = { 0.f, 0.f, 0.f, 0.f }, acca = accp;
      for (int d0 = hi; d0 < D; d0 += 16)
        {
          const f4 li = *(const f4 *)(ls + (16 * bi + lo) * LD + d0), lj = *(const f4 *)(ls + (16 * bj + lo) * LD + d0);
          const f4 qi = *(const f4 *)(qs + (16 * bi + lo) * LD + d0), kj = *(const f4 *)(ks + (16 * bj + lo) * LD + d0);
          f4 mid = { 0.f, 0.f, 0.f, 0.f };
          if (bj < bi)
            mid = *(const f4 *)(es + bj * D + d0);
          for (int b = bj + 1; b < bi; ++b)
            mid += *(const f4 *)(es + b * D + d0);
          f4 ki = { 0.f, 0.f, 0.f, 0.f };
          if (DELTA)
            ki = *(const f4 *)(ks + (16 * bi + lo) * LD + d0);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            {
              const float fi = expf (li[e]), x = kj[e] * expf (mid[e] - lj[e]);
              accp = mfma4 (qi[e] * fi, x, accp);
              if (DELTA)
                acca = mfma4 (ki[e] * fi, x, acca);
            }
        }
#pragma unroll
      for (int e = 0; e < 4; ++e)
        {
          const int i = 16 * bi + hi + e, j = 16 * bj + lo;
          stg (v.p + i * kChunk + j, j <= i ? accp[e] : 0.f);
          if (DELTA)
            A[i * kLdA + j] = j < i ? acca[e] * beta[i] : 0.f;
        }
    }
  // queries with the decay since the start of the chunk, keys with the decay to its end
  for (int it = tid; it < kChunk * D; it += kPrepThreads)
    {
      const int i = it / D, d = it - i * D;
      float l = ls[i * LD + d];
      for (int b = 0; b < i / 16; ++b)
        l += es[b * D + d];
      stg (v.qd + it, qs[i * LD + d] * expf (l));
    }
  for (int it = tid; it < kChunk * D; it += kPrepThreads)
    {
      const int d = it / kChunk, j = it - d * kChunk;
      float l = es[(j / 16) * D + d] - ls[j * LD + d];
      for (int b = j / 16 + 1; b < kBlocks; ++b)
        l += es[b * D + d];
      stg (v.kt + it, ks[j * LD + d] * expf (l));
    }
  for (int d = tid; d < D; d += kPrepThreads)
    {
      float l = 0.f;
      for (int b = 0; b < kBlocks; ++b)
        l += es[b * D + d];
      stg (v.dec + d, expf (l));
    }
  if (!DELTA)
    return;
  __syncthreads ();
  // (1 + A) x = right side, a column per thread: diag (beta) V, diag (beta) K D
  for (int col = tid; col < r.vdim + D; col += kPrepThreads)
    {
      const bool val = col < r.vdim;
      const int d = val ? 0 : col - r.vdim;
      float x[kChunk], before = 0.f;
#pragma unroll
      for (int i = 0; i < kChunk; ++i)
        {
          float y;
          if (val)
            y = load_elem (r.v, r.type, (size_t)(s0 + min (i, n - 1)) * r.vs + (size_t)h * r.vdim + col);
          else
            {
              if (i > 0 && i % 16 == 0)
                before += es[(i / 16 - 1) * D + d];
              y = ks[i * LD + d] * expf (ls[i * LD + d] + before);
            }
          x[i] = y * beta[i];
        }
#pragma unroll
      for (int i = 1; i < kChunk; ++i)
        {
          float y = x[i];
#pragma unroll
          for (int j = 0; j < i; j += 4)
            {
              const f4 w = *(const f4 *)(A + i * kLdA + j);
#pragma unroll
              for (int e = 0; e < 4; ++e)
                if (j + e < i)
                  y = __builtin_fmaf (-w[e], x[j + e], y);
            }
          x[i] = y;
        }
      float *dst = val ? v.u + col : v.w + d;
      const int stride = val ? r.vdim : D;
#pragma unroll
      for (int i = 0; i < kChunk; ++i)
        stg (dst + (size_t)i * stride, x[i]);
    }
}

// ---------------------------------------------------------------------------
// chunks: along the state
// ---------------------------------------------------------------------------
// wave w: tokens 16 w .. +15 of a chunk, and blocks w, w + 4 of the state's rows
template <int DB, bool DELTA>
__global__ __launch_bounds__ (256) void
chunk_scan_kernel (const RecurArgs a, const float *ws)
{
  constexpr int KB = (DB + 3) / 4, D = 16 * DB;
  __shared__ f4 ms[DB][64], us[kBlocks][64];
  const vkl_recurrence_args &r = a.r;
  const int h = blockIdx.x % r.H, vb = blockIdx.x / r.H;
  const int lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
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
  };
  auto fetch = [&] (int c, Operands &o) {
    const float *base = ws + ((size_t)c * r.H + h) * per;
    const ChunkView v = chunk_view (const_cast<float *> (base), D, r.vdim);
    const int row = 16 * wave + lo;
#pragma unroll
    for (int b = 0; b < DB; ++b)
      {
        o.q[b] = ldf4 (v.qd + (size_t)row * D + 16 * b + hi);
        if constexpr (DELTA)
          o.w[b] = ldf4 (v.w + (size_t)row * D + 16 * b + hi);
      }
#pragma unroll
    for (int b = 0; b < kBlocks; ++b)
      // (blocks right of the diagonal do not exist)
      o.p[b] = ldf4 (v.p + row * kChunk + 16 * min (b, wave) + hi);
#pragma unroll
    for (int i = 0; i < KB; ++i)
      {
        const int b = min (wave + 4 * i, DB - 1);
        o.dec[i] = ldf4 (v.dec + 16 * b + hi);
#pragma unroll
        for (int j = 0; j < kBlocks; ++j)
          o.k[i][j] = ldf4 (v.kt + (size_t)(16 * b + lo) * kChunk + 16 * j + hi);
      }
#pragma unroll
    for (int e = 0; e < 4; ++e)
      {
        const int t = 16 * wave + hi + e;
        if constexpr (DELTA)
          o.u[e] = ldg (v.u + (size_t)t * r.vdim + col);
        else
          {
            // (tokens past the end have keys of zero)
            const int s = min (c * kChunk + t, a.S - 1);
            o.u[e] = load_elem (r.v, r.type, (size_t)s * r.vs + (size_t)h * r.vdim + col);
          }
      }
  };
  auto chunk = [&] (int c, const Operands &o) {
    f4 acc = { 0.f, 0.f, 0.f, 0.f }, sub = acc, acc2 = acc, sub2 = acc;
#pragma unroll
    for (int b = 0; b < DB; ++b)
      {
        const f4 m = ms[b][lane];
#pragma unroll
        for (int e = 0; e < 4; e += 2)
          {
            acc = mfma4 (o.q[b][e], m[e], acc);
            if constexpr (DELTA)
              sub = mfma4 (o.w[b][e], m[e], sub);
            acc2 = mfma4 (o.q[b][e + 1], m[e + 1], acc2);
            if constexpr (DELTA)
              sub2 = mfma4 (o.w[b][e + 1], m[e + 1], sub2);
          }
      }
    us[wave][lane] = o.u - (sub + sub2);
    __syncthreads ();
#pragma unroll
    for (int b = 0; b < kBlocks; ++b)
      if (b <= wave)
        {
          const f4 u = us[b][lane];
#pragma unroll
          for (int e = 0; e < 4; e += 2)
            {
              acc = mfma4 (o.p[b][e], u[e], acc);
              acc2 = mfma4 (o.p[b][e + 1], u[e + 1], acc2);
            }
        }
    acc += acc2;
#pragma unroll
    for (int e = 0; e < 4; ++e)
      {
        const int s = c * kChunk + 16 * wave + hi + e;
        if (s < a.S)
          stg (r.out + (size_t)s * r.os + (size_t)h * r.vdim + col, acc[e]);
      }
#pragma unroll
    for (int i = 0; i < KB; ++i)
      {
        const int b = wave + 4 * i;
        if (b >= DB)
          continue;
        f4 m = o.dec[i] * ms[b][lane];
#pragma unroll
        for (int j = 0; j < kBlocks; ++j)
          {
            const f4 u = us[j][lane];
#pragma unroll
            for (int e = 0; e < 4; ++e)
              m = mfma4 (o.k[i][j][e], u[e], m);
          }
        ms[b][lane] = m;
      }
    __syncthreads ();
  };
  Operands x, y;
  fetch (0, x);
  __syncthreads ();
  for (int c = 0; c < chunks; c += 2)
    {
      fetch (min (c + 1, chunks - 1), y);
      chunk (c, x);
      if (c + 1 >= chunks)
        break;
      fetch (min (c + 2, chunks - 1), x);
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

template <bool DELTA>
int
launch_tokens (const RecurArgs &a, hipStream_t s)
{
  const dim3 grid ((unsigned)(a.r.H * (a.r.vdim / 16))), block (64);
  switch (a.r.dim / 32)
    {
    case 1: recur_tokens_kernel<2, DELTA><<<grid, block, 0, s>>> (a); break;
    case 2: recur_tokens_kernel<4, DELTA><<<grid, block, 0, s>>> (a); break;
    case 3: recur_tokens_kernel<6, DELTA><<<grid, block, 0, s>>> (a); break;
    case 4: recur_tokens_kernel<8, DELTA><<<grid, block, 0, s>>> (a); break;
    case 5: recur_tokens_kernel<10, DELTA><<<grid, block, 0, s>>> (a); break;
    case 6: recur_tokens_kernel<12, DELTA><<<grid, block, 0, s>>> (a); break;
    case 7: recur_tokens_kernel<14, DELTA><<<grid, block, 0, s>>> (a); break;
    default: recur_tokens_kernel<16, DELTA><<<grid, block, 0, s>>> (a); break;
    }
  return (int)hipGetLastError ();
}

template <bool DELTA>
int
launch_chunks (const RecurArgs &a, float *ws, hipStream_t s)
{
  static LdsLimit limit;
  const size_t lds = prep_lds_bytes (a.r.dim);
  const auto prep = chunk_prep_kernel<DELTA>;
  if (int e = limit.raise ((const void *)prep, lds))
    return e;
  const int chunks = (a.S + kChunk - 1) / kChunk;
  prep<<<dim3 ((unsigned)(chunks * a.r.H)), dim3 (kPrepThreads), lds, s>>> (a, ws);
  if (hipError_t e = hipGetLastError ())
    return (int)e;
  const dim3 grid ((unsigned)(a.r.H * (a.r.vdim / 16))), block (256);
  switch (a.r.dim / 32)
    {
    case 1: chunk_scan_kernel<2, DELTA><<<grid, block, 0, s>>> (a, ws); break;
    case 2: chunk_scan_kernel<4, DELTA><<<grid, block, 0, s>>> (a, ws); break;
    case 3: chunk_scan_kernel<6, DELTA><<<grid, block, 0, s>>> (a, ws); break;
    default: chunk_scan_kernel<8, DELTA><<<grid, block, 0, s>>> (a, ws); break;
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
template <bool WIDE>
__global__ __launch_bounds__ (256) void
gated_norm_kernel (const GatedNormArgs a)
{
  __shared__ float red[8];
  constexpr int T = WIDE ? 256 : 64;
  const int t = WIDE ? threadIdx.x : (threadIdx.x & 63);
  const size_t it = WIDE ? blockIdx.x : (size_t)blockIdx.x * 4 + (threadIdx.x >> 6);
  if (!WIDE && it >= (size_t)a.S * a.groups)
    return;
  const size_t s = it / a.groups, g0 = (it - s * a.groups) * (size_t)a.gw;
  const float *x = a.x + s * a.xs + g0;
  float ss = 0.f;
  for (int c = t * 4; c < a.gw; c += T * 4)
    {
      const f4 v = ldf4 (x + c);
#pragma unroll
      for (int e = 0; e < 4; ++e)
        ss = __builtin_fmaf (v[e], v[e], ss);
    }
  ss = WIDE ? group_sum (ss, red) : wave_sum (ss);
  const float alpha = 1.0f / sqrtf (ss / (float)a.n + a.eps);
  for (int c = t * 4; c < a.gw; c += T * 4)
    {
      const f4 v = ldf4 (x + c), w = ldf4 (a.w + c), g = load4 (a.gate, a.type, s * a.gs + g0 + c);
      f4 o;
#pragma unroll
      for (int e = 0; e < 4; ++e)
        o[e] = v[e] * alpha * w[e] * sigmoid (g[e]);
      const size_t at = s * a.os + g0 + c;
      if (a.type == VKL_TYPE_F32)
        stf4 ((float *)a.out + at, o);
      else
        stg ((unsigned long long *)((uint16_t *)a.out + at),
             (unsigned long long)f2bf (o[0]) | ((unsigned long long)f2bf (o[1]) << 16)
                 | ((unsigned long long)f2bf (o[2]) << 32) | ((unsigned long long)f2bf (o[3]) << 48));
    }
}

// ---------------------------------------------------------------------------
// one token
// ---------------------------------------------------------------------------
constexpr int kStepThreads = 512, kStepWaves = 8;

// y[i] = w[i, :] x for the rows i of one head, eight lanes per row
template <typename F>
__device__ __forceinline__ void
head_rows (const uint16_t *w, int rows, int K, const float *x, F put)
{
  const int sub = threadIdx.x & 7;
  for (int i0 = 0; i0 < rows; i0 += kStepThreads / 8)
    {
      const int i = i0 + (threadIdx.x >> 3), ic = min (i, rows - 1);
      float acc = 0.f;
      for (int k = sub * 8; k < K; k += 64)
        {
          float f[8];
          widen8 (ldg4 (w + (size_t)ic * K + k), f);
          const f4 x0 = *(const f4 *)(x + k), x1 = *(const f4 *)(x + k + 4);
#pragma unroll
          for (int e = 0; e < 4; ++e)
            acc = __builtin_fmaf (f[e], x0[e], acc), acc = __builtin_fmaf (f[4 + e], x1[e], acc);
        }
      acc = row_sum<8> (acc);
      if (sub == 0 && i < rows)
        put (i, acc);
    }
}

// DJ: dim / 16.  A wave takes blocks of 16 value columns in turn; the state of the
// first is requested before anything else.
template <int DJ, bool DELTA>
__global__ __launch_bounds__ (kStepThreads) void
recur_step_kernel (const RecurStepArgs a)
{
  constexpr int D = 16 * DJ, MV = 256;
  __shared__ __align__ (16) float q[D], k[D], g[D], v[MV], o[MV], z[MV];
  extern __shared__ __align__ (16) float lds_step[]; // a1 | g1
  __shared__ float red[kStepWaves];
  const int h = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lo = lane & 15, hi = 4 * (lane >> 4);
  const uint32_t pos = a.pos.get ();
  float *st = a.state + (size_t)h * D * a.vdim + lo;
  f4 m[DJ];
  auto fetch = [&] (int vb) {
#pragma unroll
    for (int j = 0; j < DJ; ++j)
#pragma unroll
      for (int e = 0; e < 4; ++e)
        m[j][e] = ldg (st + (size_t)(16 * j + hi + e) * a.vdim + 16 * vb);
  };
  const int blocks = a.vdim / 16;
  fetch (min (wave, blocks - 1));
  __builtin_amdgcn_sched_barrier (0);
  const int G = a.H / a.rep, hq = h / a.rep;
  const int nqk = G * D, n = 2 * nqk + a.H * a.vdim;
  // q, k, v of the head
  for (int c = tid; c < 2 * D + a.vdim; c += kStepThreads)
    {
      const int ch = c < D ? hq * D + c : c < 2 * D ? nqk + hq * D + c - D : 2 * nqk + h * a.vdim + c - 2 * D;
      float x = ldg (a.qkv + ch);
      if (DELTA)
        {
          const float now = x;
          x = ldg (a.conv + (size_t)(a.taps - 1) * n + ch) * now;
          for (int back = 1; back < a.taps; ++back)
            if ((uint32_t)back <= pos)
              x = __builtin_fmaf (ldg (a.conv + (size_t)(a.taps - 1 - back) * n + ch),
                                  ldg (a.ring + (size_t)((pos - (uint32_t)back) % (uint32_t)a.taps) * n + ch), x);
          x = silu (x);
          // (the row of this position is none that the step reads; heads that share a
          // query and key leave it to the first of them)
          if (c >= 2 * D || h % a.rep == 0)
            stg (a.ring + (size_t)(pos % (uint32_t)a.taps) * n + ch, now);
        }
      if (c < D)
        q[c] = x;
      else if (c < 2 * D)
        k[c - D] = x;
      else
        v[c - 2 * D] = x;
    }
  float decay = 1.f, beta = 0.f, fq = a.qscale, fk = 1.f;
  if (DELTA)
    {
      float *a1 = lds_step, *g1 = lds_step + a.r_a;
      for (int i = tid; i < a.r_a; i += kStepThreads)
        a1[i] = ldg (a.a1 + i);
      for (int i = tid; i < a.r_g; i += kStepThreads)
        g1[i] = ldg (a.g1 + i);
      beta = sigmoid (ldg (a.b + h));
      const float rate = ldg (a.rate + h);
      __syncthreads ();
      head_rows (a.w_a2 + (size_t)h * D * a.r_a, D, a.r_a, a1, [&] (int i, float y) {
        g[i] = expf (log_decay_of (rate, y + ldg (a.dt_bias + (size_t)h * D + i)));
      });
      head_rows (a.w_g2 + (size_t)h * a.vdim * a.r_g, a.vdim, a.r_g, g1, [&] (int i, float y) { z[i] = sigmoid (y); });
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
              stg (st + (size_t)(16 * j + hi + e) * a.vdim + 16 * vb, m[j][e]);
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
  for (int c = tid; c < a.vdim; c += kStepThreads)
    stg (a.out + (size_t)h * a.vdim + c, o[c] * alpha * ldg (a.gnorm + c) * z[c]);
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
  const size_t items = (size_t)S * (n / 8), keep = (size_t)std::min (S, taps) * n;
  short_conv_kernel<<<dim3 ((unsigned)((items + 255) / 256)), dim3 (256), 0, s>>> (a);
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
vkl_recurrence (const vkl_recurrence_args *r, int S, uint32_t pos0, int form, void *scratch, size_t scratch_bytes,
                void *stream)
{
  VKL_CHECK_ARG (r && S > 0 && recur_supported (r->H, r->rep, r->dim, r->vdim));
  const size_t nqk = (size_t)(r->H / r->rep) * r->dim, nv = (size_t)r->H * r->vdim;
  VKL_CHECK_ARG (r->q && r->k && r->v && r->state && r->out && r->qs >= nqk && r->ks >= nqk && r->vs >= nv && r->os >= nv);
  VKL_CHECK_ARG ((r->type == VKL_TYPE_F32 || r->type == VKL_TYPE_BF16) && (r->qs % 8) == 0 && (r->ks % 8) == 0
                 && ((uintptr_t)r->q % 16) == 0 && ((uintptr_t)r->k % 16) == 0);
  const bool delta = r->z != nullptr;
  if (delta)
    VKL_CHECK_ARG (r->b && r->dt_bias && r->rate && r->zs >= (size_t)r->H * r->dim && (r->zs % 4) == 0
                   && ((uintptr_t)r->z % 16) == 0 && ((uintptr_t)r->dt_bias % 16) == 0 && r->bs >= (size_t)r->H);
  else
    VKL_CHECK_ARG (r->log_decay);
  VKL_CHECK_ARG (form >= VKL_RECUR_AUTO && form <= VKL_RECUR_CHUNKS && (form != VKL_RECUR_CHUNKS || r->dim <= 128));
  hipStream_t s = (hipStream_t)stream;
  RecurArgs a = { *r, S, pos0 == 0 };
  const size_t one = (size_t)r->H * chunk_floats (r->dim, r->vdim) * sizeof (float);
  if (form == VKL_RECUR_TOKENS || r->dim > 128
      || (form == VKL_RECUR_AUTO && (S < kChunkMin || !scratch || scratch_bytes < one)))
    return delta ? launch_tokens<true> (a, s) : launch_tokens<false> (a, s);
  VKL_CHECK_ARG (scratch && scratch_bytes >= one && ((uintptr_t)scratch % 16) == 0);
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
        p.r.z = r->z + (size_t)at * r->zs, p.r.b = r->b + (size_t)at * r->bs;
      if (int e = delta ? launch_chunks<true> (p, (float *)scratch, s) : launch_chunks<false> (p, (float *)scratch, s))
        return e;
    }
  return 0;
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
  if (groups == 1)
    gated_norm_kernel<true><<<dim3 ((unsigned)S), dim3 (256), 0, s>>> (a);
  else
    gated_norm_kernel<false><<<dim3 ((unsigned)(((size_t)S * groups + 3) / 4)), dim3 (256), 0, s>>> (a);
  return vkl_launch_status ();
}
