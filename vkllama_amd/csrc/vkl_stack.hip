// Operators and the one-token step of decoder stacks with bf16 weights, an
// fp32 residual stream and mixers whose values are their keys
// (include/vkl_stack.h).
//
// The step of one token streams every weight once, so its kernels are built
// like those of vkl_decode.hip: workgroups of 8 waves, two per compute unit,
// every wave over whole weight rows with two 8 KiB items in flight, the
// activation row normed and staged in LDS while the first weights travel.
// Activations are fp32 in LDS (a bf16 weight is widened by a shift; the vector
// units have three times the throughput the stream needs), so the step serves
// both number formats; only the caches differ in type.
//   1. norm + all projections of the layer input: queries, keys or latent,
//      gates, feed-forward up (parallel layers: one norm feeds both parts);
//      keys go straight to their cache row
//   2. attention over the cache, split over workgroups
//      (latent: queries through W_uk^T first, which also norms the new latent
//      into the cache; the output through W_uv and the gate)
//   3. output projection and feed-forward down as ONE product over the
//      concatenated inputs, added into the residual row
// then final norm + tied output matrix + soft cap + arg-max.
#include "../../include/vkl_stack.h"
#include "vkl_gemm.h"
#include "vkl_stack_dev.h"
#include <algorithm>
#include <mutex>
#include <vector>

namespace vkl
{
namespace
{
// ---------------------------------------------------------------------------
// embedding and norms
// ---------------------------------------------------------------------------
struct EmbedArgs
{
  const uint16_t *table;
  uint32_t VH;
  int K, W;
  const uint32_t *toks;
  const uint32_t *loop; // replayed loop: the token is toks[loop[0]]
  const float *w; // null: the plain rows times scale
  float eps, scale;
  float *out;
  size_t os;
};

// one workgroup per token; a thread keeps its values of the row in registers
// (rows of up to 16384 values; wider ones are read twice)
__global__ __launch_bounds__ (1024) void
embed_norm_kernel (const EmbedArgs a)
{
  __shared__ float red[16];
  constexpr int NV = 2; // 16-byte loads per thread
  const uint32_t i = blockIdx.x;
  uint32_t id = ldg (a.toks + (a.loop ? ldg (a.loop) : i));
  id = id < a.VH ? id : 0;
  const uint16_t *row = a.table + (size_t)id * a.K;
  float *out = a.out + (size_t)i * a.os;
  const int tid = threadIdx.x;
  if ((a.K % 8) == 0 && a.W <= NV * 8192 && ((uintptr_t)a.table % 16) == 0)
    {
      float v[NV][8], ss = 0.f;
#pragma unroll
      for (int j = 0; j < NV; ++j)
        {
          const int c = (tid + j * 1024) * 8;
          widen8 (ldg4 (row + min (c, a.K - 8)), v[j]);
#pragma unroll
          for (int e = 0; e < 8; ++e)
            if (c + e < a.W)
              ss = __builtin_fmaf (v[j][e], v[j][e], ss);
        }
      float w[NV][8];
      if (a.w)
#pragma unroll
        for (int j = 0; j < NV; ++j)
#pragma unroll
          for (int e = 0; e < 8; ++e)
            w[j][e] = ldg (a.w + min ((tid + j * 1024) * 8 + e, a.W - 1));
      const float alpha = a.w ? 1.0f / sqrtf (group_sum (ss, red) / (float)a.W + a.eps) : 1.f;
      const bool vec = (a.W % 8) == 0 && (a.os % 4) == 0 && ((uintptr_t)a.out % 16) == 0;
#pragma unroll
      for (int j = 0; j < NV; ++j)
        {
          const int c = (tid + j * 1024) * 8;
          vkl_u32x4 o[2];
#pragma unroll
          for (int e = 0; e < 8; ++e)
            {
              const float f = a.w ? v[j][e] * alpha * w[j][e] : v[j][e] * a.scale;
              o[e >> 2][e & 3] = __float_as_uint (f);
              if (!vec && c + e < a.W)
                stg (out + c + e, f);
            }
          if (vec && c < a.W)
            stg ((vkl_u32x4 *)(out + c), o[0]), stg ((vkl_u32x4 *)(out + c + 4), o[1]);
        }
      return;
    }
  float alpha = 1.f;
  if (a.w)
    {
      float ss = 0.f;
      for (int c = tid; c < a.W; c += 1024)
        {
          const float v = bf2f (ldg (row + c));
          ss = __builtin_fmaf (v, v, ss);
        }
      alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.W + a.eps);
    }
  for (int c = tid; c < a.W; c += 1024)
    {
      const float v = bf2f (ldg (row + c));
      stg (out + c, a.w ? v * alpha * ldg (a.w + c) : v * a.scale);
    }
}

struct NormArgs
{
  const float *x;
  size_t xs;
  const uint32_t *rows;
  int W, Wp;
  const float *w;
  float eps;
  void *out;
  int otype;
  size_t os;
};

// one workgroup per row; NV 16-byte loads per thread keep the row in registers,
// 0: a row of any length and alignment, read twice
template <int NV>
__global__ __launch_bounds__ (256) void
rmsnorm_f32_kernel (const NormArgs a)
{
  __shared__ float red[8];
  const size_t r = a.rows ? ldg (a.rows + blockIdx.x) : blockIdx.x;
  const float *x = a.x + r * a.xs;
  const int tid = threadIdx.x;
  float ss = 0.f;
  if constexpr (NV > 0)
    {
      float4 v[NV];
#pragma unroll
      for (int j = 0; j < NV; ++j)
        {
          // (W is a multiple of 4 here: a load is all inside or all padding)
          const int c = (tid + j * 256) * 4;
          v[j] = __builtin_bit_cast (float4, ldg4 (x + min (c, a.W - 4)));
          if (c >= a.W)
            v[j] = make_float4 (0.f, 0.f, 0.f, 0.f);
          ss = __builtin_fmaf (v[j].x, v[j].x, ss), ss = __builtin_fmaf (v[j].y, v[j].y, ss);
          ss = __builtin_fmaf (v[j].z, v[j].z, ss), ss = __builtin_fmaf (v[j].w, v[j].w, ss);
        }
      const float alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.W + a.eps);
#pragma unroll
      for (int j = 0; j < NV; ++j)
        {
          const int c = (tid + j * 256) * 4;
          if (c >= a.Wp)
            continue;
          const float4 w = __builtin_bit_cast (float4, ldg4 (a.w + min (c, a.W - 4)));
          const float o[4] = { v[j].x * alpha * w.x, v[j].y * alpha * w.y, v[j].z * alpha * w.z, v[j].w * alpha * w.w };
          const size_t at = blockIdx.x * a.os + c;
          if (a.otype == VKL_TYPE_F32)
            stg ((vkl_u32x4 *)((float *)a.out + at), vkl_u32x4{ __float_as_uint (o[0]), __float_as_uint (o[1]),
                                                              __float_as_uint (o[2]), __float_as_uint (o[3]) });
          else
            stg ((unsigned long long *)((uint16_t *)a.out + at),
                 (unsigned long long)f2bf (o[0]) | ((unsigned long long)f2bf (o[1]) << 16)
                     | ((unsigned long long)f2bf (o[2]) << 32) | ((unsigned long long)f2bf (o[3]) << 48));
        }
      return;
    }
  for (int c = tid; c < a.W; c += 256)
    {
      const float v = ldg (x + c);
      ss = __builtin_fmaf (v, v, ss);
    }
  const float alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.W + a.eps);
  for (int c = tid; c < a.Wp; c += 256)
    store_elem (a.out, a.otype, blockIdx.x * a.os + c, c < a.W ? ldg (x + c) * alpha * ldg (a.w + c) : 0.f);
}

// ---------------------------------------------------------------------------
// attention over rows that are keys and values
// ---------------------------------------------------------------------------
constexpr int kRowThreads = 256;
constexpr int kRowUnroll = 4;
constexpr int kRowSplits = 64;  // parts a context is cut into at most (one per lane)
constexpr int kRowHeads = 32;   // query heads of a workgroup at most
constexpr int kRowTarget = 512; // workgroups a launch aims for
constexpr float kNoKey = -1.0e30f;

// The counters lie in front of the parts, in a block of fixed size, so that a
// scratch area may serve launches of different shapes (each leaves its counters
// at zero): only a split context has them, and there are at most kRowTarget / 2
// of those workgroup rows then.
// Every counter has a cache line of its own: arrivals at one line take turns.
constexpr size_t kRowCounterStride = 32; // words
constexpr size_t kRowCounterBytes = kRowTarget / 2 * kRowCounterStride * sizeof (uint32_t);

struct RowAttnArgs
{
  const void *q;
  int qtype;
  size_t qs;
  const void *rows, *vals; // vals: values of their own (null: the rows are keys and values)
  size_t rs;
  int chunk, sink; // a position sees its own chunk (0: everything before it); a score 0 without a value
  int G, D, rep, tiles, ht; // rep: query heads per group; tiles of ht heads
  StepPos pos;
  float scale, tcoef;
  int tevery;
  void *out;
  int otype;
  size_t os;
  int nsplit;
  float *pm, *pl, *pacc; // parts of a split context: [S][G*tiles][nsplit][HT] (x D)
  uint32_t *cnt;         // [S][G*tiles]; null: the parts stay, the next launch combines them
};

// how a context of L positions is cut: parts of `chunk` rows, a multiple of the
// rows a workgroup takes at a time
__device__ __forceinline__ int
row_chunk (int L, int nsplit, int step)
{
  const int c = (L + nsplit - 1) / nsplit;
  return (c + step - 1) / step * step;
}

template <int LPR>
__device__ __forceinline__ float
lanes_sum (float v)
{
  v = row_sum<(LPR < 16 ? LPR : 16)> (v);
  if (LPR >= 32)
    v += __shfl_xor (v, 16, 64);
  if (LPR >= 64)
    v += __shfl_xor (v, 32, 64);
  return v;
}

template <typename CT> struct RowVec; // 8 elements of a row as they lie
template <> struct RowVec<uint16_t>
{
  uint4 a;
  __device__ __forceinline__ void
  load (const uint16_t *p)
  {
    a = ldg4 (p);
  }
  __device__ __forceinline__ void
  get (float (&f)[8]) const
  {
    widen8 (a, f);
  }
  static __device__ __forceinline__ float
  exponential (float x)
  {
    return __builtin_amdgcn_exp2f (x * 1.44269504088896340736f);
  }
};
template <> struct RowVec<float>
{
  uint4 a, b;
  __device__ __forceinline__ void
  load (const float *p)
  {
    a = ldg4 (p), b = ldg4 (p + 4);
  }
  __device__ __forceinline__ void
  get (float (&f)[8]) const
  {
    const uint32_t u[8] = { a.x, a.y, a.z, a.w, b.x, b.y, b.z, b.w };
#pragma unroll
    for (int e = 0; e < 8; ++e)
      f[e] = __uint_as_float (u[e]);
  }
  static __device__ __forceinline__ float
  exponential (float x)
  {
    return expf (x);
  }
};

// 8 neighbouring values in either type
__device__ __forceinline__ void
load8 (const void *p, int type, size_t i, float (&f)[8])
{
  if (type == VKL_TYPE_F32)
    {
      RowVec<float> v;
      v.load ((const float *)p + i);
      v.get (f);
    }
  else
    {
      RowVec<uint16_t> v;
      v.load ((const uint16_t *)p + i);
      v.get (f);
    }
}

// 16 bytes past the XCD's L2, like st_coherent_u32 (the caller waits for the
// store before it tells anybody)
__device__ __forceinline__ void
st_coherent_16 (float *p, const float (&v)[4])
{
  const vkl_u32x4 w = { __float_as_uint (v[0]), __float_as_uint (v[1]), __float_as_uint (v[2]), __float_as_uint (v[3]) };
  asm volatile ("global_store_dwordx4 %0, %1, off sc1" ::"v"(p), "v"(w) : "memory");
}

// 16 bytes that another XCD wrote through, read past this XCD's L2
__device__ __forceinline__ float4
ld_coherent_16 (const float *p)
{
  const unsigned long long a = __hip_atomic_load ((const unsigned long long *)p, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  const unsigned long long b = __hip_atomic_load ((const unsigned long long *)p + 1, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
  return make_float4 (__uint_as_float ((uint32_t)a), __uint_as_float ((uint32_t)(a >> 32)), __uint_as_float ((uint32_t)b),
                      __uint_as_float ((uint32_t)(b >> 32)));
}

// LDS of combine_parts in floats
template <int THREADS>
constexpr int
combine_lds ()
{
  return kRowHeads * kRowSplits + 4 * (THREADS - 128);
}

// The parts of nh heads (entries [part][ht] from pbase on) into their outputs, by
// a whole workgroup: a wave per head for the weights, lane p holding part p, then
// four neighbouring values per thread with the parts dealt to groups of 128
// threads.  The first values are requested together with the maxima and sums.
// (a sink takes part in the maximum and in the sum)
template <int THREADS>
__device__ __forceinline__ void
combine_parts (const RowAttnArgs &a, int ht, int nh, int active, size_t pbase, size_t out0, float *lds)
{
  constexpr int NG = THREADS / 128;
  constexpr int R = 32 / NG; // parts of a group in flight
  float *wgt = lds; // [kRowHeads][kRowSplits]
  float4 *swap = (float4 *)(lds + kRowHeads * kRowSplits);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int grp = tid >> 7, q4 = a.D / 4, outs = nh * q4;
  float4 pv[R];
  auto request = [&] (int o0, int p0) {
    const int oc = min (o0 + (tid & 127), outs - 1), h = oc / q4;
    const float *src = a.pacc + (pbase * ht + h) * a.D + (oc - h * q4) * 4;
#pragma unroll
    for (int j = 0; j < R; ++j)
      pv[j] = ld_coherent_16 (src + (size_t)min (p0 + NG * j + grp, active - 1) * ht * a.D);
  };
  constexpr int NW = THREADS / 64, HW = kRowHeads / NW; // heads per wave
  float mv[HW], lv[HW];
#pragma unroll
  for (int i = 0; i < HW; ++i)
    {
      const size_t at = (pbase + min (lane, active - 1)) * ht + min (wave + NW * i, nh - 1);
      mv[i] = __uint_as_float (ld_coherent_u32 ((const uint32_t *)a.pm + at));
      lv[i] = __uint_as_float (ld_coherent_u32 ((const uint32_t *)a.pl + at));
    }
  request (0, 0);
#pragma unroll
  for (int i = 0; i < HW; ++i)
    if (wave + NW * i < nh)
      {
        const float M = a.sink ? fmaxf (wave_max (mv[i]), 0.f) : wave_max (mv[i]);
        const float f = lane < active ? expf (mv[i] - M) : 0.f;
        wgt[(wave + NW * i) * kRowSplits + lane] = f / (wave_sum (f * lv[i]) + (a.sink ? expf (-M) : 0.f));
      }
  __syncthreads ();
  for (int o0 = 0; o0 < outs; o0 += 128)
    {
      const int o = o0 + (tid & 127), oc = min (o, outs - 1), h = oc / q4, d = (oc - h * q4) * 4;
      float4 v = make_float4 (0.f, 0.f, 0.f, 0.f);
      for (int p0 = 0; p0 < active; p0 += NG * R)
        {
          if (o0 + p0 > 0)
            request (o0, p0);
#pragma unroll
          for (int j = 0; j < R; ++j)
            {
              const float f = wgt[h * kRowSplits + p0 + NG * j + grp];
              v.x = __builtin_fmaf (f, pv[j].x, v.x), v.y = __builtin_fmaf (f, pv[j].y, v.y);
              v.z = __builtin_fmaf (f, pv[j].z, v.z), v.w = __builtin_fmaf (f, pv[j].w, v.w);
            }
        }
      if (grp)
        swap[tid - 128] = v;
      __syncthreads ();
      if (!grp && o < outs)
        {
          float r[4] = { v.x, v.y, v.z, v.w };
#pragma unroll
          for (int i = 0; i < NG - 1; ++i)
            {
              const float4 w = swap[tid + i * 128];
              r[0] += w.x, r[1] += w.y, r[2] += w.z, r[3] += w.w;
            }
#pragma unroll
          for (int e = 0; e < 4; ++e)
            store_elem (a.out, a.otype, out0 + (size_t)h * a.D + d + e, r[e]);
        }
      __syncthreads ();
    }
}

// Counts the workgroup in once its (written-through) parts are in memory; true
// in the one that arrives last.
__device__ __forceinline__ bool
last_of_parts (uint32_t *cnt, int active, uint32_t *flag)
{
  __builtin_amdgcn_s_waitcnt (0);
  __syncthreads ();
  if (threadIdx.x == 0)
    {
      const uint32_t old = __hip_atomic_fetch_add (cnt, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      const bool last = old + 1u == (uint32_t)active;
      if (last)
        st_coherent_u32 (cnt, 0u);
      *flag = last ? 1u : 0u;
    }
  __syncthreads ();
  return *flag != 0u;
}

// LPR lanes share a row, NCH chunks of 8 values per lane; HT query heads per
// workgroup.  Every group of LPR lanes walks rows of its own with a running
// maximum; the groups' results meet in LDS at the end.
// VALS: values of their own, chunks and a sink.
template <typename CT, int LPR, int NCH, int HT, bool VALS>
__global__ __launch_bounds__ (kRowThreads) void
attn_rows_kernel (const RowAttnArgs a)
{
  constexpr int RPW = 64 / LPR, RPS = 4 * RPW, U = kRowUnroll, STEP = RPS * U;
  constexpr int NS = kRowThreads / LPR; // lane groups
  constexpr int DA = LPR * 8 * NCH;     // values of a row the lanes cover
  extern __shared__ __align__ (16) float lds_rows[]; // [NS][HT][DA]
  __shared__ float sm[NS][HT], sl[NS][HT];
  __shared__ uint32_t last_s;
  const int s = blockIdx.z, gt = blockIdx.y;
  const int g = gt / a.tiles, t = gt - g * a.tiles;
  const uint32_t pos = a.pos.get () + (uint32_t)s;
  // the rows are counted from the first one that is visible
  const uint32_t low = VALS && a.chunk ? pos / (uint32_t)a.chunk * (uint32_t)a.chunk : 0u;
  const int L = (int)(pos - low) + 1;
  const int chunk = row_chunk (L, a.nsplit, STEP);
  const int active = (L + chunk - 1) / chunk;
  const int c = blockIdx.x;
  if (c >= active)
    return;
  const int l0 = c * chunk, l1 = min (L, l0 + chunk);
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  const int sub = lane % LPR, grp = lane / LPR, slot = tid / LPR;

  const int col[2] = { sub * 8, LPR * 8 + sub * 8 };
  const CT *base = (const CT *)a.rows + (size_t)low * a.rs + (size_t)g * a.D;
  const CT *vbase = VALS ? (const CT *)a.vals + (size_t)low * a.rs + (size_t)g * a.D : nullptr;
  int cc[NCH]; // columns clamped into the row (lanes past its end contribute q = 0)
#pragma unroll
  for (int n = 0; n < NCH; ++n)
    cc[n] = min (col[n], a.D - 8);

  // the first rows travel while the queries are fetched
  RowVec<CT> nx[U][NCH], nv[VALS ? U : 1][NCH];
  auto issue = [&] (int lb) {
#pragma unroll
    for (int u = 0; u < U; ++u)
#pragma unroll
      for (int n = 0; n < NCH; ++n)
        {
          const size_t o = (size_t)min (lb + (u * 4 + wave) * RPW + grp, l1 - 1) * a.rs + cc[n];
          nx[u][n].load (base + o);
          if constexpr (VALS)
            nv[u][n].load (vbase + o);
        }
  };
  issue (l0);
  __builtin_amdgcn_sched_barrier (0);
  const int h0 = g * a.rep + t * HT;
  float q[HT][NCH * 8];
  {
    float f = a.scale;
    if (a.tcoef != 0.f)
      f *= 1.0f + a.tcoef * logf ((float)((pos + 1u) / (uint32_t)a.tevery + 1u));
#pragma unroll
    for (int h = 0; h < HT; ++h)
      {
        const size_t qo = (size_t)s * a.qs + (size_t)(g * a.rep + min (t * HT + h, a.rep - 1)) * a.D;
#pragma unroll
        for (int n = 0; n < NCH; ++n)
          {
            float v[8];
            load8 (a.q, a.qtype, qo + cc[n], v);
#pragma unroll
            for (int e = 0; e < 8; ++e)
              q[h][n * 8 + e] = col[n] < a.D ? v[e] * f : 0.f;
          }
      }
  }
  float m[HT], l[HT], acc[HT][NCH * 8];
#pragma unroll
  for (int h = 0; h < HT; ++h)
    {
      m[h] = kNoKey, l[h] = 0.f;
#pragma unroll
      for (int e = 0; e < NCH * 8; ++e)
        acc[h][e] = 0.f;
    }

  for (int lb = l0; lb < l1; lb += STEP)
    {
      float row[U][NCH * 8], val[VALS ? U : 1][NCH * 8];
#pragma unroll
      for (int u = 0; u < U; ++u)
#pragma unroll
        for (int n = 0; n < NCH; ++n)
          {
            float f[8];
            nx[u][n].get (f);
#pragma unroll
            for (int e = 0; e < 8; ++e)
              row[u][n * 8 + e] = f[e];
            if constexpr (VALS)
              {
                nv[u][n].get (f);
#pragma unroll
                for (int e = 0; e < 8; ++e)
                  val[u][n * 8 + e] = f[e];
              }
          }
      issue (min (lb + STEP, l1 - 1));
#pragma unroll
      for (int h = 0; h < HT; ++h)
        {
          float sc[U], mx = m[h];
#pragma unroll
          for (int u = 0; u < U; ++u)
            {
              float d = 0.f;
#pragma unroll
              for (int e = 0; e < NCH * 8; ++e)
                d = __builtin_fmaf (q[h][e], row[u][e], d);
              d = lanes_sum<LPR> (d);
              sc[u] = lb + (u * 4 + wave) * RPW + grp < l1 ? d : kNoKey;
              mx = fmaxf (mx, sc[u]);
            }
          const float al = RowVec<CT>::exponential (m[h] - mx);
          m[h] = mx;
          l[h] *= al;
#pragma unroll
          for (int e = 0; e < NCH * 8; ++e)
            acc[h][e] *= al;
#pragma unroll
          for (int u = 0; u < U; ++u)
            {
              // (a group that has seen no row yet has mx = kNoKey: the guard
              // keeps its weights at zero)
              const float p = sc[u] > kNoKey ? RowVec<CT>::exponential (sc[u] - mx) : 0.f;
              l[h] += p;
#pragma unroll
              for (int e = 0; e < NCH * 8; ++e)
                acc[h][e] = __builtin_fmaf (p, VALS ? val[u][e] : row[u][e], acc[h][e]);
            }
        }
    }

  // the lane groups' parts
  if (sub == 0)
#pragma unroll
    for (int h = 0; h < HT; ++h)
      sm[slot][h] = m[h];
  __syncthreads ();
  const bool whole = a.cnt && active == 1; // no other part: the sink belongs here
  float M[HT];
#pragma unroll
  for (int h = 0; h < HT; ++h)
    {
      float v = VALS && a.sink && whole ? 0.f : kNoKey;
#pragma unroll
      for (int i = 0; i < NS; ++i)
        v = fmaxf (v, sm[i][h]);
      M[h] = v;
      const float f = expf (m[h] - v);
      if (sub == 0)
        sl[slot][h] = l[h] * f;
#pragma unroll
      for (int n = 0; n < NCH; ++n)
#pragma unroll
        for (int e = 0; e < 8; ++e)
          lds_rows[(slot * HT + h) * DA + col[n] + e] = acc[h][n * 8 + e] * f;
    }
  __syncthreads ();
  const int nh = min (HT, a.rep - t * HT); // heads of this tile
  const size_t pbase = ((size_t)s * gridDim.y + gt) * a.nsplit;
  for (int o = tid * 4; o < nh * a.D; o += kRowThreads * 4)
    {
      const int h = o / a.D, d = o - h * a.D;
      float v[4] = { 0.f, 0.f, 0.f, 0.f }, S = 0.f;
#pragma unroll
      for (int i = 0; i < NS; ++i)
        {
          const float4 w = *(const float4 *)(lds_rows + (i * HT + h) * DA + d);
          v[0] += w.x, v[1] += w.y, v[2] += w.z, v[3] += w.w;
        }
      float *dst = a.pacc + ((pbase + c) * HT + h) * a.D + d;
      if (!a.cnt)
        stg ((vkl_u32x4 *)dst, vkl_u32x4{ __float_as_uint (v[0]), __float_as_uint (v[1]), __float_as_uint (v[2]),
                                          __float_as_uint (v[3]) });
      else if (whole)
        {
          for (int i = 0; i < NS; ++i)
            S += sl[i][h];
          if (VALS && a.sink)
            {
              float mm = 0.f;
              for (int i = 0; i < NS; ++i)
                mm = fmaxf (mm, sm[i][h]);
              S += expf (-mm);
            }
#pragma unroll
          for (int e = 0; e < 4; ++e)
            store_elem (a.out, a.otype, (size_t)s * a.os + (size_t)(h0 + h) * a.D + d + e, v[e] / S);
        }
      else
        // (write-through: the workgroup that combines may be on another XCD)
        st_coherent_16 (dst, v);
    }
  if (whole)
    return;
  if (tid < nh)
    {
      float S = 0.f, mm = kNoKey;
      for (int i = 0; i < NS; ++i)
        S += sl[i][tid], mm = fmaxf (mm, sm[i][tid]);
      if (!a.cnt)
        {
          stg (a.pm + (pbase + c) * HT + tid, mm);
          stg (a.pl + (pbase + c) * HT + tid, S);
        }
      else
        {
          st_coherent_u32 ((uint32_t *)a.pm + (pbase + c) * HT + tid, __float_as_uint (mm));
          st_coherent_u32 ((uint32_t *)a.pl + (pbase + c) * HT + tid, __float_as_uint (S));
        }
    }
  if (!a.cnt)
    return;
  if (!last_of_parts (a.cnt + ((size_t)s * gridDim.y + gt) * kRowCounterStride, active, &last_s))
    return;
  combine_parts<kRowThreads> (a, HT, nh, active, pbase, (size_t)s * a.os + (size_t)h0 * a.D, lds_rows);
}

// heads per workgroup: as many as share a row, within the registers
int
row_head_tile (int rep, int D)
{
  const int cap = D > 256 ? 4 : 8;
  int ht = 1;
  while (ht * 2 <= cap && ht < rep)
    ht *= 2;
  return ht;
}

// the matrix-core form: bf16 rows that several heads share, of the sizes it is
// instantiated for
bool
row_mfma (int ctype, int rep, int D, bool vals = false)
{
  return !vals && ctype == VKL_TYPE_BF16 && rep >= 2 && (D <= 256 || (D <= 512 && D % 64 == 0));
}

struct RowPlan
{
  bool mfma;
  int ht, tiles, nsplit;
  size_t parts; // entries of pm / pl
};

RowPlan
row_plan (int ctype, int H, int G, int D, int S, bool vals = false)
{
  RowPlan p;
  const int rep = H / G;
  p.mfma = row_mfma (ctype, rep, D, vals);
  p.ht = p.mfma ? std::min (rep, kRowHeads) : row_head_tile (rep, D);
  p.tiles = (rep + p.ht - 1) / p.ht;
  const long groups = (long)G * p.tiles * S;
  p.nsplit = (int)std::max (1L, std::min ((long)(p.mfma ? kRowSplits : kRowSplits / 2), kRowTarget / groups));
  p.parts = (size_t)groups * p.nsplit * p.ht;
  return p;
}

// ---- the matrix-core form ----------------------------------------------------
// A workgroup of eight waves holds up to 32 query heads that share the rows of its
// part of the context, and walks the part in tiles of 64 rows.  A tile lies in LDS
// twice: as it is (first product: scores) and transposed (second product: the rows
// as values).
//   S[row, head] = sum_d C[row, d] Q[head, d]: v_mfma_f32_16x16x32_bf16, waves = 4
//     blocks of 16 rows x 2 halves of d; the halves meet in LDS in fp32
//   weights: thread (head = tid % 32, rows 4 (tid / 32) .. +3), the maximum over
//     the tile through LDS, weights to LDS as bf16 (over the tile, which is done
//     with its first form)
//   O^T[d, head] = sum_row C^T[d, row] P^T[row, head]: v_mfma_f32_32x32x16_bf16,
//     waves = blocks of 32 d in turn
// Transposed rows are stored with their 16-byte groups of eight rows XOR-swizzled by
// the block of d they come from, against bank conflicts.
constexpr int kMfThreads = 512, kMfWaves = 8;
constexpr int kMfRows = 64;
constexpr int kMfLdv = kMfRows + 8;
constexpr int kMfLds = 33; // floats per row of the exchanged scores

typedef __bf16 bf8 __attribute__ ((ext_vector_type (8)));
typedef float float4v __attribute__ ((ext_vector_type (4)));
typedef float float16v __attribute__ ((ext_vector_type (16)));

template <int NBLK>
constexpr size_t
mfma_rows_lds ()
{
  constexpr int D = 32 * NBLK, DP = (D + 63) / 64 * 64;
  const size_t need = (size_t)kMfRows * (DP + 8) * 2 + (size_t)D * kMfLdv * 2 + 2 * kMfRows * kMfLds * 4 + 16 * 32 * 4;
  const size_t comb = combine_lds<kMfThreads> () * 4 + 16;
  return need > comb ? need : comb;
}

template <int NBLK>
__global__ __launch_bounds__ (kMfThreads) void
attn_rows_mfma_kernel (const RowAttnArgs a)
{
  constexpr int D = 32 * NBLK, DP = (D + 63) / 64 * 64, LDK = DP + 8, CPR = D / 8;
  constexpr int ITEMS = kMfRows / 2 * CPR;                     // (row pair, 8 values)
  constexpr int IT = (ITEMS + kMfThreads - 1) / kMfThreads;
  constexpr bool RAG = ITEMS % kMfThreads != 0;
  constexpr int NB = (NBLK + kMfWaves - 1) / kMfWaves;         // blocks of d per wave
  constexpr int KS = DP / 64;                                  // 32-wide steps of half a row
  extern __shared__ __align__ (16) uint8_t lds_mf[];
  uint16_t *Ks = (uint16_t *)lds_mf;                           // [64][LDK]
  uint16_t *Pb = Ks;                                           // [32][kMfLdv], once the scores are out
  uint16_t *Vt = Ks + kMfRows * LDK;                           // [D][kMfLdv]
  float *Sp = (float *)(Vt + D * kMfLdv);                      // [2][64][kMfLds]
  float *red = Sp + 2 * kMfRows * kMfLds;                      // [16][32]
  static_assert (32 * kMfLdv <= kMfRows * LDK, "the weights fit over the tile");
  const int s = blockIdx.z, gt = blockIdx.y;
  const int g = gt / a.tiles, t = gt - g * a.tiles;
  const int ht = a.ht, nh = min (ht, a.rep - t * ht);
  const uint32_t pos = a.pos.get () + (uint32_t)s;
  const int L = (int)pos + 1;
  const int chunk = row_chunk (L, a.nsplit, kMfRows);
  const int active = (L + chunk - 1) / chunk;
  const int c = blockIdx.x;
  if (c >= active)
    return;
  const int l0 = c * chunk, l1 = min (L, l0 + chunk);
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int lq = lane & 31, hh = lane >> 5;
  const uint16_t *base = (const uint16_t *)a.rows + (size_t)g * D;

  auto swizzle = [] (int ch) { return (ch ^ (ch >> 3)) & 7; };
  // item: four neighbouring row pairs x a run of chunks per wave
  uint4 ra[IT][2], rb[IT][2]; // two tiles on their way
  auto item = [&] (int i, int &pair, int &ch) {
    const int it = RAG ? min (tid + i * kMfThreads, ITEMS - 1) : tid + i * kMfThreads;
    if constexpr (CPR % 16 == 0)
      ch = (it & 15) + 16 * ((it >> 6) % (CPR / 16)), pair = (it >> 6) / (CPR / 16) * 4 + ((it >> 4) & 3);
    else
      ch = (it >> 2) % CPR, pair = ((it >> 2) / CPR) * 4 + (it & 3);
  };
  auto load = [&] (int lb, uint4 (&rv)[IT][2]) {
#pragma unroll
    for (int i = 0; i < IT; ++i)
      {
        int pair, ch;
        item (i, pair, ch);
        const uint16_t *p = base + ch * 8;
        rv[i][0] = ldg4 (p + (size_t)min (lb + 2 * pair, l1 - 1) * a.rs);
        rv[i][1] = ldg4 (p + (size_t)min (lb + 2 * pair + 1, l1 - 1) * a.rs);
      }
  };
  auto store = [&] (const uint4 (&rv)[IT][2]) {
#pragma unroll
    for (int i = 0; i < IT; ++i)
      {
        if (RAG && tid + i * kMfThreads >= ITEMS)
          continue;
        int pair, ch;
        item (i, pair, ch);
        *(uint4 *)(Ks + (2 * pair) * LDK + ch * 8) = rv[i][0];
        *(uint4 *)(Ks + (2 * pair + 1) * LDK + ch * 8) = rv[i][1];
        const uint32_t x[4] = { rv[i][0].x, rv[i][0].y, rv[i][0].z, rv[i][0].w };
        const uint32_t y[4] = { rv[i][1].x, rv[i][1].y, rv[i][1].z, rv[i][1].w };
        uint32_t *dst = (uint32_t *)(Vt + (ch * 8) * kMfLdv) + ((pair >> 2) ^ swizzle (ch)) * 4 + (pair & 3);
#pragma unroll
        for (int e = 0; e < 4; ++e)
          {
            dst[(2 * e) * (kMfLdv / 2)] = (x[e] & 0xffffu) | (y[e] << 16);
            dst[(2 * e + 1) * (kMfLdv / 2)] = (x[e] >> 16) | (y[e] & 0xffff0000u);
          }
      }
    // columns that pad a row to a multiple of 64 (the weights may have lain there)
    if (DP != D && tid < kMfRows * (DP - D) / 8)
      *(uint4 *)(Ks + (tid / 4) * LDK + D + (tid & 3) * 8) = make_uint4 (0, 0, 0, 0);
  };
  load (l0, ra);
  load (min (l0 + kMfRows, l1 - 1), rb);
  __builtin_amdgcn_sched_barrier (0);

  const int blk = wave & 3, dh = wave >> 2;
  float f = a.scale;
  if (a.tcoef != 0.f)
    f *= 1.0f + a.tcoef * logf ((float)((pos + 1u) / (uint32_t)a.tevery + 1u));
  const int h0 = g * a.rep + t * ht;
  // the queries go through LDS (where the transposed rows will lie): every value
  // is fetched once, all waves need it
  uint16_t *Qs = Vt; // [32][LDK]
  static_assert (32 * LDK <= D * kMfLdv, "the queries fit over the transposed rows");
  for (int i = tid; i < 32 * (DP / 8); i += kMfThreads)
    {
      const int h = i / (DP / 8), d = (i - h * (DP / 8)) * 8;
      float v[8];
      load8 (a.q, a.qtype, (size_t)s * a.qs + (size_t)(h0 + min (h, nh - 1)) * D + (DP == D ? d : min (d, D - 8)), v);
      uint32_t w[4];
#pragma unroll
      for (int e = 0; e < 4; ++e)
        w[e] = DP == D || d < D ? f2bf (v[2 * e]) | ((uint32_t)f2bf (v[2 * e + 1]) << 16) : 0u;
      *(uint4 *)(Qs + h * LDK + d) = make_uint4 (w[0], w[1], w[2], w[3]);
    }
  __syncthreads ();
  // this wave's half of d: heads 0 .. 15 and 16 .. 31
  bf8 qf[2][KS];
#pragma unroll
  for (int n = 0; n < 2; ++n)
#pragma unroll
    for (int kt = 0; kt < KS; ++kt)
      qf[n][kt] = *(const bf8 *)(Qs + (16 * n + (lane & 15)) * LDK + dh * (DP / 2) + kt * 32 + (lane >> 4) * 8);
  float m = kNoKey, sum = 0.f; // of head lq; the sum over this thread's rows
  const int rg = tid >> 5;
  float16v oacc[NB];
#pragma unroll
  for (int b = 0; b < NB; ++b)
#pragma unroll
    for (int r = 0; r < 16; ++r)
      oacc[b][r] = 0.f;

  auto tile = [&] (int lb, uint4 (&rv)[IT][2]) {
      __syncthreads ();
      store (rv);
      __syncthreads ();
      load (min (lb + 2 * kMfRows, l1 - 1), rv);
      {
        float4v acc[2] = { { 0.f, 0.f, 0.f, 0.f }, { 0.f, 0.f, 0.f, 0.f } };
        const uint16_t *kp = Ks + (16 * blk + (lane & 15)) * LDK + dh * (DP / 2) + (lane >> 4) * 8;
#pragma unroll
        for (int kt = 0; kt < KS; ++kt)
          {
            const bf8 k = *(const bf8 *)(kp + kt * 32);
            acc[0] = __builtin_amdgcn_mfma_f32_16x16x32_bf16 (k, qf[0][kt], acc[0], 0, 0, 0);
            acc[1] = __builtin_amdgcn_mfma_f32_16x16x32_bf16 (k, qf[1][kt], acc[1], 0, 0, 0);
          }
        float *sp = Sp + (dh * kMfRows + 16 * blk + 4 * (lane >> 4)) * kMfLds + (lane & 15);
#pragma unroll
        for (int r = 0; r < 4; ++r)
          sp[r * kMfLds] = acc[0][r], sp[r * kMfLds + 16] = acc[1][r];
      }
      __syncthreads ();
      float sv[4], bm = kNoKey;
#pragma unroll
      for (int j = 0; j < 4; ++j)
        {
          const int row = 4 * rg + j;
          const float sc = (Sp[row * kMfLds + lq] + Sp[(kMfRows + row) * kMfLds + lq]) * f;
          sv[j] = lb + row < l1 ? sc : kNoKey;
          bm = fmaxf (bm, sv[j]);
        }
      red[rg * 32 + lq] = bm;
      __syncthreads ();
#pragma unroll
      for (int i = 0; i < 16; ++i)
        bm = fmaxf (bm, red[i * 32 + lq]);
      const float mn = fmaxf (m, bm);
      if (__builtin_amdgcn_ballot_w64 (mn != m) != 0)
        {
          const float al = RowVec<uint16_t>::exponential (m - mn);
          sum *= al;
#pragma unroll
          for (int b = 0; b < NB; ++b)
#pragma unroll
            for (int r = 0; r < 16; ++r)
              oacc[b][r] *= al;
          m = mn;
        }
      {
        // (a masked row: exp of a hugely negative number; the sum takes the weight
        // as the product consumes it)
        uint16_t e[4];
#pragma unroll
        for (int j = 0; j < 4; ++j)
          {
            e[j] = f2bf (RowVec<uint16_t>::exponential (sv[j] - m));
            sum += bf2f (e[j]);
          }
        uint32_t *pp = (uint32_t *)(Pb + lq * kMfLdv + 4 * rg);
        pp[0] = e[0] | ((uint32_t)e[1] << 16), pp[1] = e[2] | ((uint32_t)e[3] << 16);
      }
      __syncthreads ();
      bf8 pf[4];
#pragma unroll
      for (int ks = 0; ks < 4; ++ks)
        pf[ks] = *(const bf8 *)(Pb + lq * kMfLdv + 16 * ks + 8 * hh);
#pragma unroll
      for (int b = 0; b < NB; ++b)
        {
          const int db = wave + kMfWaves * b;
          if (NBLK % kMfWaves != 0 && db >= NBLK)
            continue;
          const int d = 32 * db + lq;
          const uint16_t *vp = Vt + d * kMfLdv;
#pragma unroll
          for (int ks = 0; ks < 4; ++ks)
            oacc[b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16 (
                *(const bf8 *)(vp + (((2 * ks + hh) ^ swizzle (d >> 3)) << 3)), pf[ks], oacc[b], 0, 0, 0);
        }
  };
  for (int lb = l0; lb < l1; lb += 2 * kMfRows)
    {
      tile (lb, ra);
      if (lb + kMfRows < l1)
        tile (lb + kMfRows, rb);
    }
  // the sums of a head's row groups
  red[rg * 32 + lq] = sum;
  __syncthreads ();
  sum = 0.f;
#pragma unroll
  for (int i = 0; i < 16; ++i)
    sum += red[i * 32 + lq];
  const size_t pbase = ((size_t)s * gridDim.y + gt) * a.nsplit;
  const bool direct = a.cnt && active == 1;
  const float inv = direct ? 1.0f / sum : 1.0f;
  if (lq < nh)
    {
      if (!direct && wave == 0 && hh == 0)
        {
          const size_t at = (pbase + c) * ht + lq;
          if (a.cnt)
            {
              st_coherent_u32 ((uint32_t *)a.pm + at, __float_as_uint (m));
              st_coherent_u32 ((uint32_t *)a.pl + at, __float_as_uint (sum));
            }
          else
            stg (a.pm + at, m), stg (a.pl + at, sum);
        }
#pragma unroll
      for (int b = 0; b < NB; ++b)
        {
          const int db = wave + kMfWaves * b;
          if (NBLK % kMfWaves != 0 && db >= NBLK)
            continue;
#pragma unroll
          for (int q4 = 0; q4 < 4; ++q4)
            {
              const int d = 32 * db + 8 * q4 + 4 * hh;
              const float v[4] = { oacc[b][4 * q4] * inv, oacc[b][4 * q4 + 1] * inv, oacc[b][4 * q4 + 2] * inv,
                                   oacc[b][4 * q4 + 3] * inv };
              if (direct)
                {
#pragma unroll
                  for (int e = 0; e < 4; ++e)
                    store_elem (a.out, a.otype, (size_t)s * a.os + (size_t)(h0 + lq) * D + d + e, v[e]);
                  continue;
                }
              float *dst = a.pacc + ((pbase + c) * ht + lq) * D + d;
              if (a.cnt) // (through LDS, to leave it in whole lines)
                *(float4 *)((float *)lds_mf + lq * D + d) = make_float4 (v[0], v[1], v[2], v[3]);
              else
                stg ((vkl_u32x4 *)dst, vkl_u32x4{ __float_as_uint (v[0]), __float_as_uint (v[1]),
                                                  __float_as_uint (v[2]), __float_as_uint (v[3]) });
            }
        }
    }
  if (!a.cnt || active == 1)
    return;
  static_assert (32 * D * 4 <= kMfRows * LDK * 2 + D * kMfLdv * 2, "a part fits over the tile");
  __syncthreads ();
  for (int o = tid * 4; o < nh * D; o += kMfThreads * 4)
    {
      const float4 w = *(const float4 *)((const float *)lds_mf + o);
      const float v[4] = { w.x, w.y, w.z, w.w };
      st_coherent_16 (a.pacc + (pbase + c) * ht * D + o, v);
    }
  // (the flag lies behind what combine_parts uses of LDS)
  uint32_t *flag = (uint32_t *)((float *)lds_mf + combine_lds<kMfThreads> ());
  if (!last_of_parts (a.cnt + ((size_t)s * gridDim.y + gt) * kRowCounterStride, active, flag))
    return;
  combine_parts<kMfThreads> (a, ht, nh, active, pbase, (size_t)s * a.os + (size_t)h0 * D, (float *)lds_mf);
}

template <int NBLK>
int
launch_mfma_k (const RowAttnArgs &a, dim3 grid, hipStream_t s)
{
  static LdsLimit limit;
  constexpr size_t lds = mfma_rows_lds<NBLK> ();
  if (int e = limit.raise ((const void *)attn_rows_mfma_kernel<NBLK>, lds))
    return e;
  attn_rows_mfma_kernel<NBLK><<<grid, dim3 (kMfThreads), lds, s>>> (a);
  return (int)hipGetLastError ();
}

int
launch_mfma (const RowAttnArgs &a, dim3 grid, hipStream_t s)
{
  switch (a.D / 32)
    {
    case 1: return launch_mfma_k<1> (a, grid, s);
    case 2: return launch_mfma_k<2> (a, grid, s);
    case 3: return launch_mfma_k<3> (a, grid, s);
    case 4: return launch_mfma_k<4> (a, grid, s);
    case 5: return launch_mfma_k<5> (a, grid, s);
    case 6: return launch_mfma_k<6> (a, grid, s);
    case 7: return launch_mfma_k<7> (a, grid, s);
    case 8: return launch_mfma_k<8> (a, grid, s);
    case 10: return launch_mfma_k<10> (a, grid, s);
    case 12: return launch_mfma_k<12> (a, grid, s);
    case 14: return launch_mfma_k<14> (a, grid, s);
    case 16: return launch_mfma_k<16> (a, grid, s);
    default: return (int)hipErrorInvalidValue;
    }
}

template <typename CT, int LPR, int NCH, int HT, bool VALS>
int
launch_rows_k (const RowAttnArgs &a, dim3 grid, hipStream_t s)
{
  static LdsLimit limit;
  const size_t lds = sizeof (float) * std::max ((size_t)kRowThreads * 8 * NCH * HT, (size_t)combine_lds<kRowThreads> ());
  if (int e = limit.raise ((const void *)attn_rows_kernel<CT, LPR, NCH, HT, VALS>, lds))
    return e;
  attn_rows_kernel<CT, LPR, NCH, HT, VALS><<<grid, dim3 (kRowThreads), lds, s>>> (a);
  return (int)hipGetLastError ();
}

template <typename CT, int LPR, int NCH, bool VALS>
int
launch_rows_ht (const RowAttnArgs &a, int ht, dim3 grid, hipStream_t s)
{
  switch (ht)
    {
    case 1: return launch_rows_k<CT, LPR, NCH, 1, VALS> (a, grid, s);
    case 2: return launch_rows_k<CT, LPR, NCH, 2, VALS> (a, grid, s);
    case 4: return launch_rows_k<CT, LPR, NCH, 4, VALS> (a, grid, s);
    default:
      if constexpr (LPR <= 32)
        return launch_rows_k<CT, LPR, NCH, 8, VALS> (a, grid, s);
      return (int)hipErrorInvalidValue;
    }
}

template <typename CT, bool VALS>
int
launch_rows (const RowAttnArgs &a, int ht, dim3 grid, hipStream_t s)
{
  if (a.D <= 32)
    return launch_rows_ht<CT, 4, 1, VALS> (a, ht, grid, s);
  if (a.D <= 64)
    return launch_rows_ht<CT, 8, 1, VALS> (a, ht, grid, s);
  if (a.D <= 128)
    return launch_rows_ht<CT, 16, 1, VALS> (a, ht, grid, s);
  if (a.D <= 256)
    return launch_rows_ht<CT, 32, 1, VALS> (a, ht, grid, s);
  if (a.D <= 512)
    return launch_rows_ht<CT, 64, 1, VALS> (a, ht, grid, s);
  return launch_rows_ht<CT, 64, 2, VALS> (a, ht, grid, s);
}

size_t
row_scratch_bytes (int ctype, int H, int G, int D, int S, bool vals = false)
{
  const RowPlan p = row_plan (ctype, H, G, D, S, vals);
  return kRowCounterBytes + p.parts * (2 + (size_t)D) * sizeof (float) + 256;
}

// the parts of a launch that leaves them to the next one
struct RowParts
{
  const float *pm, *pl, *pacc;
  int nsplit, ht, tiles, step; // tiles: head tiles of ht heads each (one group)
};

// rows a workgroup takes at a time (STEP of the kernel)
int
row_step (int D)
{
  const int lpr = D <= 32 ? 4 : D <= 64 ? 8 : D <= 128 ? 16 : D <= 256 ? 32 : 64;
  return 4 * (64 / lpr) * kRowUnroll;
}

// an attention launch over p: the plan and the scratch area fill in the rest
int
rows_launch (RowAttnArgs a, int ctype, int H, int S, void *scratch, RowParts *parts, hipStream_t s)
{
  const RowPlan p = row_plan (ctype, H, a.G, a.D, S, a.vals != nullptr);
  a.rep = H / a.G, a.tiles = p.tiles, a.ht = p.ht, a.nsplit = p.nsplit;
  a.cnt = parts ? nullptr : (uint32_t *)scratch;
  a.pm = (float *)((uint8_t *)scratch + kRowCounterBytes);
  a.pl = a.pm + p.parts;
  a.pacc = a.pl + p.parts;
  if (parts)
    *parts = { a.pm, a.pl, a.pacc, p.nsplit, p.ht, p.tiles, p.mfma ? kMfRows : row_step (a.D) };
  const dim3 grid ((unsigned)p.nsplit, (unsigned)(a.G * p.tiles), (unsigned)S);
  if (p.mfma)
    return launch_mfma (a, grid, s);
  if (a.vals)
    return ctype == VKL_TYPE_F32 ? launch_rows<float, true> (a, p.ht, grid, s)
                                 : launch_rows<uint16_t, true> (a, p.ht, grid, s);
  return ctype == VKL_TYPE_F32 ? launch_rows<float, false> (a, p.ht, grid, s)
                               : launch_rows<uint16_t, false> (a, p.ht, grid, s);
}

int
rows_attention (const void *q, int qtype, size_t qs, const void *rows, int ctype, size_t rs, int H, int G, int D,
                int S, StepPos pos, float scale, float tcoef, int tevery, void *out, int otype, size_t os,
                void *scratch, RowParts *parts, hipStream_t s)
{
  RowAttnArgs a = {};
  a.q = q, a.qtype = qtype, a.qs = qs, a.rows = rows, a.rs = rs, a.G = G, a.D = D;
  a.pos = pos, a.scale = scale, a.tcoef = tcoef, a.tevery = tevery;
  a.out = out, a.otype = otype, a.os = os;
  return rows_launch (a, ctype, H, S, scratch, parts, s);
}

// keys and values of their own
int
kv_attention (const void *q, int qtype, size_t qs, const void *rows, const void *vals, int ctype, size_t rs, int H,
              int G, int D, int S, StepPos pos, float scale, int chunk, int sink, void *out, int otype, size_t os,
              void *scratch, hipStream_t s)
{
  RowAttnArgs a = {};
  a.q = q, a.qtype = qtype, a.qs = qs, a.rows = rows, a.vals = vals, a.rs = rs, a.G = G, a.D = D;
  a.pos = pos, a.scale = scale, a.chunk = chunk, a.sink = sink;
  a.out = out, a.otype = otype, a.os = os;
  return rows_launch (a, ctype, H, S, scratch, nullptr, s);
}

// ---------------------------------------------------------------------------
// queries, keys and values between their projections and the attention
// ---------------------------------------------------------------------------
constexpr int kPrepMax = 1024; // values of a head at most

struct PrepArgs
{
  vkl_attn_rows_prep p;
  StepPos pos;
  int S;
};

// A workgroup takes `run` heads of a token, of the query heads, the keys and the
// values in a row; sines and cosines of the position are shared.  A wave per head.
__global__ __launch_bounds__ (256) void
attn_prepare_kernel (const PrepArgs a, int run, int runs)
{
  __shared__ float cs[kPrepMax / 2], sn[kPrepMax / 2];
  const vkl_attn_rows_prep &p = a.p;
  const int per = p.H + 2 * p.G, lane = threadIdx.x & 63;
  const int s = blockIdx.x / runs, first = (blockIdx.x - s * runs) * run;
  const size_t pos = (size_t)a.pos.get () + (size_t)s, crow = pos * (size_t)p.G * p.dim;
  for (int i = threadIdx.x; i < p.npair; i += 256)
    {
      // the angle to within a turn in double, its sine and cosine in float
      double t = (double)pos * ldg (p.freq + i) * 0.15915494309189533577;
      t -= rint (t);
      sincosf ((float)(t * 6.28318530717958647693), sn + i, cs + i);
    }
  __syncthreads ();
  for (int part = first + (threadIdx.x >> 6); part < min (first + run, per); part += 4)
    {
      if (part >= p.H + p.G)
        {
          const int g = part - p.H - p.G;
          if (!p.v)
            continue;
          const size_t at = crow + (size_t)g * p.dim;
          for (int c = lane; c < p.dim; c += 64)
            {
              float v = load_elem (p.v, p.kvtype, (size_t)s * p.kvs + (size_t)g * p.dim + c);
              if (p.first)
                v = (1.0f - p.mix) * v
                    + (c < p.fdim ? p.mix * load_elem (p.first, p.ctype, (pos * p.G + g) * p.fdim + c) : 0.f);
              store_elem (p.vo, p.ctype, at + c, v);
            }
          continue;
        }
      const bool key = part >= p.H;
      const void *src = key ? p.k : p.q;
      if (!src)
        continue;
      const int type = key ? p.kvtype : p.qtype, h = key ? part - p.H : part;
      const size_t at = (size_t)s * (key ? p.kvs : p.qs) + (size_t)h * p.dim;
      float x[kPrepMax / 64], ss = 0.f;
#pragma unroll
      for (int j = 0; j < kPrepMax / 64; ++j)
        {
          const int c = lane + 64 * j;
          x[j] = 0.f;
          if (64 * j >= p.dim || c >= p.n)
            continue;
          const float v = load_elem (src, type, at + c);
          x[j] = v;
          if (c < 2 * p.npair)
            {
              const bool low = c < p.npair;
              const int i = low ? c : c - p.npair;
              const float w = load_elem (src, type, at + (low ? c + p.npair : i));
              x[j] = low ? v * cs[i] - w * sn[i] : v * cs[i] + w * sn[i];
            }
          ss = __builtin_fmaf (x[j], x[j], ss);
        }
      const float alpha = 1.0f / sqrtf (wave_sum (ss) / (float)p.n + p.eps);
#pragma unroll
      for (int j = 0; j < kPrepMax / 64; ++j)
        {
          const int c = lane + 64 * j;
          if (64 * j >= p.dim || c >= p.dim)
            continue;
          if (key)
            store_elem (p.ko, p.ctype, crow + (size_t)h * p.dim + c, x[j] * alpha);
          else
            store_elem (p.qo, p.qotype, (size_t)s * p.qos + (size_t)h * p.dim + c, x[j] * alpha);
        }
    }
}

// The same in vectors: LPH lanes per head, eight neighbouring values each; heads of up
// to 8 LPH values, pairs and strides multiples of eight.
__device__ __forceinline__ void
store8 (void *p, int type, size_t i, const float (&f)[8])
{
  if (type == VKL_TYPE_F32)
    {
      vkl_u32x4 w[2];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        w[e >> 2][e & 3] = __float_as_uint (f[e]);
      stg ((vkl_u32x4 *)((float *)p + i), w[0]), stg ((vkl_u32x4 *)((float *)p + i + 4), w[1]);
      return;
    }
  vkl_u32x4 w;
#pragma unroll
  for (int e = 0; e < 4; ++e)
    w[e] = f2bf (f[2 * e]) | ((uint32_t)f2bf (f[2 * e + 1]) << 16);
  stg ((vkl_u32x4 *)((uint16_t *)p + i), w);
}

template <int LPH>
__global__ __launch_bounds__ (256) void
attn_prepare_vec_kernel (const PrepArgs a, int runs)
{
  constexpr int HPW = 256 / LPH; // heads of a workgroup
  __shared__ __align__ (16) float cs[LPH * 4], sn[LPH * 4];
  const vkl_attn_rows_prep &p = a.p;
  const int per = p.H + 2 * p.G, sub = threadIdx.x % LPH, c = 8 * sub;
  const int s = blockIdx.x / runs, part = (blockIdx.x - s * runs) * HPW + (int)threadIdx.x / LPH;
  const size_t pos = (size_t)a.pos.get () + (size_t)s, crow = pos * (size_t)p.G * p.dim;
  const bool value = part >= p.H + p.G, key = !value && part >= p.H;
  const int h = value ? part - p.H - p.G : key ? part - p.H : part;
  const void *src = value ? p.v : key ? p.k : p.q;
  const int type = value || key ? p.kvtype : p.qtype;
  const bool live = part < per && src && c < p.dim;
  const size_t at = (size_t)s * (value || key ? p.kvs : p.qs) + (size_t)h * p.dim + c, cat = crow + (size_t)h * p.dim + c;
  const bool turned = c < 2 * p.npair, low = c < p.npair;
  float x[8] = {}, y[8] = {};
  if (live)
    {
      load8 (src, type, at, x);
      if (value && p.first && c < p.fdim)
        load8 (p.first, p.ctype, (pos * p.G + h) * p.fdim + c, y);
      else if (!value && turned)
        load8 (src, type, low ? at + p.npair : at - p.npair, y);
    }
  if ((int)threadIdx.x < p.npair)
    {
      // the angle to within a turn in double, its sine and cosine in float
      double t = (double)pos * ldg (p.freq + threadIdx.x) * 0.15915494309189533577;
      t -= rint (t);
      sincosf ((float)(t * 6.28318530717958647693), sn + threadIdx.x, cs + threadIdx.x);
    }
  __syncthreads ();
  if (value)
    {
      if (!live)
        return;
      if (p.first)
#pragma unroll
        for (int e = 0; e < 8; ++e)
          x[e] = (1.0f - p.mix) * x[e] + p.mix * y[e];
      store8 (p.vo, p.ctype, cat, x);
      return;
    }
  float ss = 0.f;
  const int i0 = turned ? (low ? c : c - p.npair) : 0;
#pragma unroll
  for (int e = 0; e < 8; ++e)
    {
      if (turned)
        x[e] = low ? x[e] * cs[i0 + e] - y[e] * sn[i0 + e] : x[e] * cs[i0 + e] + y[e] * sn[i0 + e];
      x[e] = c + e < p.n ? x[e] : 0.f;
      ss = __builtin_fmaf (x[e], x[e], ss);
    }
  const float alpha = 1.0f / sqrtf (lanes_sum<LPH> (ss) / (float)p.n + p.eps);
  if (!live)
    return;
#pragma unroll
  for (int e = 0; e < 8; ++e)
    x[e] *= alpha;
  if (key)
    store8 (p.ko, p.ctype, cat, x);
  else
    store8 (p.qo, p.qotype, (size_t)s * p.qos + (size_t)h * p.dim + c, x);
}

template <int LPH>
void
launch_prepare_vec (const PrepArgs &a, hipStream_t s)
{
  const int runs = (a.p.H + 2 * a.p.G + 256 / LPH - 1) / (256 / LPH);
  attn_prepare_vec_kernel<LPH><<<dim3 ((unsigned)(a.S * runs)), dim3 (256), 0, s>>> (a, runs);
}

int
attn_prepare (const vkl_attn_rows_prep &p, int S, StepPos pos, hipStream_t s)
{
  PrepArgs a = { p, pos, S };
  uintptr_t mis = 0;
  for (const void *q : { p.q, (const void *)p.qo, p.k, p.v, (const void *)p.ko, (const void *)p.vo, p.first })
    mis |= (uintptr_t)q % 16;
  if (p.dim % 8 == 0 && p.fdim % 8 == 0 && p.dim <= 256 && p.npair % 8 == 0 && p.qs % 8 == 0 && p.qos % 8 == 0 && p.kvs % 8 == 0 && !mis)
    {
      if (p.dim <= 32)
        launch_prepare_vec<4> (a, s);
      else if (p.dim <= 64)
        launch_prepare_vec<8> (a, s);
      else if (p.dim <= 128)
        launch_prepare_vec<16> (a, s);
      else
        launch_prepare_vec<32> (a, s);
      return (int)hipGetLastError ();
    }
  const int per = p.H + 2 * p.G, run = S < 64 ? 4 : 16, runs = (per + run - 1) / run;
  attn_prepare_kernel<<<dim3 ((unsigned)(S * runs)), dim3 (256), 0, s>>> (a, run, runs);
  return (int)hipGetLastError ();
}

// ---------------------------------------------------------------------------
// one small matrix per head
// ---------------------------------------------------------------------------
struct HeadArgs
{
  const uint16_t *w;
  int R, K, bph; // bph: workgroups per head
  int heads;
  const void *x;
  int xtype;
  size_t xs, xh;
  void *y;
  int ytype;
  size_t ys, yh;
  const float *gate;
  size_t gs;
  // an extra workgroup norms a row of fp32 values into a cache row (the new
  // token's latent), null: none
  const float *nx;
  const float *nw;
  int nW, nWp;
  float neps;
  void *ncache;
  int ntype;
  StepPos pos;
  // x as the parts an attention launch left (one token): combined here
  RowParts parts;
};

constexpr int kHeadRows = 4; // row groups per wave

template <int LPR, bool PARTS>
__global__ __launch_bounds__ (256) void
head_matvec_kernel (const HeadArgs a)
{
  __shared__ float red[8];
  __shared__ __align__ (16) float xc[PARTS ? 1024 : 4];
  __shared__ float wgt[kRowSplits];
  const int tid = threadIdx.x, wave = tid >> 6, lane = tid & 63;
  if ((int)blockIdx.x == a.heads * a.bph)
    {
      float ss = 0.f;
      for (int c = tid; c < a.nW; c += 256)
        {
          const float v = ldg (a.nx + c);
          ss = __builtin_fmaf (v, v, ss);
        }
      const float alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.nW + a.neps);
      const size_t o = (size_t)a.pos.get () * a.nWp;
      for (int c = tid; c < a.nWp; c += 256)
        store_elem (a.ncache, a.ntype, o + c, c < a.nW ? ldg (a.nx + c) * alpha * ldg (a.nw + c) : 0.f);
      return;
    }
  // (a head's workgroups are numbered so that, with a multiple of 8 heads, they
  // share an XCD and what they read of the head)
  const int h = blockIdx.x % a.heads, b = blockIdx.x / a.heads, s = blockIdx.y;
  constexpr int RPW = 64 / LPR;
  const int sub = lane % LPR, grp = lane / LPR;
  const int r0 = (b * 4 + wave) * RPW * kHeadRows + grp; // rows r0 + i * RPW
  const uint16_t *w = a.w + (size_t)h * a.R * a.K;
  const size_t xo = (size_t)s * a.xs + (size_t)h * a.xh;
  if constexpr (PARTS)
    {
      const RowParts &p = a.parts;
      const int L = (int)a.pos.get () + 1;
      const int chunk = row_chunk (L, p.nsplit, p.step), active = (L + chunk - 1) / chunk;
      const size_t pbase = (size_t)(h / p.ht) * p.nsplit;
      const int hh = h % p.ht;
      // lane p holds part p
      static_assert (kRowSplits == 64, "one part per lane");
      const size_t at = (pbase + min (lane, active - 1)) * p.ht + hh;
      const float mi = ldg (p.pm + at), li = ldg (p.pl + at);
      const float M = wave_max (mi);
      const float f = lane < active ? expf (mi - M) : 0.f;
      const float S = wave_sum (f * li);
      if (wave == 0)
        wgt[lane] = f / S;
      __syncthreads ();
      const int half = tid >> 7;
      for (int k0 = 0; k0 < a.K; k0 += 512)
        {
          // four neighbouring values per thread, the parts in two halves of the workgroup
          const int k = k0 + (tid & 127) * 4, kc = min (k, a.K - 4);
          const float *src = p.pacc + (pbase * p.ht + hh) * a.K + kc;
          float4 v = make_float4 (0.f, 0.f, 0.f, 0.f);
          for (int p0 = 0; p0 < active; p0 += 32)
            {
              float4 pv[16];
#pragma unroll
              for (int j = 0; j < 16; ++j)
                pv[j] = __builtin_bit_cast (float4, ldg4 (src + (size_t)min (p0 + 2 * j + half, active - 1) * p.ht * a.K));
#pragma unroll
              for (int j = 0; j < 16; ++j)
                {
                  const float g = wgt[p0 + 2 * j + half];
                  v.x = __builtin_fmaf (g, pv[j].x, v.x), v.y = __builtin_fmaf (g, pv[j].y, v.y);
                  v.z = __builtin_fmaf (g, pv[j].z, v.z), v.w = __builtin_fmaf (g, pv[j].w, v.w);
                }
            }
          if (half && k < a.K)
            *(float4 *)(xc + k) = v;
          __syncthreads ();
          if (!half && k < a.K)
            {
              const float4 w = *(const float4 *)(xc + k);
              *(float4 *)(xc + k) = make_float4 (v.x + w.x, v.y + w.y, v.z + w.z, v.w + w.w);
            }
        }
      __syncthreads ();
    }
  float acc[kHeadRows] = {};
  for (int k0 = 0; k0 < a.K; k0 += LPR * 8)
    {
      const int k = k0 + sub * 8, kc = min (k, a.K - 8);
      uint4 wv[kHeadRows];
#pragma unroll
      for (int i = 0; i < kHeadRows; ++i)
        wv[i] = ldg4 (w + (size_t)min (r0 + i * RPW, a.R - 1) * a.K + kc);
      float xv[8];
      if constexpr (PARTS)
        {
#pragma unroll
          for (int e = 0; e < 8; ++e)
            xv[e] = xc[kc + e];
        }
      else
        load8 (a.x, a.xtype, xo + kc, xv);
      if (k >= a.K)
#pragma unroll
        for (int e = 0; e < 8; ++e)
          xv[e] = 0.f;
#pragma unroll
      for (int i = 0; i < kHeadRows; ++i)
        {
          float f[8];
          widen8 (wv[i], f);
#pragma unroll
          for (int e = 0; e < 8; ++e)
            acc[i] = __builtin_fmaf (f[e], xv[e], acc[i]);
        }
    }
  const float f = a.gate ? sigmoid (ldg (a.gate + (size_t)s * a.gs + h)) : 1.0f;
#pragma unroll
  for (int i = 0; i < kHeadRows; ++i)
    {
      const float v = lanes_sum<LPR> (acc[i]);
      if (sub == 0 && r0 + i * RPW < a.R)
        store_elem (a.y, a.ytype, (size_t)s * a.ys + (size_t)h * a.yh + r0 + i * RPW, v * f);
    }
}

int
head_matvec (HeadArgs a, int S, hipStream_t s)
{
  const int lpr = a.K <= 32 ? 4 : a.K <= 64 ? 8 : a.K <= 128 ? 16 : a.K <= 256 ? 32 : 64;
  const int rows = 4 * (64 / lpr) * kHeadRows;
  a.bph = (a.R + rows - 1) / rows;
  const dim3 grid ((unsigned)(a.heads * a.bph + (a.nx ? 1 : 0)), (unsigned)S), block (256);
#define VKL_HEAD(L)                                                           \
  if (a.parts.pacc)                                                           \
    head_matvec_kernel<L, true><<<grid, block, 0, s>>> (a);                   \
  else                                                                        \
    head_matvec_kernel<L, false><<<grid, block, 0, s>>> (a);                  \
  break
  switch (lpr)
    {
    case 4: VKL_HEAD (4);
    case 8: VKL_HEAD (8);
    case 16: VKL_HEAD (16);
    case 32: VKL_HEAD (32);
    default: VKL_HEAD (64);
    }
#undef VKL_HEAD
  return (int)hipGetLastError ();
}

// ---------------------------------------------------------------------------
// the weight-streaming product of the step
// ---------------------------------------------------------------------------
constexpr int kGvThreads = 512, kGvWaves = 8;
enum
{
  GV_SEGS = 0,  // outputs by segment
  GV_ADD = 1,   // y[n] += sum
  GV_LOGITS = 2, // y[n] = soft cap, arg-max partials
  GV_GATED = 3   // GV_ADD of a row that is normed and gated on the way in
};

// an item: 8 loads of 512 columns per lane; two rows of four, or, where rows are
// few and long, one row of eight (every wave then has a row of its own)
template <int MODE>
constexpr int
gv_rows ()
{
  return MODE == GV_ADD || MODE == GV_GATED ? 1 : 2;
}
template <int MODE>
constexpr int
gv_span ()
{
  return 8 / gv_rows<MODE> () * 512;
}

struct GvSeg
{
  int n0, n;
  void *y;
  int f32, act;
  size_t pos_stride; // y moves by this per position (a cache row)
};

struct GvArgs
{
  const uint16_t *w;
  int N, K;
  const float *x;    // [K]
  const float *norm; // [K] (zero beyond W), RMS norm over W values
  const float *gate; // GV_GATED: times sigmoid (gate[c])
  int W;
  float eps;
  int nseg;
  GvSeg seg[kGemmSegs];
  StepPos pos;
  float *y;
  float cap;
  // arg-max: partials [grid] of (value, id), the counter, where the id goes
  float *amax_v;
  uint32_t *amax_i, *amax_cnt;
  uint32_t *next_tok; // optional
  uint32_t *loop, *ids; // replayed loop: ids[index + 1], then both words advance
  int pick;
  bool stream; // see NT of the kernel
};

__device__ __forceinline__ bool
amax_better (float v, uint32_t i, float bv, uint32_t bi)
{
  return v > bv || (v == bv && i < bi);
}

// XV: float4 per thread that hold the activation row while the first weights
// are requested; 0: a row of any length, staged before them
// NT: the weights of a step exceed what the caches hold, they are requested past
// them
template <int MODE, int XV, bool NT>
__global__ __launch_bounds__ (kGvThreads) void
stack_gemv_kernel (const GvArgs a)
{
  // column c of the row: block c / 512, first or second half of lane (c % 512) / 8
  extern __shared__ __align__ (16) float xl[];
  __shared__ float red[16];
  __shared__ float bv_s[kGvWaves];
  __shared__ uint32_t bi_s[kGvWaves + 1];
  constexpr bool NORM = MODE != GV_ADD, GATE = MODE == GV_GATED;
  constexpr int ROWS = gv_rows<MODE> (), STEPS = 8 / ROWS, SPAN = gv_span<MODE> ();
  const int tid = threadIdx.x, lane = tid & 63;
  const int wave = __builtin_amdgcn_readfirstlane (tid >> 6);
  const int nspan = (a.K + SPAN - 1) / SPAN;
  const int units = (a.N + ROWS - 1) / ROWS;
  const int w0 = blockIdx.x * kGvWaves + wave, nw = gridDim.x * kGvWaves;
  const int mine = w0 < units ? (units - w0 + nw - 1) / nw : 0;
  const int items = mine * nspan;

  uint4 bufa[8], bufb[8];
  auto issue = [&] (int it, uint4 (&b)[8]) {
    const int ic = min (it, max (items - 1, 0));
    const int un = ic / nspan, sp = ic - un * nspan;
    const int row0 = min (w0 + un * nw, units - 1) * ROWS;
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
      {
        const uint16_t *p = a.w + (size_t)min (row0 + r, a.N - 1) * a.K;
#pragma unroll
        for (int u = 0; u < STEPS; ++u)
          {
            const uint16_t *c = p + min (sp * SPAN + u * 512 + lane * 8, a.K - 8);
            b[r * STEPS + u] = NT ? ldg4_stream (c) : ldg4 (c);
          }
      }
  };
  auto put = [&] (int c, const float4 v) { // c: a multiple of 4
    const int o = (c >> 9) * 512 + ((c >> 2) & 1) * 256 + ((c & 511) >> 3) * 4;
    *(float4 *)(xl + o) = v;
  };
  const int kpad = nspan * SPAN;
  if constexpr (XV > 0)
    {
      float4 xv[XV], nv[XV], gv[XV];
#pragma unroll
      for (int j = 0; j < XV; ++j)
        {
          const int c = min ((tid + j * kGvThreads) * 4, a.K - 4);
          xv[j] = __builtin_bit_cast (float4, ldg4 (a.x + c));
          if (NORM)
            nv[j] = __builtin_bit_cast (float4, ldg4 (a.norm + c));
          if (GATE)
            gv[j] = __builtin_bit_cast (float4, ldg4 (a.gate + c));
        }
      __builtin_amdgcn_sched_barrier (0);
      issue (0, bufa);
      __builtin_amdgcn_sched_barrier (0);
      float alpha = 1.f;
      if (NORM)
        {
          float ss = 0.f;
#pragma unroll
          for (int j = 0; j < XV; ++j)
            if ((tid + j * kGvThreads) * 4 < a.K)
              {
                ss = __builtin_fmaf (xv[j].x, xv[j].x, ss), ss = __builtin_fmaf (xv[j].y, xv[j].y, ss);
                ss = __builtin_fmaf (xv[j].z, xv[j].z, ss), ss = __builtin_fmaf (xv[j].w, xv[j].w, ss);
              }
          alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.W + a.eps);
        }
#pragma unroll
      for (int j = 0; j < XV; ++j)
        {
          const int c = (tid + j * kGvThreads) * 4;
          float4 v = xv[j];
          if (NORM)
            {
              v.x = v.x * alpha * nv[j].x, v.y = v.y * alpha * nv[j].y;
              v.z = v.z * alpha * nv[j].z, v.w = v.w * alpha * nv[j].w;
            }
          if (GATE)
            v.x *= sigmoid (gv[j].x), v.y *= sigmoid (gv[j].y), v.z *= sigmoid (gv[j].z), v.w *= sigmoid (gv[j].w);
          if (c >= a.K)
            v = make_float4 (0.f, 0.f, 0.f, 0.f);
          if (c < kpad)
            put (c, v);
        }
    }
  else
    {
      float alpha = 1.f;
      if (NORM)
        {
          float ss = 0.f;
          for (int c = tid; c < a.K; c += kGvThreads)
            {
              const float v = ldg (a.x + c);
              ss = __builtin_fmaf (v, v, ss);
            }
          alpha = 1.0f / sqrtf (group_sum (ss, red) / (float)a.W + a.eps);
        }
      for (int c = tid * 4; c < kpad; c += kGvThreads * 4)
        {
          float4 v = make_float4 (0.f, 0.f, 0.f, 0.f);
          if (c < a.K)
            {
              v = __builtin_bit_cast (float4, ldg4 (a.x + c));
              if (NORM)
                {
                  const float4 n = __builtin_bit_cast (float4, ldg4 (a.norm + c));
                  v.x = v.x * alpha * n.x, v.y = v.y * alpha * n.y;
                  v.z = v.z * alpha * n.z, v.w = v.w * alpha * n.w;
                }
              if (GATE)
                {
                  const float4 g = __builtin_bit_cast (float4, ldg4 (a.gate + c));
                  v.x *= sigmoid (g.x), v.y *= sigmoid (g.y), v.z *= sigmoid (g.z), v.w *= sigmoid (g.w);
                }
            }
          put (c, v);
        }
      issue (0, bufa);
    }
  __syncthreads ();

  const uint32_t pos = MODE == GV_SEGS ? a.pos.get () : 0u;
  float sum[ROWS];
#pragma unroll
  for (int r = 0; r < ROWS; ++r)
    sum[r] = 0.f;
  float best_v = -INFINITY;
  uint32_t best_i = 0xffffffffu;
  auto compute = [&] (int it, const uint4 (&b)[8]) {
    const int un = it / nspan, sp = it - un * nspan;
#pragma unroll
    for (int u = 0; u < STEPS; ++u)
      {
        const float *xp = xl + (sp * STEPS + u) * 512 + lane * 4;
        const float4 x0 = *(const float4 *)xp, x1 = *(const float4 *)(xp + 256);
        const float xv[8] = { x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w };
#pragma unroll
        for (int r = 0; r < ROWS; ++r)
          {
            float f[8];
            widen8 (b[r * STEPS + u], f);
#pragma unroll
            for (int e = 0; e < 8; ++e)
              sum[r] = __builtin_fmaf (f[e], xv[e], sum[r]);
          }
      }
    if (sp != nspan - 1)
      return;
    const int row0 = (w0 + un * nw) * ROWS;
#pragma unroll
    for (int r = 0; r < ROWS; ++r)
      {
        float v = wave_sum (sum[r]);
        sum[r] = 0.f;
        const int n = row0 + r;
        if (n >= a.N)
          continue;
        if (MODE == GV_ADD || MODE == GV_GATED)
          {
            if (lane == 0)
              stg (a.y + n, ldg (a.y + n) + v);
          }
        else if (MODE == GV_LOGITS)
          {
            if (a.cap > 0.f)
              v = a.cap * tanhf (v / a.cap);
            if (lane == 0)
              stg (a.y + n, v);
            if (amax_better (v, (uint32_t)n, best_v, best_i))
              best_v = v, best_i = (uint32_t)n;
          }
        else
          {
#pragma unroll
            for (int i = 0; i < kGemmSegs; ++i)
              if (i < a.nseg && n >= a.seg[i].n0 && n < a.seg[i].n0 + a.seg[i].n)
                {
                  const GvSeg &sg = a.seg[i];
                  const float y = activate (sg.act, v);
                  if (lane == 0)
                    store_elem (sg.y, sg.f32 ? VKL_TYPE_F32 : VKL_TYPE_BF16,
                                (size_t)pos * sg.pos_stride + (n - sg.n0), y);
                }
          }
      }
  };
  // (no branch around a request inside the loop: the waits then count exactly; the
  // last one or two items stand behind it)
  int it = 0;
  for (; it + 2 < items; it += 2)
    {
      issue (it + 1, bufb);
      compute (it, bufa);
      issue (it + 2, bufa);
      compute (it + 1, bufb);
    }
  if (it + 1 < items)
    {
      issue (it + 1, bufb);
      compute (it, bufa);
      compute (it + 1, bufb);
    }
  else if (it < items)
    compute (it, bufa);
  if (MODE != GV_LOGITS || !a.pick)
    return;
  // arg-max: the workgroup's best, then the last workgroup over all of them
  if (lane == 0)
    bv_s[wave] = best_v, bi_s[wave] = best_i;
  __syncthreads ();
  if (tid == 0)
    {
      for (int i = 1; i < kGvWaves; ++i)
        if (amax_better (bv_s[i], bi_s[i], best_v, best_i))
          best_v = bv_s[i], best_i = bi_s[i];
      st_coherent_u32 ((uint32_t *)a.amax_v + blockIdx.x, __float_as_uint (best_v));
      st_coherent_u32 (a.amax_i + blockIdx.x, best_i);
      __builtin_amdgcn_s_waitcnt (0);
      const uint32_t old = __hip_atomic_fetch_add (a.amax_cnt, 1u, __ATOMIC_RELAXED, __HIP_MEMORY_SCOPE_AGENT);
      const bool last = old + 1u == gridDim.x;
      if (last)
        st_coherent_u32 (a.amax_cnt, 0u);
      bi_s[kGvWaves] = last ? 1u : 0u;
    }
  __syncthreads ();
  if (bi_s[kGvWaves] == 0u || tid >= 64)
    return;
  best_v = -INFINITY, best_i = 0xffffffffu;
  for (int i = lane; i < (int)gridDim.x; i += 64)
    {
      const float v = __uint_as_float (ld_coherent_u32 ((const uint32_t *)a.amax_v + i));
      const uint32_t id = ld_coherent_u32 (a.amax_i + i);
      if (amax_better (v, id, best_v, best_i))
        best_v = v, best_i = id;
    }
#pragma unroll
  for (int o = 32; o > 0; o >>= 1)
    {
      const float ov = __shfl_xor (best_v, o, 64);
      const uint32_t oi = __shfl_xor (best_i, o, 64);
      if (amax_better (ov, oi, best_v, best_i))
        best_v = ov, best_i = oi;
    }
  if (lane == 0)
    {
      const uint32_t id = best_i == 0xffffffffu ? 0u : best_i;
      if (a.next_tok)
        *a.next_tok = id;
      if (a.loop)
        {
          const uint32_t index = a.loop[0];
          a.ids[index + 1] = id;
          a.loop[0] = index + 1u, a.loop[1] += 1u;
        }
    }
}

constexpr int kGvMaxLds = 128 << 10;

bool
gv_supported (int K)
{
  return (size_t)((K + 4095) / 4096) * 4096 * sizeof (float) <= (size_t)kGvMaxLds; // (the longest span)
}

template <int MODE, int XV, bool NT>
int
launch_gv_nt (const GvArgs &a, int grid, size_t lds, hipStream_t s)
{
  static LdsLimit limit;
  if (int e = limit.raise ((const void *)stack_gemv_kernel<MODE, XV, NT>, lds))
    return e;
  stack_gemv_kernel<MODE, XV, NT><<<dim3 ((unsigned)grid), dim3 (kGvThreads), lds, s>>> (a);
  return (int)hipGetLastError ();
}

template <int MODE, int XV>
int
launch_gv_k (const GvArgs &a, int grid, size_t lds, hipStream_t s)
{
  return a.stream ? launch_gv_nt<MODE, XV, true> (a, grid, lds, s) : launch_gv_nt<MODE, XV, false> (a, grid, lds, s);
}

template <int MODE>
int
launch_gv (const GvArgs &a, int n_cu, hipStream_t s)
{
  if (!gv_supported (a.K))
    return (int)hipErrorInvalidValue;
  constexpr int SPAN = gv_span<MODE> ();
  const int units = (a.N + gv_rows<MODE> () - 1) / gv_rows<MODE> ();
  const int grid = std::min (2 * n_cu, (units + kGvWaves - 1) / kGvWaves);
  const size_t lds = (size_t)((a.K + SPAN - 1) / SPAN) * SPAN * sizeof (float);
  // (the loads of the row have to cover its padding to whole spans)
  if (SPAN == 2048 && a.K <= 2048)
    return launch_gv_k<MODE, 1> (a, grid, lds, s);
  if (a.K <= 4096)
    return launch_gv_k<MODE, 2> (a, grid, lds, s);
  if (a.K <= 8192)
    return launch_gv_k<MODE, 4> (a, grid, lds, s);
  if (a.K <= 16384)
    return launch_gv_k<MODE, 8> (a, grid, lds, s);
  return launch_gv_k<MODE, 0> (a, grid, lds, s);
}

// ---------------------------------------------------------------------------
// the step
// ---------------------------------------------------------------------------
struct StackScratch
{
  uint32_t *sync; // [0] arg-max counter, [16..17] loop state, [20..23] sampler parameters
  uint32_t *cnt;  // attention counters and parts
  float *x, *q, *c, *g, *cat, *qa, *ff, *logits, *amax_v;
  uint32_t *amax_i;
  size_t bytes;
};

constexpr int kMaxGrid = 2048;

size_t
round64 (int n)
{
  return ((size_t)n + 63) / 64 * 64;
}

StackScratch
carve_stack (const vkl_stack_model *m)
{
  StackScratch s = {};
  size_t q = 0, c = 0, g = 0, cat = 0, qa = 0, attn = 0, ff = 0;
  for (int i = 0; i < m->n_runs; ++i)
    {
      const vkl_stack_layer &l = m->layers_h[i];
      q = std::max (q, (size_t)l.H * l.dim);
      cat = std::max (cat, (size_t)l.k_out);
      ff = std::max (ff, (size_t)l.ff_p);
      if (l.mixer == VKL_MIX_KV)
        {
          c = std::max (c, (size_t)2 * l.G * l.dim);
          attn = std::max (attn, row_scratch_bytes (m->ctype, l.H, l.G, l.dim, 1, true));
        }
      else if (l.mixer == VKL_MIX_DELTA || l.mixer == VKL_MIX_DECAY)
        {
          c = std::max (c, (size_t)2 * l.G * l.dim + (size_t)l.H * l.vdim);
          g = std::max (g, l.mixer == VKL_MIX_DELTA ? round64 (l.H) + round64 (l.r_a) + round64 (l.r_g)
                                                    : (size_t)l.k_out);
        }
      else if (l.mixer == VKL_MIX_LATENT)
        {
          c = std::max (c, (size_t)l.rank_p), g = std::max (g, (size_t)l.H);
          qa = std::max (qa, (size_t)l.H * l.rank_p);
          attn = std::max (attn, row_scratch_bytes (m->ctype, l.H, 1, l.rank_p, 1));
        }
      else
        attn = std::max (attn, row_scratch_bytes (m->ctype, l.H, l.G, l.dim, 1));
    }
  uint8_t *base = (uint8_t *)m->scratch;
  size_t off = 0;
  auto take = [&] (size_t bytes) {
    uint8_t *p = base + off;
    off += (bytes + 255) / 256 * 256;
    return p;
  };
  s.sync = (uint32_t *)take (4096);
  s.cnt = (uint32_t *)take (attn);
  s.x = (float *)take ((size_t)m->width_p * 4);
  s.q = (float *)take (q * 4);
  s.c = (float *)take (c * 4);
  s.g = (float *)take (g * 4);
  s.cat = (float *)take (cat * 4);
  s.qa = (float *)take (qa * 4);
  s.ff = (float *)take (ff * 4);
  s.logits = (float *)take ((size_t)m->vocab * 4);
  s.amax_v = (float *)take (kMaxGrid * 4);
  s.amax_i = (uint32_t *)take (kMaxGrid * 4);
  s.bytes = off;
  return s;
}

int
check_stack (const vkl_stack_model *m)
{
  VKL_CHECK_ARG (m && m->layers_h && m->embed && m->final_norm && m->scratch);
  VKL_CHECK_ARG (m->width > 0 && m->width <= m->width_p && (m->width_p % 64) == 0 && m->vocab > 0 && m->maxlen > 0
                 && m->n_runs > 0);
  VKL_CHECK_ARG (m->ctype == VKL_TYPE_F32 || m->ctype == VKL_TYPE_BF16);
  VKL_CHECK_ARG (gv_supported (m->width_p));
  for (int i = 0; i < m->n_runs; ++i)
    {
      const vkl_stack_layer &l = m->layers_h[i];
      VKL_CHECK_ARG (l.mixer >= VKL_MIX_SHARED_KV && l.mixer <= VKL_MIX_DECAY);
      const bool recur = l.mixer == VKL_MIX_DELTA || l.mixer == VKL_MIX_DECAY;
      VKL_CHECK_ARG (l.norm && l.w_in && l.w_out && (l.cache || recur) && l.H > 0 && l.G > 0 && (l.H % l.G) == 0);
      VKL_CHECK_ARG (l.dim > 0 && (l.dim % 32) == 0 && l.vdim > 0 && (l.vdim % 32) == 0);
      VKL_CHECK_ARG ((l.k_out % 64) == 0 && gv_supported (l.k_out) && l.ff >= 0);
      if (l.norm2)
        VKL_CHECK_ARG (l.ff > 0 && l.w_up && l.w_down && (l.ff_p % 64) == 0 && l.ff_p >= l.ff && gv_supported (l.ff_p)
                       && l.H * l.vdim <= l.k_out);
      else
        VKL_CHECK_ARG (l.ff_col >= l.H * l.vdim && l.ff_col + l.ff <= l.k_out);
      VKL_CHECK_ARG (l.temp_coef == 0.f || l.temp_every > 0);
      VKL_CHECK_ARG (l.kv0 >= (recur ? l.G : l.H) * l.dim);
      if (l.mixer == VKL_MIX_KV)
        {
          VKL_CHECK_ARG (l.vcache && l.dim <= kPrepMax && l.vdim == l.dim && l.n > 0 && l.n <= l.dim && l.chunk >= 0);
          VKL_CHECK_ARG (l.npair >= 0 && 2 * l.npair <= l.n && (l.npair == 0 || l.freq));
          VKL_CHECK_ARG (!l.vfirst || l.fdim > 0);
          VKL_CHECK_ARG (l.v0 == l.kv0 + l.G * l.dim && l.v0 + l.G * l.dim <= l.n_in);
        }
      else if (recur)
        {
          // (the three kinds of rows are one stretch)
          const int end = 2 * l.G * l.dim + l.H * l.vdim;
          VKL_CHECK_ARG (recur_supported (l.H, l.H / l.G, l.dim, l.vdim) && l.state && l.gnorm);
          VKL_CHECK_ARG (l.kv0 == l.G * l.dim && l.v0 == 2 * l.G * l.dim && l.n > 0 && l.n <= l.dim && l.vn > 0
                         && l.vn <= l.vdim);
          if (l.mixer == VKL_MIX_DECAY)
            VKL_CHECK_ARG (l.G == l.H && l.log_decay && l.g0 >= end && l.g0 + l.H * l.vdim <= l.n_in);
          else
            VKL_CHECK_ARG (l.conv && l.ring && l.taps >= 1 && l.taps <= 16 && l.dt_bias && l.rate && l.w_a2 && l.w_g2
                           && l.r_a > 0 && (l.r_a % 8) == 0 && l.r_g > 0 && (l.r_g % 8) == 0 && l.r_a + l.r_g <= 12288 && l.b0 >= end
                           && l.a0 >= l.b0 + l.H && l.g0 >= l.a0 + l.r_a && l.g0 + l.r_g <= l.n_in);
        }
      else if (l.mixer == VKL_MIX_LATENT)
        {
          VKL_CHECK_ARG (l.w_ukt && l.w_uv && l.c_norm && l.rank > 0 && l.rank <= l.rank_p && (l.rank_p % 32) == 0
                         && l.rank_p <= 1024 && l.G == 1);
          VKL_CHECK_ARG (l.g0 >= l.kv0 + l.rank && l.up0 >= l.g0 + l.H && l.up0 + l.ff <= l.n_in);
        }
      else
        VKL_CHECK_ARG (l.dim <= 1024 && l.vdim == l.dim && l.up0 >= l.kv0 + l.G * l.dim && l.up0 + l.ff <= l.n_in);
    }
  return 0;
}

struct StepArgs
{
  const vkl_stack_model *m;
  StackScratch s;
  StepPos pos;
  const uint32_t *toks; // the token, or the ids of a replayed loop
  float *logits;
  uint32_t *next_tok;
  uint32_t *loop, *ids;
  bool sampled;
  bool stream; // weights of the step beyond what the caches hold
  int n_cu;
};

// memory-side cache and L2s
constexpr size_t kCacheBytes = (size_t)288 << 20;

bool
weights_stream (const vkl_stack_model &m)
{
  size_t n = (size_t)m.vocab * m.width_p;
  for (int i = 0; i < m.n_runs; ++i)
    {
      const vkl_stack_layer &l = m.layers_h[i];
      n += (size_t)l.n_in * m.width_p + (size_t)m.width * l.k_out;
      if (l.norm2)
        n += (size_t)l.ff * m.width_p + (size_t)m.width * l.ff_p;
    }
  return n * 2 > kCacheBytes;
}

// a layer whose feed-forward part follows its mixer; a: the first product
int
launch_two_norm_layer (const StepArgs &p, const vkl_stack_layer &l, GvArgs a, hipStream_t st)
{
  const vkl_stack_model &m = *p.m;
  GvArgs o = {};
  o.w = (const uint16_t *)l.w_out, o.N = m.width, o.K = l.k_out;
  o.x = p.s.cat, o.y = p.s.x, o.stream = p.stream;
  if (l.mixer == VKL_MIX_KV)
    {
      a.nseg = 2;
      a.seg[0] = { 0, l.H * l.dim, p.s.q, 1, VKL_ACT_NONE, 0 };
      a.seg[1] = { l.kv0, 2 * l.G * l.dim, p.s.c, 1, VKL_ACT_NONE, 0 };
      if (int e = launch_gv<GV_SEGS> (a, p.n_cu, st))
        return e;
      vkl_attn_rows_prep r = {};
      r.H = l.H, r.G = l.G, r.dim = l.dim, r.n = l.n, r.npair = l.npair, r.freq = l.freq, r.eps = m.eps;
      r.q = r.qo = p.s.q, r.qtype = r.qotype = r.kvtype = VKL_TYPE_F32;
      r.k = p.s.c, r.v = p.s.c + l.G * l.dim, r.ko = l.cache, r.vo = l.vcache;
      r.first = l.vfirst, r.fdim = l.fdim, r.mix = l.vmix, r.ctype = m.ctype;
      if (int e = attn_prepare (r, 1, p.pos, st))
        return e;
      if (int e = kv_attention (p.s.q, VKL_TYPE_F32, 0, l.cache, l.vcache, m.ctype, (size_t)l.G * l.dim, l.H, l.G,
                                l.dim, 1, p.pos, l.scale, l.chunk, l.sink, p.s.cat, VKL_TYPE_F32, 0, p.s.cnt, st))
        return e;
      if (int e = launch_gv<GV_ADD> (o, p.n_cu, st))
        return e;
    }
  else
    {
      const bool delta = l.mixer == VKL_MIX_DELTA;
      float *b = p.s.g, *a1 = b + round64 (l.H), *g1 = a1 + round64 (l.r_a);
      a.seg[0] = { 0, 2 * l.G * l.dim + l.H * l.vdim, p.s.c, 1, delta ? VKL_ACT_NONE : VKL_ACT_SILU, 0 };
      if (delta)
        {
          a.nseg = 4;
          a.seg[1] = { l.b0, l.H, b, 1, VKL_ACT_NONE, 0 };
          a.seg[2] = { l.a0, l.r_a, a1, 1, VKL_ACT_NONE, 0 };
          a.seg[3] = { l.g0, l.r_g, g1, 1, VKL_ACT_NONE, 0 };
        }
      else
        {
          a.nseg = 2;
          a.seg[1] = { l.g0, l.H * l.vdim, p.s.g, 1, VKL_ACT_NONE, 0 };
        }
      if (int e = launch_gv<GV_SEGS> (a, p.n_cu, st))
        return e;
      RecurStepArgs r = {};
      r.H = l.H, r.rep = l.H / l.G, r.dim = l.dim, r.vdim = l.vdim, r.n = l.n, r.vn = l.vn, r.pos = p.pos;
      r.qkv = p.s.c, r.state = l.state, r.out = p.s.cat, r.qscale = l.qscale;
      if (delta)
        {
          r.conv = l.conv, r.ring = l.ring, r.taps = l.taps, r.b = b, r.a1 = a1, r.g1 = g1;
          r.w_a2 = (const uint16_t *)l.w_a2, r.w_g2 = (const uint16_t *)l.w_g2, r.r_a = l.r_a, r.r_g = l.r_g;
          r.dt_bias = l.dt_bias, r.rate = l.rate, r.gnorm = l.gnorm, r.unit_eps = l.unit_eps, r.eps = m.eps;
          if (int e = delta_step_launch (r, st))
            return e;
          if (int e = launch_gv<GV_ADD> (o, p.n_cu, st))
            return e;
        }
      else
        {
          r.log_decay = l.log_decay, r.out_pad = l.k_out - l.H * l.vdim;
          if (int e = decay_step_launch (r, st))
            return e;
          o.norm = l.gnorm, o.gate = p.s.g, o.W = l.H * l.vn, o.eps = m.eps;
          if (int e = launch_gv<GV_GATED> (o, p.n_cu, st))
            return e;
        }
    }
  if (!l.norm2)
    return 0;
  GvArgs u = {};
  u.w = (const uint16_t *)l.w_up, u.N = l.ff, u.K = m.width_p;
  u.x = p.s.x, u.norm = l.norm2, u.W = m.width, u.eps = m.eps, u.pos = p.pos, u.stream = p.stream;
  u.nseg = 1;
  u.seg[0] = { 0, l.ff, p.s.ff, 1, l.ff_act, 0 };
  if (int e = launch_gv<GV_SEGS> (u, p.n_cu, st))
    return e;
  GvArgs d = {};
  d.w = (const uint16_t *)l.w_down, d.N = m.width, d.K = l.ff_p;
  d.x = p.s.ff, d.y = p.s.x, d.stream = p.stream;
  return launch_gv<GV_ADD> (d, p.n_cu, st);
}

int
launch_stack_layer (const StepArgs &p, const vkl_stack_layer &l, hipStream_t st)
{
  const vkl_stack_model &m = *p.m;
  const bool latent = l.mixer == VKL_MIX_LATENT;
  GvArgs a = {};
  a.w = (const uint16_t *)l.w_in, a.N = l.n_in, a.K = m.width_p;
  a.x = p.s.x, a.norm = l.norm, a.W = m.width, a.eps = m.eps, a.pos = p.pos, a.stream = p.stream;
  int n = 0;
  if (l.mixer == VKL_MIX_KV || l.mixer == VKL_MIX_DELTA || l.mixer == VKL_MIX_DECAY)
    return launch_two_norm_layer (p, l, a, st);
  a.seg[n++] = { 0, l.H * l.dim, p.s.q, 1, 0, 0 };
  if (latent)
    {
      a.seg[n++] = { l.kv0, l.rank, p.s.c, 1, 0, 0 };
      a.seg[n++] = { l.g0, l.H, p.s.g, 1, 0, 0 };
    }
  else
    a.seg[n++] = { l.kv0, l.G * l.dim, l.cache, m.ctype == VKL_TYPE_F32, 0, (size_t)l.G * l.dim };
  if (l.ff)
    a.seg[n++] = { l.up0, l.ff, p.s.cat + l.ff_col, 1, l.ff_act, 0 };
  a.nseg = n;
  if (int e = launch_gv<GV_SEGS> (a, p.n_cu, st))
    return e;
  if (latent)
    {
      HeadArgs h = {};
      h.w = (const uint16_t *)l.w_ukt, h.heads = l.H, h.R = l.rank_p, h.K = l.dim;
      h.x = p.s.q, h.xtype = VKL_TYPE_F32, h.xh = (size_t)l.dim;
      // (rounded here if the attention takes them as bf16 operands anyway)
      const int qt = row_mfma (m.ctype, l.H, l.rank_p) ? VKL_TYPE_BF16 : VKL_TYPE_F32;
      h.y = p.s.qa, h.ytype = qt, h.yh = (size_t)l.rank_p;
      h.nx = p.s.c, h.nw = l.c_norm, h.nW = l.rank, h.nWp = l.rank_p, h.neps = m.eps;
      h.ncache = l.cache, h.ntype = m.ctype, h.pos = p.pos;
      if (int e = head_matvec (h, 1, st))
        return e;
      HeadArgs v = {};
      if (int e = rows_attention (p.s.qa, qt, 0, l.cache, m.ctype, (size_t)l.rank_p, l.H, 1, l.rank_p, 1,
                                  p.pos, l.scale, l.temp_coef, l.temp_every, nullptr, VKL_TYPE_F32, 0, p.s.cnt,
                                  &v.parts, st))
        return e;
      v.pos = p.pos;
      v.w = (const uint16_t *)l.w_uv, v.heads = l.H, v.R = l.vdim, v.K = l.rank_p;
      v.y = p.s.cat, v.ytype = VKL_TYPE_F32, v.yh = (size_t)l.vdim;
      v.gate = p.s.g;
      if (int e = head_matvec (v, 1, st))
        return e;
    }
  else if (int e = rows_attention (p.s.q, VKL_TYPE_F32, 0, l.cache, m.ctype, (size_t)l.G * l.dim, l.H, l.G, l.dim, 1,
                                   p.pos, l.scale, l.temp_coef, l.temp_every, p.s.cat, VKL_TYPE_F32, 0, p.s.cnt, nullptr, st))
    return e;
  GvArgs o = {};
  o.w = (const uint16_t *)l.w_out, o.N = m.width, o.K = l.k_out;
  o.x = p.s.cat, o.y = p.s.x, o.stream = p.stream;
  return launch_gv<GV_ADD> (o, p.n_cu, st);
}

int
launch_stack_step (const StepArgs &p, hipStream_t st)
{
  const vkl_stack_model &m = *p.m;
  EmbedArgs e = {};
  e.table = (const uint16_t *)m.embed, e.VH = (uint32_t)m.vocab, e.K = m.width_p, e.W = m.width;
  e.toks = p.toks, e.loop = p.loop, e.w = m.embed_norm, e.eps = m.eps, e.scale = m.embed_scale, e.out = p.s.x, e.os = (size_t)m.width_p;
  embed_norm_kernel<<<dim3 (1), dim3 (1024), 0, st>>> (e);
  for (int i = 0; i < m.n_runs; ++i)
    if (int err = launch_stack_layer (p, m.layers_h[i], st))
      return err;
  GvArgs a = {};
  a.w = (const uint16_t *)(m.head ? m.head : m.embed), a.N = m.vocab, a.K = m.width_p;
  a.x = p.s.x, a.norm = m.final_norm, a.W = m.width, a.eps = m.eps;
  a.y = p.logits ? p.logits : p.s.logits, a.cap = m.logit_cap, a.stream = p.stream;
  a.amax_v = p.s.amax_v, a.amax_i = p.s.amax_i, a.amax_cnt = p.s.sync;
  a.pick = (p.next_tok || p.loop) && !p.sampled;
  a.next_tok = p.next_tok, a.loop = p.loop, a.ids = p.ids;
  if (int err = launch_gv<GV_LOGITS> (a, p.n_cu, st))
    return err;
  if (p.loop && p.sampled)
    return sample_loop_launch (a.y, m.vocab, p.s.sync + 20, p.loop, p.ids, st);
  return (int)hipGetLastError ();
}

int
compute_units (int *n_cu)
{
  int dev = 0;
  VKL_HIP (hipGetDevice (&dev));
  VKL_HIP (hipDeviceGetAttribute (n_cu, hipDeviceAttributeMultiprocessorCount, dev));
  VKL_CHECK_ARG (2 * *n_cu <= kMaxGrid);
  return 0;
}

__global__ void
set_stack_loop_kernel (uint32_t *sync, uint32_t pos, uint32_t k, uint32_t p_bits, uint32_t seed_lo, uint32_t seed_hi)
{
  sync[16] = 0u, sync[17] = pos;
  sync[20] = k, sync[21] = p_bits, sync[22] = seed_lo, sync[23] = seed_hi;
}

// captured steps, one per (model, buffers, way of picking the token)
struct StackGraph
{
  uint64_t key = 0;
  const void *scratch = nullptr;
  hipGraph_t graph = nullptr;
  hipGraphExec_t exec = nullptr;
};
std::vector<StackGraph> g_stack_graphs;
std::mutex g_stack_mu;
constexpr size_t kStackGraphs = 8;

void
drop_stack_graph (StackGraph &g)
{
  if (g.exec)
    (void)hipGraphExecDestroy (g.exec);
  if (g.graph)
    (void)hipGraphDestroy (g.graph);
}

uint64_t
stack_key (const vkl_stack_model *m, const void *ids, const void *logits, bool sampled)
{
  uint64_t h = 1469598103934665603ull;
  auto mix = [&h] (const void *p, size_t n) {
    for (size_t i = 0; i < n; ++i)
      h = (h ^ ((const uint8_t *)p)[i]) * 1099511628211ull;
  };
  const void *ptrs[7] = { m->embed, m->head, m->embed_norm, m->final_norm, m->scratch, ids, logits };
  const int dims[6] = { m->width, m->vocab, m->maxlen, m->n_runs, m->ctype, (int)sampled };
  mix (ptrs, sizeof (ptrs)), mix (dims, sizeof (dims)), mix (&m->eps, 4), mix (&m->logit_cap, 4), mix (&m->embed_scale, 4);
  mix (m->layers_h, sizeof (vkl_stack_layer) * (size_t)m->n_runs);
  return h;
}

int
stack_loop (const vkl_stack_model *m, uint32_t *ids, uint32_t pos0, int n_steps, float *logits, bool sampled,
            int topk, float topp, uint64_t seed, hipStream_t st)
{
  if (int e = check_stack (m))
    return e;
  VKL_CHECK_ARG (ids && n_steps >= 0 && (uint64_t)pos0 + (uint64_t)n_steps <= (uint64_t)m->maxlen);
  if (n_steps == 0)
    return 0;
  StepArgs p = {};
  p.m = m, p.s = carve_stack (m), p.stream = weights_stream (*m);
  if (int e = compute_units (&p.n_cu))
    return e;
  p.loop = p.s.sync + 16, p.ids = ids, p.toks = ids;
  p.pos = { p.loop, 0u };
  p.logits = logits, p.sampled = sampled;
  set_stack_loop_kernel<<<dim3 (1), dim3 (1), 0, st>>> (p.s.sync, pos0, (uint32_t)topk,
                                                        __builtin_bit_cast (uint32_t, topp), (uint32_t)seed,
                                                        (uint32_t)(seed >> 32));
  std::lock_guard<std::mutex> lock (g_stack_mu);
  const uint64_t key = stack_key (m, ids, logits, sampled);
  StackGraph *g = nullptr;
  for (StackGraph &c : g_stack_graphs)
    if (c.key == key && c.scratch == m->scratch)
      g = &c;
  if (!g)
    {
      StackGraph n;
      n.key = key, n.scratch = m->scratch;
      VKL_HIP (hipStreamBeginCapture (st, hipStreamCaptureModeThreadLocal));
      int err = launch_stack_step (p, st);
      const hipError_t e = hipStreamEndCapture (st, &n.graph);
      if (!err && e != hipSuccess)
        err = (int)e;
      if (!err)
        err = (int)hipGraphInstantiate (&n.exec, n.graph, nullptr, nullptr, 0);
      if (err)
        {
          drop_stack_graph (n);
          return err;
        }
      if (g_stack_graphs.size () >= kStackGraphs)
        {
          drop_stack_graph (g_stack_graphs.front ());
          g_stack_graphs.erase (g_stack_graphs.begin ());
        }
      g_stack_graphs.push_back (n);
      g = &g_stack_graphs.back ();
    }
  for (int i = 0; i < n_steps; ++i)
    VKL_HIP (hipGraphLaunch (g->exec, st));
  return vkl_launch_status ();
}
} // namespace
} // namespace vkl

using namespace vkl;

extern "C" int
vkl_embed_norm_bf16 (const void *table, uint32_t VH, int K, int W, const uint32_t *toks, uint32_t n, const float *w,
                     float eps, float *out, size_t os, void *stream)
{
  VKL_CHECK_ARG (table && toks && out && VH > 0 && n > 0 && W > 0 && K >= W && os >= (size_t)W);
  EmbedArgs a = {};
  a.table = (const uint16_t *)table, a.VH = VH, a.K = K, a.W = W, a.toks = toks, a.w = w, a.eps = eps, a.scale = 1.f;
  a.out = out, a.os = os;
  embed_norm_kernel<<<dim3 (n), dim3 (1024), 0, (hipStream_t)stream>>> (a);
  return vkl_launch_status ();
}

extern "C" int
vkl_embed_rows_bf16 (const void *table, uint32_t VH, int K, int W, const uint32_t *toks, uint32_t n, float scale,
                     float *out, size_t os, void *stream)
{
  VKL_CHECK_ARG (table && toks && out && VH > 0 && n > 0 && W > 0 && K >= W && os >= (size_t)W);
  EmbedArgs a = {};
  a.table = (const uint16_t *)table, a.VH = VH, a.K = K, a.W = W, a.toks = toks, a.scale = scale;
  a.out = out, a.os = os;
  embed_norm_kernel<<<dim3 (n), dim3 (1024), 0, (hipStream_t)stream>>> (a);
  return vkl_launch_status ();
}

extern "C" int
vkl_rmsnorm_f32 (const float *x, size_t xs, const uint32_t *rows, int n, int W, const float *w, float eps, void *out,
                 int otype, size_t os, int Wp, void *stream)
{
  VKL_CHECK_ARG (x && w && out && n > 0 && W > 0 && Wp >= W && xs >= (size_t)W && os >= (size_t)Wp);
  VKL_CHECK_ARG (otype == VKL_TYPE_F32 || otype == VKL_TYPE_BF16);
  const NormArgs a = { x, xs, rows, W, Wp, w, eps, out, otype, os };
  const dim3 grid ((unsigned)n), block (256);
  hipStream_t st = (hipStream_t)stream;
  const bool vec = (W % 4) == 0 && (Wp % 4) == 0 && (xs % 4) == 0 && (os % 4) == 0 && ((uintptr_t)x % 16) == 0
                   && ((uintptr_t)w % 16) == 0 && ((uintptr_t)out % 16) == 0;
  if (vec && Wp <= 1024)
    rmsnorm_f32_kernel<1><<<grid, block, 0, st>>> (a);
  else if (vec && Wp <= 2048)
    rmsnorm_f32_kernel<2><<<grid, block, 0, st>>> (a);
  else if (vec && Wp <= 4096)
    rmsnorm_f32_kernel<4><<<grid, block, 0, st>>> (a);
  else if (vec && Wp <= 8192)
    rmsnorm_f32_kernel<8><<<grid, block, 0, st>>> (a);
  else
    rmsnorm_f32_kernel<0><<<grid, block, 0, st>>> (a);
  return vkl_launch_status ();
}

extern "C" size_t
vkl_attn_rows_scratch_bytes (int ctype, int H, int G, int dim, int S)
{
  if (H <= 0 || G <= 0 || H % G || dim <= 0 || S <= 0)
    return 0;
  return row_scratch_bytes (ctype, H, G, dim, S);
}

extern "C" int
vkl_attn_rows (const void *q, int qtype, size_t qs, const void *rows, int ctype, size_t rs, int H, int G, int dim,
               int S, uint32_t pos0, float scale, float temp_coef, int temp_every, void *out, int otype, size_t os,
               void *scratch, void *stream)
{
  VKL_CHECK_ARG (q && rows && out && scratch && H > 0 && G > 0 && (H % G) == 0 && S > 0 && S <= 65535);
  VKL_CHECK_ARG (dim > 0 && (dim % 32) == 0 && dim <= 1024 && rs >= (size_t)G * dim && (rs % 8) == 0);
  VKL_CHECK_ARG (temp_coef == 0.f || temp_every > 0);
  VKL_CHECK_ARG (((uintptr_t)rows % 16) == 0 && qs >= (size_t)H * dim && os >= (size_t)H * dim);
  VKL_CHECK_ARG ((qtype == VKL_TYPE_F32 || qtype == VKL_TYPE_BF16) && (ctype == VKL_TYPE_F32 || ctype == VKL_TYPE_BF16)
                 && (otype == VKL_TYPE_F32 || otype == VKL_TYPE_BF16));
  return rows_attention (q, qtype, qs, rows, ctype, rs, H, G, dim, S, StepPos{ nullptr, pos0 }, scale, temp_coef,
                         temp_every, out, otype, os, scratch, nullptr, (hipStream_t)stream);
}

extern "C" size_t
vkl_attn_kv_rows_scratch_bytes (int ctype, int H, int G, int dim, int S)
{
  if (H <= 0 || G <= 0 || H % G || dim <= 0 || S <= 0)
    return 0;
  return row_scratch_bytes (ctype, H, G, dim, S, true);
}

extern "C" int
vkl_attn_kv_rows (const void *q, int qtype, size_t qs, const void *rows, const void *vals, int ctype, size_t rs, int H,
                  int G, int dim, int S, uint32_t pos0, float scale, int chunk, int sink, void *out, int otype,
                  size_t os, void *scratch, void *stream)
{
  VKL_CHECK_ARG (q && rows && vals && out && scratch && H > 0 && G > 0 && (H % G) == 0 && S > 0 && S <= 65535);
  VKL_CHECK_ARG (dim > 0 && (dim % 32) == 0 && dim <= 1024 && rs >= (size_t)G * dim && (rs % 8) == 0 && chunk >= 0);
  VKL_CHECK_ARG (((uintptr_t)rows % 16) == 0 && ((uintptr_t)vals % 16) == 0 && ((uintptr_t)q % 16) == 0
                 && (qs % 8) == 0 && qs >= (size_t)H * dim && os >= (size_t)H * dim);
  VKL_CHECK_ARG ((qtype == VKL_TYPE_F32 || qtype == VKL_TYPE_BF16) && (ctype == VKL_TYPE_F32 || ctype == VKL_TYPE_BF16)
                 && (otype == VKL_TYPE_F32 || otype == VKL_TYPE_BF16));
  return kv_attention (q, qtype, qs, rows, vals, ctype, rs, H, G, dim, S, StepPos{ nullptr, pos0 }, scale, chunk, sink,
                       out, otype, os, scratch, (hipStream_t)stream);
}

extern "C" int
vkl_attn_prepare (const vkl_attn_rows_prep *p, int S, uint32_t pos0, void *stream)
{
  VKL_CHECK_ARG (p && S > 0 && p->H > 0 && p->G > 0 && p->dim > 0 && p->dim <= kPrepMax && p->n > 0 && p->n <= p->dim);
  VKL_CHECK_ARG (p->npair >= 0 && 2 * p->npair <= p->n && (p->npair == 0 || p->freq) && S <= 1 << 20);
  VKL_CHECK_ARG ((!p->q || (p->qo && p->qs >= (size_t)p->H * p->dim && p->qos >= (size_t)p->H * p->dim)) && (!p->k || p->ko)
                 && (!p->v || p->vo) && (!p->first || p->fdim > 0) && p->kvs >= (size_t)p->G * p->dim);
  return attn_prepare (*p, S, StepPos{ nullptr, pos0 }, (hipStream_t)stream);
}

extern "C" int
vkl_head_matvec (const void *w, int H, int R, int K, const void *x, int xtype, size_t xs, size_t xh, void *y,
                 int ytype, size_t ys, size_t yh, const float *gate, size_t gs, int S, void *stream)
{
  VKL_CHECK_ARG (w && x && y && H > 0 && R > 0 && K > 0 && (K % 32) == 0 && S > 0 && S <= 65535);
  VKL_CHECK_ARG ((xtype == VKL_TYPE_F32 || xtype == VKL_TYPE_BF16) && (ytype == VKL_TYPE_F32 || ytype == VKL_TYPE_BF16));
  VKL_CHECK_ARG (xh >= (size_t)K && yh >= (size_t)R && (xs % 8) == 0 && (xh % 8) == 0 && ((uintptr_t)x % 16) == 0
                 && ((uintptr_t)w % 16) == 0);
  VKL_CHECK_ARG (S == 1 || (xs >= (size_t)H * xh && ys >= (size_t)H * yh));
  HeadArgs a = {};
  a.w = (const uint16_t *)w, a.heads = H, a.R = R, a.K = K, a.x = x, a.xtype = xtype, a.xs = xs, a.xh = xh;
  a.y = y, a.ytype = ytype, a.ys = ys, a.yh = yh, a.gate = gate, a.gs = gs;
  return head_matvec (a, S, (hipStream_t)stream);
}

extern "C" size_t
vkl_stack_scratch_bytes (const vkl_stack_model *m)
{
  if (!m || !m->layers_h || m->n_runs <= 0)
    return 0;
  return carve_stack (m).bytes;
}

extern "C" int
vkl_stack_supported (const vkl_stack_model *m)
{
  return check_stack (m) == 0 ? 1 : 0;
}

extern "C" int
vkl_stack_step (const vkl_stack_model *m, const uint32_t *tok, uint32_t pos, float *logits32, uint32_t *next_tok,
                void *stream)
{
  if (int e = check_stack (m))
    return e;
  VKL_CHECK_ARG (tok && pos < (uint32_t)m->maxlen);
  StepArgs p = {};
  p.m = m, p.s = carve_stack (m), p.stream = weights_stream (*m);
  if (int e = compute_units (&p.n_cu))
    return e;
  p.pos = { nullptr, pos }, p.toks = tok, p.logits = logits32, p.next_tok = next_tok;
  return launch_stack_step (p, (hipStream_t)stream);
}

extern "C" int
vkl_stack_loop (const vkl_stack_model *m, uint32_t *ids, uint32_t pos0, int n_steps, float *logits32, void *stream)
{
  return stack_loop (m, ids, pos0, n_steps, logits32, false, 1, -1.f, 0, (hipStream_t)stream);
}

extern "C" int
vkl_stack_loop_sampled (const vkl_stack_model *m, uint32_t *ids, uint32_t pos0, int n_steps, float *logits32,
                        int topk, float topp, uint64_t seed, void *stream)
{
  VKL_CHECK_ARG (topp >= 0.f || topk >= 1);
  VKL_CHECK_ARG (topp < 0.f || topp <= 1.0f);
  return stack_loop (m, ids, pos0, n_steps, logits32, true, topk, topp, seed, (hipStream_t)stream);
}

extern "C" void
vkl_stack_release (const vkl_stack_model *m)
{
  if (!m)
    return;
  std::lock_guard<std::mutex> lock (g_stack_mu);
  for (size_t i = 0; i < g_stack_graphs.size ();)
    if (g_stack_graphs[i].scratch == m->scratch)
      {
        drop_stack_graph (g_stack_graphs[i]);
        g_stack_graphs.erase (g_stack_graphs.begin () + (long)i);
      }
    else
      ++i;
}
