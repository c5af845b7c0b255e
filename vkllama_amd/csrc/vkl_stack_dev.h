// Device helpers shared by the kernels of decoder stacks (vkl_stack.hip,
// vkl_recur.hip), and the launches of vkl_recur.hip that the one-token step uses.
#ifndef VKL_STACK_DEV_H
#define VKL_STACK_DEV_H
#include "../../include/vkl_stack.h"
#include "vkl_act.h"
#include "vkl_common.h"
#include "vkl_decode_dev.h"

namespace vkl
{
// a position known on the host, or kept on the device by a replayed loop
// ({index into the ids, position})
struct StepPos
{
  const uint32_t *loop;
  uint32_t val;
  __device__ __forceinline__ uint32_t
  get () const
  {
    return loop ? ldg (loop + 1) : val;
  }
};

__device__ __forceinline__ void
widen8 (const uint4 w, float (&f)[8])
{
  const uint32_t u[4] = { w.x, w.y, w.z, w.w };
#pragma unroll
  for (int i = 0; i < 4; ++i)
    {
      f[2 * i] = __uint_as_float (u[i] << 16);
      f[2 * i + 1] = __uint_as_float (u[i] & 0xffff0000u);
    }
}

__device__ __forceinline__ float
sigmoid (float z)
{
  return 1.0f / (1.0f + expf (-z));
}

__device__ __forceinline__ float
load_elem (const void *p, int type, size_t i)
{
  return type == VKL_TYPE_F32 ? ldg ((const float *)p + i) : bf2f (ldg ((const uint16_t *)p + i));
}

__device__ __forceinline__ void
store_elem (void *p, int type, size_t i, float v)
{
  if (type == VKL_TYPE_F32)
    stg ((float *)p + i, v);
  else
    stg ((uint16_t *)p + i, f2bf (v));
}

// sum over a workgroup of up to 1024 threads; red: a float of LDS per wave
__device__ __forceinline__ float
group_sum (float v, float *red)
{
  v = wave_sum (v);
  if ((threadIdx.x & 63) == 0)
    red[threadIdx.x >> 6] = v;
  __syncthreads ();
  float s = 0.f;
  for (unsigned i = 0; i < blockDim.x / 64; ++i)
    s += red[i];
  __syncthreads ();
  return s;
}

// One token of a recurrent mixer (vkl_recur.hip): all values fp32.
struct RecurStepArgs
{
  int H, rep, dim, vdim, n, vn; // n, vn: sizes without padding
  StepPos pos;
  const float *qkv;       // the token's projections q | k | v
  const float *log_decay; // decaying sums
  // delta rule
  const float *conv;
  float *ring;
  int taps;
  const float *b, *a1, *g1;
  const uint16_t *w_a2, *w_g2;
  int r_a, r_g;
  const float *dt_bias, *rate, *gnorm;
  float qscale, unit_eps, eps;
  float *state;
  float *out; // [H*vdim]: delta rule normed and gated, decaying sums as they are
  int out_pad; // zeros written behind the heads (decaying sums: their norm reads them)
};
int delta_step_launch (const RecurStepArgs &a, hipStream_t s);
int decay_step_launch (const RecurStepArgs &a, hipStream_t s);
bool recur_supported (int H, int rep, int dim, int vdim);
} // namespace vkl
#endif
