// y[M,N] = x[M,K] W[N,K]^T in 32-bit: fp32 activations, bf16 weights (exact as
// fp32), products and sums on v_mfma_f32_32x32x2_f32, which multiplies and adds
// in full fp32.  The output columns fall into segments (GemmSegArgs).
//
// Workgroup = 4 waves on a 64 x 64 output tile, each wave one 32 x 32 block;
// k-steps of 32 through LDS, the next step's loads in flight in registers.
#include "vkl_common.h"
#include "vkl_gemm.h"
#include "vkl_gemm_finish.h"

namespace vkl
{
namespace
{
typedef float float16v __attribute__ ((ext_vector_type (16)));
constexpr int FT = 64, FBK = 32, FLD = FBK + 1;

__global__ __launch_bounds__ (256) void
gemm_f32_kernel (const GemmSegArgs a)
{
  __shared__ float xs[FT * FLD], ws[FT * FLD];
  __shared__ float park[FT * 68];
  const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
  const int m0 = blockIdx.y * FT, n0 = blockIdx.x * FT;
  const int wm = wave >> 1, wn = wave & 1;
  // a thread moves 8 neighbouring values of one row of each tile per step
  const int row = tid >> 2, col = (tid & 3) * 8;
  const float *xp = a.xf + (size_t)min (m0 + row, a.M - 1) * a.xs + col;
  const uint16_t *wp = a.wh[0] + (size_t)min (n0 + row, a.N - 1) * a.ws + col;
  float16v acc;
#pragma unroll
  for (int r = 0; r < 16; ++r)
    acc[r] = 0.f;
  uint4 x0 = ldg4 (xp), x1 = ldg4 (xp + 4), w0 = ldg4 (wp);
  for (int k = 0; k < a.K; k += FBK)
    {
      __syncthreads ();
      const uint32_t xw[8] = { x0.x, x0.y, x0.z, x0.w, x1.x, x1.y, x1.z, x1.w };
      const uint32_t ww[4] = { w0.x, w0.y, w0.z, w0.w };
#pragma unroll
      for (int e = 0; e < 8; ++e)
        {
          xs[row * FLD + col + e] = __uint_as_float (xw[e]);
          ws[row * FLD + col + e] = bf2f ((uint16_t)(ww[e >> 1] >> (16 * (e & 1))));
        }
      __syncthreads ();
      const int kn = min (k + FBK, a.K - FBK);
      x0 = ldg4 (xp + kn), x1 = ldg4 (xp + kn + 4), w0 = ldg4 (wp + kn);
      const float *xa = xs + (wm * 32 + (lane & 31)) * FLD + (lane >> 5);
      const float *wb = ws + (wn * 32 + (lane & 31)) * FLD + (lane >> 5);
#pragma unroll
      for (int kk = 0; kk < FBK; kk += 2)
        acc = __builtin_amdgcn_mfma_f32_32x32x2f32 (xa[kk], wb[kk], acc, 0, 0, 0);
    }
  // through LDS to eight neighbouring columns per thread
#pragma unroll
  for (int r = 0; r < 16; ++r)
    park[(wm * 32 + (r >> 2) * 8 + (lane >> 5) * 4 + (r & 3)) * 68 + wn * 32 + (lane & 31)] = acc[r];
  __syncthreads ();
#pragma unroll
  for (int i = 0; i < 2; ++i)
    {
      const int c = tid + i * 256, r = c >> 3, n = (c & 7) * 8;
      float v[8], g[8];
#pragma unroll
      for (int e = 0; e < 8; ++e)
        v[e] = park[r * 68 + n + e], g[e] = 0.f;
      gemm_finish8<false> (a, v, g, m0 + r, n0 + n, 0, 0, nullptr);
    }
}
} // namespace

int
gemm_f32_launch (const GemmSegArgs &a, hipStream_t s)
{
  const int tn = (a.N + FT - 1) / FT, tm = (a.M + FT - 1) / FT;
  if (tm > 65535)
    return (int)hipErrorInvalidValue;
  gemm_f32_kernel<<<dim3 ((unsigned)tn, (unsigned)tm), dim3 (256), 0, s>>> (a);
  return (int)hipGetLastError ();
}
} // namespace vkl
