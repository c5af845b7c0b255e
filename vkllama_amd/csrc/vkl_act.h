// Activations of the products of decoder stacks.
#ifndef VKL_ACT_H
#define VKL_ACT_H
#include "../../include/vkl_stack.h"
#include "vkl_common.h"

namespace vkl
{
// what a product stores for a sum (VKL_ACT_...)
__device__ __forceinline__ float
activate (int act, float v)
{
  if (act == VKL_ACT_SILU)
    return silu (v);
  if (act == VKL_ACT_RELU2)
    {
      v = fmaxf (v, 0.f);
      return v * v;
    }
  if (act == VKL_ACT_GELU)
    return 0.5f * v * (1.0f + erff (v * 0.70710678118654752440f));
  return v;
}
} // namespace vkl
#endif
