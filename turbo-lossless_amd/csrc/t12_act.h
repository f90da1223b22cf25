// Unary functions of a projection's fp32 sums, shared by the kernels that apply them (T12Act, t12_mixers.h).
#pragma once
#include <hip/hip_runtime.h>
#include "t12_mixers.h"

template <int KIND>
__device__ __forceinline__ float t12_apply_act(float z, float a, float b)
{
    if (KIND == T12_ACT_XIELU) return z > 0.0f ? a * z * z + 0.5f * z : b * (expm1f(z) - z) + 0.5f * z;
    if (KIND == T12_ACT_SOFTCAP) return a * tanhf(z / a);
    return z;
}

__device__ __forceinline__ float t12_sigmoid(float x) { return 1.0f / (1.0f + expf(-x)); }

// Gated linear unit of a (gate, up) pair of sums.
__device__ __forceinline__ float t12_apply_glu(float g, float u, const T12Glu& p)
{
    g = fminf(g, p.limit);
    u = __builtin_amdgcn_fmed3f(u, -p.limit, p.limit);
    return g / (1.0f + expf(-p.slope * g)) * (u + p.offset);
}

// What SiLU(gate) * up is in these terms.
inline T12Glu t12_silu_glu() { return {__builtin_inff(), 1.0f, 0.0f}; }
