// Device side shared by the latent attention kernels: cache geometry and launch parameters.
#pragma once
#include "t12_abi.h"
#include "t12_act.h"
#include "t12_device.h"

namespace latent_attn {

constexpr int BLK = 32;                    // positions per cache block

struct LatentParams {
    T12LatentAttn a;
    const float* in;
    int ld;
    const T12Row* rows;
    int n, run;
    void* q;                               // [row][head][row_p]: the query in the latent's coordinates, then its rotated part
    void* mean;                            // [row][head][rank_p]: weighted mean of the latents; or, with parts, their
    float2* parts;                         // [row][head][splits]: (largest score, sum of weights) of every stretch of keys, whose
    int splits;                            // weighted sums are then fp32 [row][head][splits][rank_p] in mean
};

template <typename T>
__device__ __forceinline__ T to_cache(float v);
template <>
__device__ __forceinline__ float to_cache<float>(float v) { return v; }
template <>
__device__ __forceinline__ uint16_t to_cache<uint16_t>(float v) { return t12_f32_to_bf16(v); }
__device__ __forceinline__ float from_cache(float v) { return v; }
__device__ __forceinline__ float from_cache(uint16_t v) { return t12_bf16_to_f32(v); }

__device__ __forceinline__ uint32_t pack_bf16(float lo, float hi)
{
    typedef __attribute__((ext_vector_type(2))) float f2;
    return __builtin_bit_cast(uint32_t, __builtin_convertvector((f2){lo, hi}, t12_bf16x2));
}

// What the pieces of a position's row are turned by: eight positions next to each other all differ, and four within an aligned
// four differ above the lowest bit (they read two pieces each at once).
__device__ __forceinline__ int turn(int position) { return ((position << 1) & 6) | ((position >> 2) & 1); }
// Where element e of a position's row lies within the row.
__device__ __forceinline__ int place(const T12LatentAttn& a, int position, int e)
{
    return a.matrix ? ((e >> 3) ^ turn(position)) * 8 + (e & 7) : e;
}

}  // namespace latent_attn
