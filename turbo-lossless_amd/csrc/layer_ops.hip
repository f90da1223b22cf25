// Layer pieces around the mixers: embeddings (learned positions, normed), the 32-bit RMSNorm, norms around sublayers, unary
// activations, gated linear units.

#include "t12_act.h"
#include "t12_device.h"
#include "t12_host.h"

namespace {

__global__ __launch_bounds__(256) void embed_positions_kernel(const uint16_t* __restrict__ table, int n_vocab,
                                                              const uint16_t* __restrict__ pos, int n_positions,
                                                              const int* __restrict__ tokens, const T12Row* __restrict__ rows,
                                                              float* __restrict__ out, int width)
{
    const int r = blockIdx.y, i = blockIdx.x * 256 + threadIdx.x;
    if (i >= width) return;
    const int t = tokens[r], p = rows[r].position;
    float v = t >= 0 && t < n_vocab ? t12_bf16_to_f32(table[(size_t)t * width + i]) : 0.0f;
    if (p >= 0 && p < n_positions) v += t12_bf16_to_f32(pos[(size_t)p * width + i]);
    out[(size_t)r * width + i] = v;
}

// Sum over a workgroup of whole waves, in every thread; red holds a float per wave.
__device__ __forceinline__ float block_sum(float v, float* red)
{
    v = t12_wave_sum(v);
    __syncthreads();                                       // red may still be read
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = v;
    __syncthreads();
    float s = 0.0f;
    for (int w = 0; w < (int)blockDim.x / 64; w++) s += red[w];
    return s;
}

__global__ __launch_bounds__(256) void embed_norm_kernel(const uint16_t* __restrict__ table, int n_vocab, const int* __restrict__ tokens,
                                                         const float* __restrict__ w, float eps, float* __restrict__ out, int width)
{
    __shared__ float red[4];
    const int t = tokens[blockIdx.x];
    const bool known = t >= 0 && t < n_vocab;
    const uint16_t* row = table + (size_t)(known ? t : 0) * width;
    float ss = 0.0f;
    if (width % 8 == 0 && width <= 8192 && ((uintptr_t)table | (uintptr_t)out | (uintptr_t)w) % 16 == 0) {
        uint4 e[4];                                        // everything the thread needs, requested at once
#pragma unroll
        for (int q = 0; q < 4; q++) {
            const int i = (threadIdx.x + q * 256) * 8;
            e[q] = i < width ? *(const uint4*)(row + i) : make_uint4(0, 0, 0, 0);
        }
#pragma unroll
        for (int q = 0; q < 4; q++)
            for (uint32_t u : {e[q].x, e[q].y, e[q].z, e[q].w}) {
                const float a = __builtin_bit_cast(float, u << 16), b = __builtin_bit_cast(float, u & 0xFFFF0000u);
                ss += a * a + b * b;
            }
        const float rn = known ? 1.0f / sqrtf(block_sum(ss, red) / (float)width + eps) : 0.0f;
#pragma unroll
        for (int q = 0; q < 4; q++) {
            const int i = (threadIdx.x + q * 256) * 8;
            if (i >= width) continue;
            const uint32_t u[4] = {e[q].x, e[q].y, e[q].z, e[q].w};
#pragma unroll
            for (int h = 0; h < 2; h++) {
                const t12_f32x4 g = *(const t12_f32x4*)(w + i + 4 * h);
                t12_f32x4 v;
#pragma unroll
                for (int k = 0; k < 4; k++)
                    v[k] = __builtin_bit_cast(float, k & 1 ? u[2 * h + (k >> 1)] & 0xFFFF0000u : u[2 * h + (k >> 1)] << 16) * rn * g[k];
                *(t12_f32x4*)(out + (size_t)blockIdx.x * width + i + 4 * h) = v;
            }
        }
        return;
    }
    for (int i = threadIdx.x; i < width; i += 256) {
        const float v = t12_bf16_to_f32(row[i]);
        ss += v * v;
    }
    const float rn = known ? 1.0f / sqrtf(block_sum(ss, red) / (float)width + eps) : 0.0f;
    for (int i = threadIdx.x; i < width; i += 256) out[(size_t)blockIdx.x * width + i] = t12_bf16_to_f32(row[i]) * rn * w[i];
}

// One workgroup per row; a thread's values stay in registers between the two norms (width <= 8 x threads x ITEMS).  y
// values: the sum of nsplit partial rows, or y itself.
struct PostNormParams {
    const float* y;
    int nsplit;
    size_t split_stride;
    int ld;
    const float* residual;
    const float* post_w;
    const float* norm_w;
    float eps;
    float* x_out;
    void* h;
    int width;
};
template <bool F32, bool VEC>
__global__ __launch_bounds__(1024) void post_norm_add_kernel(const PostNormParams p)
{
    constexpr int E = VEC ? 4 : 1, ITEMS = VEC ? 2 : 8;
    __shared__ float red[16];
    const size_t r = blockIdx.x;
    const int step = blockDim.x * E;
    float v[ITEMS][E], res[ITEMS][E], pw[ITEMS][E], nw[ITEMS][E];
    auto fetch = [](float (&d)[E], const float* src) {
        if (VEC) {
            const t12_f32x4 a = *(const t12_f32x4*)src;
#pragma unroll
            for (int e = 0; e < E; e++) d[e] = a[e];
        } else d[0] = *src;
    };
    float ss = 0.0f;
#pragma unroll
    for (int q = 0; q < ITEMS; q++) {                      // (everything is requested ahead of the first sum)
        const int i = threadIdx.x * E + q * step;
#pragma unroll
        for (int e = 0; e < E; e++) v[q][e] = 0.0f;
        if (i < p.width) {
            fetch(res[q], p.residual + r * p.width + i);
            fetch(pw[q], p.post_w + i);
            fetch(nw[q], p.norm_w + i);
            const float* src = p.y + r * p.ld + i;
            for (int z = 0; z < p.nsplit; z++) {
                float a[E];
                fetch(a, src + z * p.split_stride);
#pragma unroll
                for (int e = 0; e < E; e++) v[q][e] += a[e];
            }
#pragma unroll
            for (int e = 0; e < E; e++) ss += v[q][e] * v[q][e];
        }
    }
    const float pn = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
    ss = 0.0f;
#pragma unroll
    for (int q = 0; q < ITEMS; q++)
        if ((int)threadIdx.x * E + q * step < p.width) {
#pragma unroll
            for (int e = 0; e < E; e++) {
                v[q][e] = res[q][e] + v[q][e] * pn * pw[q][e];
                ss += v[q][e] * v[q][e];
            }
        }
    const float rn = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
#pragma unroll
    for (int q = 0; q < ITEMS; q++) {
        const int i = threadIdx.x * E + q * step;
        if (i >= p.width) continue;
        float* x = p.x_out + r * p.width + i;
        if constexpr (VEC) {
            *(t12_f32x4*)x = (t12_f32x4){v[q][0], v[q][1], v[q][2], v[q][3]};
            t12_f32x4 h;
#pragma unroll
            for (int e = 0; e < 4; e++) h[e] = v[q][e] * rn * nw[q][e];
            if (F32) *(t12_f32x4*)((float*)p.h + r * p.width + i) = h;
            else
                *(uint2*)((uint16_t*)p.h + r * p.width + i) = make_uint2(t12_f32_to_bf16(h[0]) | ((uint32_t)t12_f32_to_bf16(h[1]) << 16),
                                                                         t12_f32_to_bf16(h[2]) | ((uint32_t)t12_f32_to_bf16(h[3]) << 16));
        } else {
            *x = v[q][0];
            const float h = v[q][0] * rn * nw[q][0];
            if (F32) ((float*)p.h)[r * p.width + i] = h;
            else ((uint16_t*)p.h)[r * p.width + i] = t12_f32_to_bf16(h);
        }
    }
}

// Any width: x_out carries the values between the passes.
template <bool F32>
__global__ __launch_bounds__(1024) void post_norm_add_wide_kernel(const PostNormParams p)
{
    __shared__ float red[16];
    const size_t r = blockIdx.x;
    float* x = p.x_out + r * p.width;
    float ss = 0.0f;
    for (int i = threadIdx.x; i < p.width; i += blockDim.x) {
        float v = 0.0f;
        for (int z = 0; z < p.nsplit; z++) v += p.y[z * p.split_stride + r * p.ld + i];
        x[i] = v;                                          // (y itself, or another buffer: each thread its own places)
        ss += v * v;
    }
    const float pn = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
    ss = 0.0f;
    for (int i = threadIdx.x; i < p.width; i += blockDim.x) {
        const float v = p.residual[r * p.width + i] + x[i] * pn * p.post_w[i];
        x[i] = v;
        ss += v * v;
    }
    const float rn = 1.0f / sqrtf(block_sum(ss, red) / (float)p.width + p.eps);
    for (int i = threadIdx.x; i < p.width; i += blockDim.x) {
        const float h = x[i] * rn * p.norm_w[i];
        if (F32) ((float*)p.h)[r * p.width + i] = h;
        else ((uint16_t*)p.h)[r * p.width + i] = t12_f32_to_bf16(h);
    }
}

template <bool F32>
__global__ __launch_bounds__(256) void glu_kernel(const float* __restrict__ gate, const float* __restrict__ up, const T12Glu glu, void* out,
                                                  size_t n)
{
    const size_t i = (size_t)blockIdx.x * 256 + threadIdx.x;
    if (i >= n) return;
    const float v = t12_apply_glu(gate[i], up[i], glu);
    if (F32) ((float*)out)[i] = v;
    else ((uint16_t*)out)[i] = t12_f32_to_bf16(v);
}

__global__ __launch_bounds__(256) void rms_norm_f32_kernel(const float* __restrict__ x, const float* __restrict__ w,
                                                           float* __restrict__ y, int n, float eps)
{
    __shared__ float red[4];
    const float* row = x + (size_t)blockIdx.x * n;
    float ss = 0.0f;
    for (int i = threadIdx.x; i < n; i += 256) ss += row[i] * row[i];
    ss = t12_wave_sum(ss);
    if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
    __syncthreads();
    const float rn = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)n + eps);
    for (int i = threadIdx.x; i < n; i += 256) y[(size_t)blockIdx.x * n + i] = row[i] * rn * w[i];
}

template <int KIND, bool F32>
__global__ __launch_bounds__(256) void act_kernel(const float* x, float a, float b, void* out, size_t n, int wide)
{
    const size_t i = ((size_t)blockIdx.x * 256 + threadIdx.x) * 4;
    if (i + 3 < n && wide) {
        float4 v = *(const float4*)(x + i);
        v.x = t12_apply_act<KIND>(v.x, a, b);
        v.y = t12_apply_act<KIND>(v.y, a, b);
        v.z = t12_apply_act<KIND>(v.z, a, b);
        v.w = t12_apply_act<KIND>(v.w, a, b);
        if (F32) *(float4*)((float*)out + i) = v;
        else *(uint2*)((uint16_t*)out + i) = make_uint2(t12_f32_to_bf16(v.x) | ((uint32_t)t12_f32_to_bf16(v.y) << 16),
                                                        t12_f32_to_bf16(v.z) | ((uint32_t)t12_f32_to_bf16(v.w) << 16));
        return;
    }
    for (size_t j = i; j < min(i + 4, n); j++) {
        const float v = t12_apply_act<KIND>(x[j], a, b);
        if (F32) ((float*)out)[j] = v;
        else ((uint16_t*)out)[j] = t12_f32_to_bf16(v);
    }
}

// The function of sums whose K-split partial rows the GEMM left in its workspace (ascending splits, like its own reduction).
template <int KIND>
__global__ __launch_bounds__(256) void act_partials_kernel(const float* __restrict__ ws, int nsplit, size_t split_stride, int ld, float a,
                                                           float b, uint16_t* __restrict__ out, int M)
{
    const int m = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (m >= M) return;
    const float* src = ws + (size_t)blockIdx.y * ld + m;
    uint16_t* o = out + (size_t)blockIdx.y * M + m;
    for (int i = 0; i < 4 && m + i < M; i++) {
        float v = 0.0f;
        for (int z = 0; z < nsplit; z++) v += src[(size_t)z * split_stride + i];
        o[i] = t12_f32_to_bf16(t12_apply_act<KIND>(v, a, b));
    }
}

// Four neighbouring sums at a time: rows and strides of whole 16-byte pieces.
template <int KIND>
__global__ __launch_bounds__(256) void act_partials4_kernel(const float* __restrict__ ws, int nsplit, size_t split_stride, int ld, float a,
                                                            float b, uint16_t* __restrict__ out, int M)
{
    const int m = (blockIdx.x * 256 + threadIdx.x) * 4;
    if (m >= M) return;
    const float* src = ws + (size_t)blockIdx.y * ld + m;
    t12_f32x4 v = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int z = 0; z < nsplit; z++) v += *(const t12_f32x4*)(src + (size_t)z * split_stride);
#pragma unroll
    for (int i = 0; i < 4; i++) v[i] = t12_apply_act<KIND>(v[i], a, b);
    *(uint2*)(out + (size_t)blockIdx.y * M + m) = make_uint2(t12_f32_to_bf16(v[0]) | ((uint32_t)t12_f32_to_bf16(v[1]) << 16),
                                                             t12_f32_to_bf16(v[2]) | ((uint32_t)t12_f32_to_bf16(v[3]) << 16));
}

}  // namespace

extern "C" {

int t12_embed_positions(const void* table_bf16, int n_vocab, const void* pos_bf16, int n_positions, const int* tokens,
                        const T12Row* rows, float* out, int width, int n, void* stream)
{
    T12_REQUIRE(table_bf16 && pos_bf16 && tokens && rows && out && width >= 1 && n >= 1, "t12_embed_positions: bad operands");
    hipLaunchKernelGGL(embed_positions_kernel, dim3((width + 255) / 256, n), dim3(256), 0, (hipStream_t)stream,
                       (const uint16_t*)table_bf16, n_vocab, (const uint16_t*)pos_bf16, n_positions, tokens, rows, out, width);
    T12_CHECK_LAUNCH("t12_embed_positions");
    return T12_OK;
}

int t12_embed_norm(const void* table_bf16, int n_vocab, const int* tokens, const float* weight, float eps, float* out, int width,
                   int n, void* stream)
{
    T12_REQUIRE(table_bf16 && n_vocab >= 1 && tokens && weight && out && width >= 1 && n >= 1, "t12_embed_norm: bad operands");
    hipLaunchKernelGGL(embed_norm_kernel, dim3(n), dim3(256), 0, (hipStream_t)stream, (const uint16_t*)table_bf16, n_vocab, tokens, weight,
                       eps, out, width);
    T12_CHECK_LAUNCH("t12_embed_norm");
    return T12_OK;
}

int t12_post_norm_add(const float* y, const T12GemmPartials* part, const float* residual, const float* post_w, const float* norm_w,
                      float eps, float* x_out, void* h, int h_f32, int width, int n, void* stream)
{
    T12_REQUIRE((part ? part->ws != nullptr && part->nsplit >= 1 && part->ld >= width : y != nullptr) && residual && post_w && norm_w &&
                    x_out && x_out != residual && h && width >= 1 && n >= 1,
                "t12_post_norm_add: bad operands");
    PostNormParams p = {part ? part->ws : y, part ? part->nsplit : 1, part ? part->split_stride : 0, part ? part->ld : width, residual,
                        post_w, norm_w, eps, x_out, h, width};
    hipStream_t st = (hipStream_t)stream;
    auto aligned = [](const void* q) { return (uintptr_t)q % 16 == 0; };
    if (width % 4 == 0 && width <= 8192 && p.ld % 4 == 0 && p.split_stride % 4 == 0 && aligned(p.y) && aligned(x_out) && aligned(residual) && aligned(post_w) && aligned(norm_w) && aligned(h)) {
        const int threads = width <= 4096 ? (width / 4 + 63) / 64 * 64 : 1024;
        if (h_f32) hipLaunchKernelGGL((post_norm_add_kernel<true, true>), dim3(n), dim3(threads), 0, st, p);
        else hipLaunchKernelGGL((post_norm_add_kernel<false, true>), dim3(n), dim3(threads), 0, st, p);
    } else if (width <= 8192) {
        const int threads = (((width + 7) / 8 + 63) / 64) * 64;
        if (h_f32) hipLaunchKernelGGL((post_norm_add_kernel<true, false>), dim3(n), dim3(threads), 0, st, p);
        else hipLaunchKernelGGL((post_norm_add_kernel<false, false>), dim3(n), dim3(threads), 0, st, p);
    } else {
        if (h_f32) hipLaunchKernelGGL(post_norm_add_wide_kernel<true>, dim3(n), dim3(1024), 0, st, p);
        else hipLaunchKernelGGL(post_norm_add_wide_kernel<false>, dim3(n), dim3(1024), 0, st, p);
    }
    T12_CHECK_LAUNCH("t12_post_norm_add");
    return T12_OK;
}

int t12_glu(const float* gate, const float* up, const T12Glu* glu, void* out, int out_f32, size_t n, void* stream)
{
    T12_REQUIRE(gate && up && glu && out && n >= 1, "t12_glu: bad operands");
    const dim3 grid((unsigned)((n + 255) / 256));
    if (out_f32) hipLaunchKernelGGL(glu_kernel<true>, grid, dim3(256), 0, (hipStream_t)stream, gate, up, *glu, out, n);
    else hipLaunchKernelGGL(glu_kernel<false>, grid, dim3(256), 0, (hipStream_t)stream, gate, up, *glu, out, n);
    T12_CHECK_LAUNCH("t12_glu");
    return T12_OK;
}

int t12_rms_norm_f32(const float* x, const float* weight, float* y, int width, float eps, int n, void* stream)
{
    T12_REQUIRE(x && weight && y && width >= 1 && n >= 1, "t12_rms_norm_f32: bad operands");
    hipLaunchKernelGGL(rms_norm_f32_kernel, dim3(n), dim3(256), 0, (hipStream_t)stream, x, weight, y, width, eps);
    T12_CHECK_LAUNCH("t12_rms_norm_f32");
    return T12_OK;
}

int t12_act(const float* x, const T12Act* act, void* out, int out_f32, size_t n, void* stream)
{
    T12_REQUIRE(x && act && out && n >= 1, "t12_act: bad operands");
    T12_REQUIRE(act->kind == T12_ACT_XIELU || act->kind == T12_ACT_SOFTCAP, "t12_act: unknown function %d", act->kind);
    const dim3 grid((unsigned)((n + 1023) / 1024));
    const int wide = (uintptr_t)x % 16 == 0 && (uintptr_t)out % (out_f32 ? 16 : 8) == 0;
    hipStream_t st = (hipStream_t)stream;
    if (act->kind == T12_ACT_XIELU) {
        if (out_f32) hipLaunchKernelGGL((act_kernel<T12_ACT_XIELU, true>), grid, dim3(256), 0, st, x, act->a, act->b, out, n, wide);
        else hipLaunchKernelGGL((act_kernel<T12_ACT_XIELU, false>), grid, dim3(256), 0, st, x, act->a, act->b, out, n, wide);
    } else {
        if (out_f32) hipLaunchKernelGGL((act_kernel<T12_ACT_SOFTCAP, true>), grid, dim3(256), 0, st, x, act->a, act->b, out, n, wide);
        else hipLaunchKernelGGL((act_kernel<T12_ACT_SOFTCAP, false>), grid, dim3(256), 0, st, x, act->a, act->b, out, n, wide);
    }
    T12_CHECK_LAUNCH("t12_act");
    return T12_OK;
}

int t12_act_partials(const T12GemmPartials* part, const T12Act* act, void* out_bf16, int M, int B, void* stream)
{
    T12_REQUIRE(part && part->ws && part->nsplit >= 1 && act && act->kind == T12_ACT_XIELU && out_bf16 && M >= 1 && B >= 1,
                "t12_act_partials: bad operands");
    const bool wide = M % 4 == 0 && part->ld % 4 == 0 && part->split_stride % 4 == 0 && (uintptr_t)part->ws % 16 == 0 && (uintptr_t)out_bf16 % 8 == 0;
    const dim3 grid((M + 1023) / 1024, B);
    hipStream_t st = (hipStream_t)stream;
    if (wide)
        hipLaunchKernelGGL(act_partials4_kernel<T12_ACT_XIELU>, grid, dim3(256), 0, st, part->ws, part->nsplit, part->split_stride, part->ld,
                           act->a, act->b, (uint16_t*)out_bf16, M);
    else
        hipLaunchKernelGGL(act_partials_kernel<T12_ACT_XIELU>, grid, dim3(256), 0, st, part->ws, part->nsplit, part->split_stride, part->ld,
                           act->a, act->b, (uint16_t*)out_bf16, M);
    T12_CHECK_LAUNCH("t12_act_partials");
    return T12_OK;
}

}  // extern "C"
