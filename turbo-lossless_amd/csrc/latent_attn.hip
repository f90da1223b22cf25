// Latent attention (T12LatentAttn, t12_mixers.h): every head's keys and values are projections of one cached vector per token.
//
// The projections are taken out of the sum over keys: a head's query is multiplied with its key projection once, scores are then
// inner products with the cached latent (and the shared rotated part), and the weighted mean of the latents is multiplied with
// the value projection at the end.  So attention runs over one shared "head" of rank + rot_dim channels whose values are the
// first rank of them, and a token's cache is that one row.

#include <algorithm>

#include "latent_attn.h"
#include "t12_host.h"

using namespace latent_attn;

namespace {

// ---- what a row stores and asks with.  One workgroup per row: the normed latent and the rotated key part into the cache; the
// rotated parts of the queries, and zeros in the padding, into the query rows.
template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(const LatentParams p)
{
    __shared__ float red[4];
    const T12LatentAttn& a = p.a;
    const int r = blockIdx.x, tid = threadIdx.x, half = a.rot_dim / 2;
    const T12Row row = p.rows[r];
    const float* x = p.in + (size_t)r * p.ld;
    const float* c = x + a.c_off;
    T* cache = (T*)a.cache + (size_t)(row.slot >> 1) * a.cache_elems + (size_t)row.position * a.row_p;
    float ss = 0.0f;
    for (int i = tid; i < a.rank; i += 256) ss += c[i] * c[i];
    ss = t12_wave_sum(ss);
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    __syncthreads();
    const float rn = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.rank + a.eps);
    for (int i = tid; i < a.rank; i += 256) cache[place(a, row.position, i)] = to_cache<T>(c[i] * rn * a.norm_w[i]);
    for (int i = tid; i < half; i += 256) {
        float sn, cs;
        sincosf((float)row.position * a.freqs[i], &sn, &cs);
        const float u = c[a.rank + i], v = c[a.rank + half + i];
        cache[place(a, row.position, a.rank_p + i)] = to_cache<T>(u * cs - v * sn);
        cache[place(a, row.position, a.rank_p + half + i)] = to_cache<T>(v * cs + u * sn);
    }
    T* q = (T*)p.q + (size_t)r * a.heads * a.row_p;
    const int qd = a.dim + a.rot_dim;
    for (int i = tid; i < a.heads * half; i += 256) {
        const int h = i / half, e = i % half;
        float sn, cs;
        sincosf((float)row.position * a.freqs[e], &sn, &cs);
        const float* y = x + a.q_off + h * qd + a.dim;
        const float u = y[e], v = y[half + e];
        q[(size_t)h * a.row_p + a.rank_p + e] = to_cache<T>(u * cs - v * sn);
        q[(size_t)h * a.row_p + a.rank_p + half + e] = to_cache<T>(v * cs + u * sn);
    }
    const int pad = a.row_p - a.rank - a.rot_dim, low = a.rank_p - a.rank;
    for (int i = tid; i < a.heads * pad; i += 256) {
        const int e = i % pad;
        q[(size_t)(i / pad) * a.row_p + (e < low ? a.rank + e : a.rank_p + a.rot_dim + e - low)] = to_cache<T>(0.0f);
    }
}

// ---- a product per head: y[r, h, m] = sum_k W[h M + m, k] x[r, h, k].  General form: any sizes, one wave per sixteen outputs
// of a (row, head); sums in fp32.
template <typename T>
struct HeadIn;                             // how a head's vector is read
struct FromProjection {                    // fp32 projections of the pass, rounded to what the state computes in
    const float* in;
    int ld, off, head_ld;
    bool round;
    __device__ __forceinline__ float at(int r, int h, int k) const
    {
        const float v = in[(size_t)r * ld + off + h * head_ld + k];
        return round ? t12_bf16_to_f32(t12_f32_to_bf16(v)) : v;
    }
};
template <typename T>
struct FromRows {                          // mean latents [row][head][rank_p]
    const T* x;
    int heads, head_ld;
    __device__ __forceinline__ float at(int r, int h, int k) const { return from_cache(x[((size_t)r * heads + h) * head_ld + k]); }
};

template <typename IN, typename OUT>
__global__ __launch_bounds__(256) void heads_general_kernel(T12Segment w, int heads, int M, int K, IN in, OUT out, int n)
{
    const int r = blockIdx.x, h = blockIdx.y, lane = threadIdx.x & 63;
    for (int m = blockIdx.z * 4 + (threadIdx.x >> 6); m < M; m += gridDim.z * 4) {
        const size_t row = (size_t)h * M + m, base = row * K;
        float acc = 0.0f;
        for (int k = lane; k < K; k += 64) {
            const size_t e = base + k;
            const uint32_t g = (w.gr[e >> 1] >> (4 * (e & 1))) & 0xFu;
            if (g != 0 || !w.row_off) acc += t12_bf16_to_f32(t12_decode_scalar(w.sm[e], g, w.base_exp)) * in.at(r, h, k);
        }
        if (w.row_off)
            for (int q = w.row_off[row] + lane; q < w.row_off[row + 1]; q += 64)
                acc += t12_bf16_to_f32((uint16_t)w.correct[q]) * in.at(r, h, w.cols[q]);
        acc = t12_wave_sum(acc);
        if (lane == 0) out.put(r, h, m, acc);
    }
}

template <typename T>
struct ToQuery {
    T* q;
    int heads, row_p;
    __device__ __forceinline__ void put(int r, int h, int m, float v) const { q[((size_t)r * heads + h) * row_p + m] = to_cache<T>(v); }
};
template <typename T>
struct ToGated {                           // times the head's sigmoid gate
    T* out;
    int out_ld, vdim;
    const float* in;
    int ld, g_off;
    __device__ __forceinline__ void put(int r, int h, int m, float v) const
    {
        out[(size_t)r * out_ld + h * vdim + m] = to_cache<T>(v * t12_sigmoid(in[(size_t)r * ld + g_off + h]));
    }
};

// ---- attention, general form: one workgroup per (row, head), any sizes, fp32 arithmetic.  Dynamic LDS: the query [row_p].
template <typename T>
__global__ __launch_bounds__(256) void latent_general_kernel(const LatentParams p)
{
    extern __shared__ float q[];
    __shared__ float wgt[256], red[4];
    const T12LatentAttn& a = p.a;
    const int r = blockIdx.x, h = blockIdx.y, tid = threadIdx.x;
    const T12Row row = p.rows[r];
    const T* cache = (const T*)a.cache + (size_t)(row.slot >> 1) * a.cache_elems;
    const T* qr = (const T*)p.q + ((size_t)r * a.heads + h) * a.row_p;
    for (int i = tid; i < a.row_p; i += 256) q[i] = from_cache(qr[i]);
    const int total = row.position + 1;
    for (int c0 = 0; c0 < a.rank; c0 += 256) {             // channels of the mean (one round unless rank > 256)
        const int c = c0 + tid;
        float acc = 0.0f, top = -INFINITY, sum = 0.0f;
        for (int t0 = 0; t0 < total; t0 += 256) {
            const int t = t0 + tid;
            float s = -INFINITY;
            __syncthreads();                               // q is there; wgt and red may still be read
            if (t < total) {
                s = 0.0f;
                for (int e = 0; e < a.row_p; e++) s += q[e] * from_cache(cache[(size_t)t * a.row_p + place(a, t, e)]);
                s *= a.scale;
            }
            float best = s;
#pragma unroll
            for (int off = 32; off > 0; off >>= 1) best = fmaxf(best, __shfl_xor(best, off, 64));
            if ((tid & 63) == 0) red[tid >> 6] = best;
            __syncthreads();
            best = fmaxf(fmaxf(fmaxf(red[0], red[1]), fmaxf(red[2], red[3])), top);
            const float back = expf(top - best);           // (first tile: e^-inf = 0)
            top = best;
            wgt[tid] = t < total ? expf(s - best) : 0.0f;
            __syncthreads();
            acc *= back;
            sum *= back;
            for (int i = 0; i < min(256, total - t0); i++) {
                const float w = wgt[i];
                sum += w;
                if (c < a.rank) acc += w * from_cache(cache[(size_t)(t0 + i) * a.row_p + place(a, t0 + i, c)]);
            }
        }
        if (c < a.rank) ((T*)p.mean)[((size_t)r * a.heads + h) * a.rank_p + c] = to_cache<T>(acc / sum);
    }
}

template <typename T>
void launch_general(const LatentParams& p, void* out, int out_ld, hipStream_t st)
{
    const T12LatentAttn& a = p.a;
    const FromProjection q = {p.in, p.ld, a.q_off, a.dim + a.rot_dim, sizeof(T) == 2};
    const ToQuery<T> to = {(T*)p.q, a.heads, a.row_p};
    hipLaunchKernelGGL((heads_general_kernel<FromProjection, ToQuery<T>>), dim3(p.n, a.heads, (a.rank + 63) / 64), dim3(256), 0, st, *a.k_up,
                       a.heads, a.rank, a.dim, q, to, p.n);
    hipLaunchKernelGGL(latent_general_kernel<T>, dim3(p.n, a.heads), dim3(256), (size_t)a.row_p * sizeof(float), st, p);
    const FromRows<T> mean = {(const T*)p.mean, a.heads, a.rank_p};
    const ToGated<T> gated = {(T*)out, out_ld, a.vdim, p.in, p.ld, a.g_off};
    hipLaunchKernelGGL((heads_general_kernel<FromRows<T>, ToGated<T>>), dim3(p.n, a.heads, (a.vdim + 63) / 64), dim3(256), 0, st, *a.v_up,
                       a.heads, a.vdim, a.rank, mean, gated, p.n);
}

}  // namespace

extern "C" {

int t12_latent_plan(T12LatentAttn* a, int max_positions, int rows)
{
    T12_REQUIRE(a && a->heads >= 1 && a->dim >= 1 && a->vdim >= 1 && a->rank >= 1 && a->rank <= 8192 && a->rot_dim >= 2 && a->rot_dim % 2 == 0 &&
                    a->rot_dim <= 8192,
                "t12_latent_plan: impossible heads or sizes");
    T12_REQUIRE(max_positions >= 1 && rows >= 1 && (a->elem_bytes == 2 || a->elem_bytes == 4), "t12_latent_plan: %d positions, %d rows or element size %d invalid",
                max_positions, rows, a->elem_bytes);
    a->matrix = 0;
    a->rank_p = (a->rank + 31) / 32 * 32;
    a->row_p = a->rank_p + (a->rot_dim + 31) / 32 * 32;
    const size_t blocks = (max_positions + BLK - 1) / BLK, el = a->elem_bytes;
    a->cache_elems = blocks * BLK * a->row_p;
    const size_t q = (size_t)rows * a->heads * a->row_p * el, mean = (size_t)rows * a->heads * a->rank_p * el;
    a->work_floats = (q + 15) / 16 * 4 + (mean + 15) / 16 * 4;
    return T12_OK;
}

int t12_latent_attention(const T12LatentAttn* a, const float* in, int ld, const T12Row* rows, int n, int run, int max_position, float* work,
                         void* out, int out_f32, int out_ld, void* stream)
{
    T12_REQUIRE(a && in && rows && work && out && a->cache && a->k_up && a->v_up && a->norm_w && a->freqs && n >= 1,
                "t12_latent_attention: null operand or no rows");
    T12_REQUIRE(a->rank_p >= a->rank && a->row_p >= a->rank_p + a->rot_dim, "t12_latent_attention: t12_latent_plan has not been called");
    T12_REQUIRE(a->q_off >= 0 && a->q_off + a->heads * (a->dim + a->rot_dim) <= ld && a->c_off >= 0 && a->c_off + a->rank + a->rot_dim <= ld &&
                    a->g_off >= 0 && a->g_off + a->heads <= ld && out_ld >= a->heads * a->vdim,
                "t12_latent_attention: a projection lies outside a row of %d, or output rows of %d are too short", ld, out_ld);
    T12_REQUIRE(a->k_up->M == a->heads * a->rank && a->v_up->M == a->heads * a->vdim, "t12_latent_attention: an up-projection has the wrong number of rows");
    T12_REQUIRE((out_f32 != 0) == (a->elem_bytes == 4), "t12_latent_attention: outputs have the cache's precision");
    T12_REQUIRE(max_position >= 0 && (size_t)max_position < a->cache_elems / a->row_p && (uintptr_t)work % 16 == 0,
                "t12_latent_attention: position %d outside the cache, or workspace not aligned", max_position);
    hipStream_t st = (hipStream_t)stream;
    LatentParams p = {};
    p.a = *a;
    p.in = in;
    p.ld = ld;
    p.rows = rows;
    p.n = n;
    p.run = run;
    p.q = work;
    p.mean = work + ((size_t)n * a->heads * a->row_p * a->elem_bytes + 15) / 16 * 4;
    if (a->elem_bytes == 4) hipLaunchKernelGGL(latent_store_kernel<float>, dim3(n), dim3(256), 0, st, p);
    else hipLaunchKernelGGL(latent_store_kernel<uint16_t>, dim3(n), dim3(256), 0, st, p);
    if (a->elem_bytes == 4) launch_general<float>(p, out, out_ld, st);
    else launch_general<uint16_t>(p, out, out_ld, st);
    T12_CHECK_LAUNCH("t12_latent_attention");
    return T12_OK;
}

}  // extern "C"
