// Latent attention (T12LatentAttn, t12_mixers.h): every head's keys and values are projections of one cached vector per token.
//
// The projections are taken out of the sum over keys: a head's query is multiplied with its key projection once, scores are then
// inner products with the cached latent (and the shared rotated part), and the weighted mean of the latents is multiplied with
// the value projection at the end.  So attention runs over one shared "head" of rank + rot_dim channels whose values are the
// first rank of them, and a token's cache is that one row.
//
// A pass is the cache store with the rotations, the key projection of the queries, attention, the value projection with the gate;
// with few rows the store runs beside the key projection, in workgroups of its own.  All of them run on the matrix cores for the
// sizes that have instances; 32-bit states and other sizes take the general forms.

#include <algorithm>
#include <mutex>

#include "latent_attn.h"
#include "t12_host.h"

using namespace latent_attn;

namespace {

constexpr int MAX_SPLITS = 32;             // stretches of keys a row's attention is cut into

// ---- what a row stores and asks with, by one workgroup of 256 threads: the normed latent and the rotated key part into the cache;
// the rotated parts of the queries, and zeros in the padding, into the query rows.
template <typename T>
__device__ __forceinline__ void store_row(const LatentParams& p, int r)
{
    __shared__ float red[4];
    __shared__ float2 turned[64];                          // (cos, sin) of the row's angles, as many as there is room for
    const T12LatentAttn& a = p.a;
    const int tid = threadIdx.x, half = a.rot_dim / 2;
    const T12Row row = p.rows[r];
    const float* x = p.in + (size_t)r * p.ld;
    const float* c = x + a.c_off;
    T* cache = (T*)a.cache + (size_t)(row.slot >> 1) * a.cache_elems + (size_t)row.position * a.row_p;
    float ss = 0.0f;
    for (int i = tid; i < a.rank; i += 256) ss += c[i] * c[i];
    ss = t12_wave_sum(ss);
    __syncthreads();                                       // red and turned may still be read for the row before
    if ((tid & 63) == 0) red[tid >> 6] = ss;
    auto angle = [&](int i) {
        float2 t;
        sincosf((float)row.position * a.freqs[i], &t.y, &t.x);
        return t;
    };
    for (int i = tid; i < min(half, 64); i += 256) turned[i] = angle(i);
    __syncthreads();
    const float rn = 1.0f / sqrtf((red[0] + red[1] + red[2] + red[3]) / (float)a.rank + a.eps);
    for (int i = tid; i < a.rank; i += 256) cache[place(a, row.position, i)] = to_cache<T>(c[i] * rn * a.norm_w[i]);
    for (int i = tid; i < half; i += 256) {
        const float2 t = i < 64 ? turned[i] : angle(i);
        const float u = c[a.rank + i], v = c[a.rank + half + i];
        cache[place(a, row.position, a.rank_p + i)] = to_cache<T>(u * t.x - v * t.y);
        cache[place(a, row.position, a.rank_p + half + i)] = to_cache<T>(v * t.x + u * t.y);
    }
    T* q = (T*)p.q + (size_t)r * a.heads * a.row_p;
    const int qd = a.dim + a.rot_dim;
    for (int i = tid; i < a.heads * half; i += 256) {
        const int h = i / half, e = i % half;
        const float2 t = e < 64 ? turned[e] : angle(e);
        const float* y = x + a.q_off + h * qd + a.dim;
        const float u = y[e], v = y[half + e];
        q[(size_t)h * a.row_p + a.rank_p + e] = to_cache<T>(u * t.x - v * t.y);
        q[(size_t)h * a.row_p + a.rank_p + half + e] = to_cache<T>(v * t.x + u * t.y);
    }
    const int pad = a.row_p - a.rank - a.rot_dim, low = a.rank_p - a.rank;
    for (int i = tid; i < a.heads * pad; i += 256) {
        const int e = i % pad;
        q[(size_t)(i / pad) * a.row_p + (e < low ? a.rank + e : a.rank_p + a.rot_dim + e - low)] = to_cache<T>(0.0f);
    }
}

template <typename T>
__global__ __launch_bounds__(256) void latent_store_kernel(const LatentParams p)
{
    store_row<T>(p, blockIdx.x);
}

// LDS slot of (unit of eight columns, row): rows are rotated by the unit, so that neighbouring units of a row (how activations are
// written) and neighbouring rows of a unit (how they are read) lie on different banks.
template <int ROWS>
__device__ __forceinline__ int slot(int u, int r) { return u * ROWS + ((r + u) & (ROWS - 1)); }

// Rows r0 ... of a head's activations into LDS; columns past K and rows past n are zero.  Sixteen threads share a row.
__device__ __forceinline__ uint4 paired(const float (&v)[8])
{
    return make_uint4(pack_bf16(v[0], v[4]), pack_bf16(v[1], v[5]), pack_bf16(v[2], v[6]), pack_bf16(v[3], v[7]));
}
__device__ __forceinline__ uint4 masked(uint4 w, bool live)
{
    const uint32_t m = live ? ~0u : 0u;
    return make_uint4(w.x & m, w.y & m, w.z & m, w.w & m);
}
template <int ROWS, typename IN>
__device__ __forceinline__ void stage_rows(const IN& in, uint4* lds, int r0, int n, int h, int units, int K)
{
    for (int u = threadIdx.x & 15; u < units; u += 16)
        for (int r = threadIdx.x >> 4; r < ROWS; r += 16) {
            float v[8];
            const bool live = u * 8 < K && r0 + r < n;
            if (live) in.at8(r0 + r, h, u * 8, K - u * 8, v);
            lds[slot<ROWS>(u, r)] = live ? paired(v) : make_uint4(0, 0, 0, 0);
        }
}

// The same with the loads of U units in flight together: in.request(r, h, k) reads eight elements that exist, Raw::unpack gives them.
template <int ROWS, int U, typename IN>
__device__ __forceinline__ void stage_rows_ahead(const IN& in, uint4* lds, int r0, int n, int h, int units, int K)
{
    constexpr int RS = ROWS / 16;
    for (int u0 = threadIdx.x & 15; u0 < units; u0 += 16 * U) {
        typename IN::Raw raw[U][RS];
#pragma unroll
        for (int j = 0; j < U; j++)
#pragma unroll
            for (int i = 0; i < RS; i++)
                raw[j][i] = in.request(min(r0 + ((int)threadIdx.x >> 4) + i * 16, n - 1), h, min((u0 + j * 16) * 8, K - 8));
#pragma unroll
        for (int j = 0; j < U; j++)
#pragma unroll
            for (int i = 0; i < RS; i++) {
                const int u = u0 + j * 16, r = (threadIdx.x >> 4) + i * 16;
                float v[8];
                raw[j][i].unpack(v);
                if (U == 1 || u < units) lds[slot<ROWS>(u, r)] = masked(paired(v), u * 8 < K && r0 + r < n);
            }
    }
}

// ---- a product per head: y[r, h, m] = sum_k W[h M + m, k] x[r, h, k].  General form: any sizes, one wave per sixteen outputs
// of a (row, head); sums in fp32.
struct FromProjection {                    // fp32 projections of the pass, rounded to what the state computes in
    const float* in;
    int ld, off, head_ld;
    bool round, wide;                      // wide: every vector is 16-byte aligned
    struct Raw {
        t12_f32x4 a, b;
        __device__ __forceinline__ void unpack(float (&v)[8]) const
        {
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = e < 4 ? a[e & 3] : b[e & 3];
        }
    };
    __device__ __forceinline__ Raw request(int r, int h, int k) const
    {
        const float* x = in + (size_t)r * ld + off + h * head_ld + k;
        return {*(const t12_f32x4*)x, *(const t12_f32x4*)(x + 4)};
    }
    __device__ __forceinline__ float at(int r, int h, int k) const
    {
        const float v = in[(size_t)r * ld + off + h * head_ld + k];
        return round ? t12_bf16_to_f32(t12_f32_to_bf16(v)) : v;
    }
    // eight consecutive elements; left: how many there are
    __device__ __forceinline__ void at8(int r, int h, int k, int left, float (&v)[8]) const
    {
        const float* x = in + (size_t)r * ld + off + h * head_ld + k;
        if (left >= 8 && (uintptr_t)x % 16 == 0) {
            const t12_f32x4 a = *(const t12_f32x4*)x, b = *(const t12_f32x4*)(x + 4);
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = e < 4 ? a[e & 3] : b[e & 3];
            return;
        }
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] = e < left ? x[e] : 0.0f;
    }
    template <int ROWS>
    __device__ __forceinline__ void stage(uint4* lds, int r0, int n, int h, int units, int K) const
    {
        if (wide) stage_rows_ahead<ROWS, 1>(*this, lds, r0, n, h, units, K);
        else stage_rows<ROWS>(*this, lds, r0, n, h, units, K);
    }
};
template <typename T>
struct FromRows {                          // mean latents [row][head][rank_p]
    const T* x;
    int heads, head_ld;
    struct Raw {
        uint4 w;
        __device__ __forceinline__ void unpack(float (&v)[8]) const
        {
            const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = __builtin_bit_cast(float, e & 1 ? u[e >> 1] & 0xFFFF0000u : u[e >> 1] << 16);
        }
    };
    __device__ __forceinline__ Raw request(int r, int h, int k) const { return {*(const uint4*)(x + ((size_t)r * heads + h) * head_ld + k)}; }
    __device__ __forceinline__ float at(int r, int h, int k) const { return from_cache(x[((size_t)r * heads + h) * head_ld + k]); }
    // (bf16 rows are padded: eight elements are always there)
    __device__ __forceinline__ void at8(int r, int h, int k, int left, float (&v)[8]) const
    {
        const uint4 w = *(const uint4*)(x + ((size_t)r * heads + h) * head_ld + k);
        const uint32_t u[4] = {w.x, w.y, w.z, w.w};
#pragma unroll
        for (int e = 0; e < 8; e++)
            v[e] = e < left ? __builtin_bit_cast(float, e & 1 ? u[e >> 1] & 0xFFFF0000u : u[e >> 1] << 16) : 0.0f;
    }
    template <int ROWS>
    __device__ __forceinline__ void stage(uint4* lds, int r0, int n, int h, int units, int K) const
    {
        stage_rows_ahead<ROWS, 2>(*this, lds, r0, n, h, units, K);
    }
};
struct FromParts {                         // sums of stretches of keys, put together here
    const float* sums;
    const float2* parts;
    int heads, head_ld, splits;
    __device__ __forceinline__ float at(int r, int h, int k) const
    {
        const size_t unit = (size_t)r * heads + h;
        float top = -1e30f, total = 0.0f, v = 0.0f;
        for (int z = 0; z < splits; z++) top = fmaxf(top, parts[unit * splits + z].x);
        for (int z = 0; z < splits; z++) {
            const float w = exp2f(parts[unit * splits + z].x - top);
            total += w * parts[unit * splits + z].y;
            v += w * sums[(unit * splits + z) * head_ld + k];
        }
        return t12_bf16_to_f32(t12_f32_to_bf16(v / total));
    }
    __device__ __forceinline__ void at8(int r, int h, int k, int left, float (&v)[8]) const
    {
        const size_t unit = (size_t)r * heads + h;
        const float2* q = parts + unit * splits;
        const float* x = sums + unit * splits * head_ld + k;          // (rows are padded: eight elements are always there)
        constexpr int G = 8;                                           // stretches whose loads are in flight together
        float top = -1e30f, total = 0.0f;
        for (int z0 = 0; z0 < splits; z0 += G) {
            float2 w[G];
#pragma unroll
            for (int z = 0; z < G; z++) w[z] = q[min(z0 + z, splits - 1)];
#pragma unroll
            for (int z = 0; z < G; z++) top = fmaxf(top, w[z].x);
        }
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] = 0.0f;
        for (int z0 = 0; z0 < splits; z0 += G) {
            float2 w[G];
            t12_f32x4 a[G], b[G];
#pragma unroll
            for (int z = 0; z < G; z++) {
                const int zz = min(z0 + z, splits - 1);
                w[z] = q[zz];
                a[z] = *(const t12_f32x4*)(x + (size_t)zz * head_ld);
                b[z] = *(const t12_f32x4*)(x + (size_t)zz * head_ld + 4);
            }
#pragma unroll
            for (int z = 0; z < G; z++) {
                const float f = z0 + z < splits ? exp2f(w[z].x - top) : 0.0f;
                total += f * w[z].y;
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] += f * (e < 4 ? a[z][e & 3] : b[z][e & 3]);
            }
        }
        const float inv = 1.0f / total;
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] = e < left ? v[e] * inv : 0.0f;
    }
    template <int ROWS>
    __device__ __forceinline__ void stage(uint4* lds, int r0, int n, int h, int units, int K) const
    {
        if (n > 1 || units > 64) {
            stage_rows<ROWS>(*this, lds, r0, n, h, units, K);
            return;
        }
        // a single row: the waves take the stretches in turn, and their sums are put together
        __shared__ float share[4][64][8];
        __shared__ float2 weight[4];
        const int u = threadIdx.x & 63, wave = threadIdx.x >> 6;
        const float2* q = parts + (size_t)h * splits;
        const float* x = sums + (size_t)h * splits * head_ld + min(u * 8, head_ld - 8);
        constexpr int G = 8;                               // all stretches there can be: 4 x G
        float2 w[G];
        t12_f32x4 a[G], b[G];
#pragma unroll
        for (int z = 0; z < G; z++) {
            const int zz = min(wave + 4 * z, splits - 1);
            w[z] = q[zz];
            a[z] = *(const t12_f32x4*)(x + (size_t)zz * head_ld);
            b[z] = *(const t12_f32x4*)(x + (size_t)zz * head_ld + 4);
        }
        float top = -1e30f, total = 0.0f, v[8];
#pragma unroll
        for (int z = 0; z < G; z++) top = fmaxf(top, w[z].x);
#pragma unroll
        for (int e = 0; e < 8; e++) v[e] = 0.0f;
#pragma unroll
        for (int z = 0; z < G; z++) {
            const float f = wave + 4 * z < splits ? exp2f(w[z].x - top) : 0.0f;
            total += f * w[z].y;
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] += f * (e < 4 ? a[z][e & 3] : b[z][e & 3]);
        }
#pragma unroll
        for (int e = 0; e < 8; e++) share[wave][u][e] = v[e];
        if (u == 0) weight[wave] = make_float2(top, total);
        __syncthreads();
        for (int c = threadIdx.x & 15; c < units; c += 16) {
            const int r = threadIdx.x >> 4;
            float y[8], all = -1e30f, sum = 0.0f;
#pragma unroll
            for (int g = 0; g < 4; g++) all = fmaxf(all, weight[g].x);
#pragma unroll
            for (int e = 0; e < 8; e++) y[e] = 0.0f;
#pragma unroll
            for (int g = 0; g < 4; g++) {
                const float f = exp2f(weight[g].x - all);
                sum += f * weight[g].y;
#pragma unroll
                for (int e = 0; e < 8; e++) y[e] += f * share[g][c][e];
            }
            const float inv = 1.0f / sum;
#pragma unroll
            for (int e = 0; e < 8; e++) y[e] = c * 8 + e < K ? y[e] * inv : 0.0f;
            for (int q = r; q < ROWS; q += 16) lds[slot<ROWS>(c, q)] = q == 0 ? paired(y) : make_uint4(0, 0, 0, 0);
        }
    }
};
static_assert(MAX_SPLITS <= 32, "a single row's stretches are taken by four waves, eight each");

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
    __device__ __forceinline__ float factor(int, int) const { return 1.0f; }
    // four consecutive outputs (bf16), of which `left` exist; wide: always all of them, at aligned places
    __device__ __forceinline__ void put4(int r, int h, int m, int left, t12_f32x4 v, bool) const
    {
        T* o = q + ((size_t)r * heads + h) * row_p + m;
        const uint2 w = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
        if (left >= 4) *(uint2*)o = w;
        else
            for (int e = 0; e < left; e++) o[e] = to_cache<T>(v[e]);
    }
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
    __device__ __forceinline__ float factor(int r, int h) const { return t12_sigmoid(in[(size_t)r * ld + g_off + h]); }
    __device__ __forceinline__ void put4(int r, int h, int m, int left, t12_f32x4 v, bool wide) const
    {
        T* o = out + (size_t)r * out_ld + h * vdim + m;
        const uint2 w = make_uint2(pack_bf16(v[0], v[1]), pack_bf16(v[2], v[3]));
        if (wide) *(uint2*)o = w;
        else
            for (int e = 0; e < min(left, 4); e++) o[e] = to_cache<T>(v[e]);
    }
};

// ---- the product per head on the matrix cores: K a multiple of 32, base_exp in 0..240.  A workgroup has 16 NT rows of a head and a
// stretch of its outputs, 64 MT at a time, a wave 16 MT of them; a lane takes 32 consecutive columns of MT weight rows per
// 128-column block (two sign/mantissa pieces, one of nibbles), which feed four MFMAs each with the activations in the same order.
// The accumulators start from the escapes' corrections, whose list for the workgroup's rows is brought into LDS ahead (a list or a
// stretch too long for it is read where it lies).  STORE: the workgroups with blockIdx.y == 0 store the rows of their tile
// (latent attention's cache) instead.
// Dynamic LDS: activations, 16-byte units of eight columns (paired like the decoded weights), slot<16 NT>.
template <int NT, int MT, bool STORE, typename IN, typename OUT>
__global__ __launch_bounds__(256) void heads_matrix_kernel(T12Segment w, int M, int K, IN in, OUT out, int n, int wide, const LatentParams lp)
{
    extern __shared__ uint4 lds[];
    constexpr int ROWS = 16 * NT, LIST_ROWS = 512, LIST = 512;
    __shared__ int list_row[LIST_ROWS + 1];                // first entry of every output row
    __shared__ float2 list[LIST];                          // (column, correct - wrong)
    const int r0 = blockIdx.x * ROWS, h = (int)blockIdx.y - (STORE ? 1 : 0), tid = threadIdx.x;
    if (STORE && h < 0) {
        for (int r = r0 + blockIdx.z; r < min(r0 + ROWS, n); r += gridDim.z) store_row<uint16_t>(lp, r);
        return;
    }
    const int lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), l = lane & 15, g4 = lane >> 4;
    const int blocks = (K + 127) / 128, units = blocks * 16, tiles = (M + 64 * MT - 1) / (64 * MT);
    const int per = (tiles + (int)gridDim.z - 1) / (int)gridDim.z, t0 = blockIdx.z * per, t1 = min(t0 + per, tiles);
    if (t0 >= t1) return;
    const uint32_t be2 = t12_opaque(((uint32_t)w.base_exp << 7) | ((uint32_t)w.base_exp << 23));
    uint4 s0[MT], s1[MT], gg[MT];
    auto request = [&](int t, int b) {                     // (columns past K: the row's first ones again, times zero)
        const int k = b * 128 + 32 * g4, at = k < K ? k : 0;
#pragma unroll
        for (int i = 0; i < MT; i++) {
            const size_t row = ((size_t)h * M + min(((t * 4 + wave) * MT + i) * 16 + l, M - 1)) * K;
            s0[i] = *(const uint4*)(w.sm + row + at);
            s1[i] = *(const uint4*)(w.sm + row + at + 16);
            gg[i] = *(const uint4*)(w.gr + (row + at) / 2);
        }
    };
    request(t0, 0);
    const int out0 = t0 * 64 * MT, outs = min(M - out0, (t1 - t0) * 64 * MT);
    bool listed = false;
    if (w.row_off) {
        const int* rows = w.row_off + (size_t)h * M + out0;
        const int e0 = rows[0], e1 = rows[outs];
        listed = outs <= LIST_ROWS && e1 - e0 <= LIST;
        if (listed) {
            for (int i = tid; i <= outs; i += 256) list_row[i] = rows[i] - e0;
            for (int i = tid; i < e1 - e0; i += 256)
                list[i] = make_float2(__builtin_bit_cast(float, w.cols[e0 + i]),
                                      t12_bf16_to_f32((uint16_t)w.correct[e0 + i]) - t12_bf16_to_f32((uint16_t)w.wrong[e0 + i]));
        }
    }
    float factor[NT];
#pragma unroll
    for (int c = 0; c < NT; c++) factor[c] = out.factor(min(r0 + c * 16 + l, n - 1), h);
    in.template stage<ROWS>(lds, r0, n, h, units, K);
    __syncthreads();
    auto correct = [&](float (&a)[NT], int k, float delta) {
        const int e = k & 7;
#pragma unroll
        for (int c = 0; c < NT; c++)
            a[c] += delta * t12_bf16_to_f32(((const uint16_t*)(lds + slot<ROWS>(k >> 3, c * 16 + l)))[(e & 3) * 2 + (e >> 2)]);
    };
    for (int t = t0; t < t1; t++) {
        const int m0 = (t * 4 + wave) * MT * 16 + 4 * g4;  // the first four of this lane's outputs
        t12_f32x4 acc[MT][NT];
#pragma unroll
        for (int i = 0; i < MT; i++)
#pragma unroll
            for (int c = 0; c < NT; c++) acc[i][c] = (t12_f32x4)(0.0f);
        if (w.row_off) {
#pragma unroll
            for (int i = 0; i < MT; i++)
#pragma unroll
                for (int r = 0; r < 4; r++) {
                    const int m = m0 + i * 16 + r;
                    float a[NT] = {};
                    if (listed) {
                        const int q0 = list_row[min(m - out0, outs)], q1 = list_row[min(m + 1 - out0, outs)];
                        for (int q = q0; q < q1; q++) correct(a, __builtin_bit_cast(int, list[q].x), list[q].y);
                    } else if (m < M) {
                        const int* at = w.row_off + (size_t)h * M + m;
                        for (int q = at[0]; q < at[1]; q++)
                            correct(a, w.cols[q], t12_bf16_to_f32((uint16_t)w.correct[q]) - t12_bf16_to_f32((uint16_t)w.wrong[q]));
                    }
#pragma unroll
                    for (int c = 0; c < NT; c++) acc[i][c][r] = a[c];
                }
        }
        for (int b = 0; b < blocks; b++) {
            uint32_t d[MT][4][4];
#pragma unroll
            for (int i = 0; i < MT; i++) {
                t12_decode8(s0[i].x, s0[i].y, gg[i].x, be2, d[i][0]);
                t12_decode8(s0[i].z, s0[i].w, gg[i].y, be2, d[i][1]);
                t12_decode8(s1[i].x, s1[i].y, gg[i].z, be2, d[i][2]);
                t12_decode8(s1[i].z, s1[i].w, gg[i].w, be2, d[i][3]);
            }
            if (b + 1 < blocks) request(t, b + 1);
            else request(min(t + 1, t1 - 1), 0);
#pragma unroll
            for (int e = 0; e < 4; e++)
#pragma unroll
                for (int c = 0; c < NT; c++) {
                    const t12_bf16x8 x = __builtin_bit_cast(t12_bf16x8, lds[slot<ROWS>(b * 16 + 4 * g4 + e, c * 16 + l)]);
#pragma unroll
                    for (int i = 0; i < MT; i++)
                        acc[i][c] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(
                            __builtin_bit_cast(t12_bf16x8, make_uint4(d[i][e][0], d[i][e][1], d[i][e][2], d[i][e][3])), x, acc[i][c], 0, 0, 0);
                }
        }
#pragma unroll
        for (int c = 0; c < NT; c++) {
            const int r = r0 + c * 16 + l;
#pragma unroll
            for (int i = 0; i < MT; i++)
                if (r < n && m0 + i * 16 < M) out.put4(r, h, m0 + i * 16, M - m0 - i * 16, acc[i][c] * factor[c], wide);
        }
    }
}

bool matrix_product(const T12Segment& w, int K) { return K % 32 == 0 && K <= 512 && w.base_exp >= 0 && w.base_exp <= 240 && (!w.row_off || w.wrong); }

template <bool STORE, typename IN, typename OUT>
void launch_heads(const T12Segment& w, int M, int K, const IN& in, const OUT& out, int wide, const LatentParams& p, hipStream_t st)
{
    // rows per workgroup: 64 for prompt passes, 16 for decode steps; outputs in as few stretches as still give the chip enough
    // workgroups (the activations of a tile are staged once per stretch)
    const int heads = p.a.heads, units = (K + 127) / 128 * 16;
    const bool prompt = p.n > 128 && K <= 512;
    const int rows = prompt ? 64 : 16, tiles = (M + (prompt ? 127 : 63)) / (prompt ? 128 : 64);
    const int groups = (p.n + rows - 1) / rows * heads, stretches = std::min(tiles, ((prompt ? 511 : 255) + groups) / groups);
    const dim3 grid((p.n + rows - 1) / rows, heads + (STORE ? 1 : 0), stretches);
    const size_t lds = (size_t)units * rows * 16;
    if constexpr (STORE) hipLaunchKernelGGL((heads_matrix_kernel<1, 1, true, IN, OUT>), grid, dim3(256), lds, st, w, M, K, in, out, p.n, wide, p);
    else if (prompt) {
        static std::once_flag once[16];                    // the attribute is per device
        int dev = 0;
        if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 16) dev = 0;
        std::call_once(once[dev], [&] {
            (void)hipFuncSetAttribute((const void*)heads_matrix_kernel<4, 2, false, IN, OUT>, hipFuncAttributeMaxDynamicSharedMemorySize, 64 * 1024);
        });
        hipLaunchKernelGGL((heads_matrix_kernel<4, 2, false, IN, OUT>), grid, dim3(256), lds, st, w, M, K, in, out, p.n, wide, p);
    } else hipLaunchKernelGGL((heads_matrix_kernel<1, 1, false, IN, OUT>), grid, dim3(256), lds, st, w, M, K, in, out, p.n, wide, p);
}

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

// ---- attention on the matrix cores.  Everything transposed, so that no operand is moved between lanes:
//
//   S^T = K Q^T    keys = A rows from LDS, columns -- (row, head) pairs -- = B from registers; lane (n, g4) = (lane % 16,
//                  lane / 16) receives keys 4 g4 .. 4 g4 + 3 of both 16-key halves of a block for column n;
//   P              softmax in fp32 with a running maximum per column; the weights enter the product as two bf16 (16 bits);
//   O^T += C^T P^T the lane's weights are its B operand as they are; A = the block's latents turned around by the LDS's
//                  transposing reads, four keys of one channel per read.
//
// Workgroup = CT x 2 waves on 16 CT columns.  The two waves of a column tile take one block of keys each for the scores, tell each
// other those, and take one half of the channels each for the sums over both blocks' keys.  Blocks come into LDS as they lie
// in the cache (their pieces are already spread over the banks), the next two while two are worked on.
// run: columns run over all (row, head) pairs of the sequence; else blockIdx.z is the row.  blockIdx.y: stretch of keys.
// Dynamic LDS: 2 x 2 blocks, then the scores [CT x 2][2][64] x 16 bytes.
typedef __attribute__((ext_vector_type(4))) short s16x4;
struct Turned {                            // eight keys of one channel: a lane's A operand
    s16x4 half[2];
};

// Transposing reads of N channel tiles, both key halves of a block.  Written out because the compiler puts a wait for all
// outstanding copies into LDS ahead of the builtin: the next blocks could not be on their way.  The reads have landed when
// the statement ends.
template <int AT, int ROWB>
__device__ __forceinline__ void read_turned(const uint32_t (&at)[4], Turned (&v)[4])
{
    asm volatile("ds_read_b64_tr_b16 %0, %8 offset:%12\n\t"
                 "ds_read_b64_tr_b16 %1, %8 offset:%13\n\t"
                 "ds_read_b64_tr_b16 %2, %9 offset:%12\n\t"
                 "ds_read_b64_tr_b16 %3, %9 offset:%13\n\t"
                 "ds_read_b64_tr_b16 %4, %10 offset:%12\n\t"
                 "ds_read_b64_tr_b16 %5, %10 offset:%13\n\t"
                 "ds_read_b64_tr_b16 %6, %11 offset:%12\n\t"
                 "ds_read_b64_tr_b16 %7, %11 offset:%13\n\t"
                 "s_waitcnt lgkmcnt(0)"
                 : "=&v"(v[0].half[0]), "=&v"(v[0].half[1]), "=&v"(v[1].half[0]), "=&v"(v[1].half[1]), "=&v"(v[2].half[0]),
                   "=&v"(v[2].half[1]), "=&v"(v[3].half[0]), "=&v"(v[3].half[1])
                 : "v"(at[0]), "v"(at[1]), "v"(at[2]), "v"(at[3]), "n"(AT), "n"(AT + 16 * ROWB)
                 : "memory");
}
template <int AT, int ROWB>
__device__ __forceinline__ void read_turned(const uint32_t (&at)[2], Turned (&v)[2])
{
    asm volatile("ds_read_b64_tr_b16 %0, %4 offset:%6\n\t"
                 "ds_read_b64_tr_b16 %1, %4 offset:%7\n\t"
                 "ds_read_b64_tr_b16 %2, %5 offset:%6\n\t"
                 "ds_read_b64_tr_b16 %3, %5 offset:%7\n\t"
                 "s_waitcnt lgkmcnt(0)"
                 : "=&v"(v[0].half[0]), "=&v"(v[0].half[1]), "=&v"(v[1].half[0]), "=&v"(v[1].half[1])
                 : "v"(at[0]), "v"(at[1]), "n"(AT), "n"(AT + 16 * ROWB)
                 : "memory");
}

// acc[e] += (channel tiles J, J + 1, ... of a block, N at a time) x both limbs of the weights
template <int EH, int N, int ROWB, int J = 0>
__device__ __forceinline__ void add_block(const uint32_t (&at)[N], t12_bf16x8 hi, t12_bf16x8 lo, t12_f32x4 (&acc)[EH])
{
    Turned v[N];
    read_turned<J / 4 * 128, ROWB>(at, v);
#pragma unroll
    for (int e = 0; e < N; e++) acc[J + e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(t12_bf16x8, v[e]), hi, acc[J + e], 0, 0, 0);
#pragma unroll
    for (int e = 0; e < N; e++) acc[J + e] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(t12_bf16x8, v[e]), lo, acc[J + e], 0, 0, 0);
    if constexpr (J + N < EH) add_block<EH, N, ROWB, J + N>(at, hi, lo, acc);
}

template <int RP, int CT>
__global__ __launch_bounds__(CT * 128, 2) void latent_matrix_kernel(const LatentParams p)
{
    constexpr int DT = RP + 2, EH = RP, ROWB = DT * 64, BLKB = BLK * ROWB, NW = CT * 2, N = EH < 4 ? EH : 4;
    extern __shared__ uint4 lds4[];
    uint8_t* lds = (uint8_t*)lds4;
    t12_f32x4* told = (t12_f32x4*)(lds + 4 * BLKB);
    const T12LatentAttn& a = p.a;
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6), n = lane & 15, g4 = lane >> 4;
    const int ct = wave % CT, ph = wave / CT;
    T12Row row = p.rows[p.run ? 0 : blockIdx.z];           // (the same for the workgroup, which the compiler cannot know)
    row.position = __builtin_amdgcn_readfirstlane(row.position);
    row.slot = __builtin_amdgcn_readfirstlane(row.slot);
    const int ncol = p.run ? p.n * a.heads : a.heads, first = blockIdx.x * CT * 16, col = first + ct * 16 + n;
    const size_t unit = (p.run ? 0 : (size_t)blockIdx.z * a.heads) + min(col, ncol - 1);
    const int pos = row.position + (p.run ? min(col, ncol - 1) / a.heads : 0);
    const int last = row.position + (p.run ? (min(first + CT * 16, ncol) - 1) / a.heads : 0);
    const int blocks = last / BLK + 1, per = ((blocks + 1) / 2 + p.splits - 1) / p.splits * 2;
    const int b0 = min((int)blockIdx.y * per, blocks), b1 = min(b0 + per, blocks);
    const uint8_t* cache = (const uint8_t*)a.cache + (size_t)(row.slot >> 1) * a.cache_elems * 2;
    // one block is BLKB / 1024 pieces of a wave's load; the waves share the pieces of both blocks
    auto request = [&](int b, int buf) {
#pragma unroll
        for (int i = 0; i < 2 * BLKB / 1024 / NW; i++) {
            const int piece = wave + i * NW, which = piece / (BLKB / 1024), at = piece % (BLKB / 1024) * 1024;
            const uint8_t* src = cache + (size_t)min(b + which, blocks - 1) * BLKB + at;
            __builtin_amdgcn_global_load_lds((const __attribute__((address_space(1))) void*)(src + lane * 16u),
                                             (__attribute__((address_space(3))) void*)(lds + (buf * 2 + which) * BLKB + at), 16, 0, 0);
        }
    };
    static_assert(2 * BLKB / 1024 % NW == 0, "the waves share the pieces evenly");
    if (b0 < b1) request(b0, 0);
    t12_bf16x8 Q[DT];
    const uint16_t* q = (const uint16_t*)p.q + unit * a.row_p + 8 * g4;
#pragma unroll
    for (int s = 0; s < DT; s++) Q[s] = *(const t12_bf16x8*)(q + s * 32);
    t12_f32x4 acc[EH];
#pragma unroll
    for (int e = 0; e < EH; e++) acc[e] = (t12_f32x4)(0.0f);
    float top = -1e30f, sum = 0.0f;
    const float scale = a.scale * 1.44269504088896341f;
    // offsets of this lane within a block: keys for the scores (two pieces, the rest by constants), turned reads (N tiles)
    int ko[2];
#pragma unroll
    for (int s = 0; s < 2; s++) ko[s] = n * ROWB + ((4 * s + g4) ^ turn(n)) * 16;
    const int vk = 4 * g4 + (n >> 2);                      // key of this lane's turned reads
    const uint32_t lds_base = (uint32_t)(uintptr_t)(__attribute__((address_space(3))) uint8_t*)lds;
    uint32_t vo[N];
#pragma unroll
    for (int e = 0; e < N; e++) {
        const int tile = ph * EH + e;
        vo[e] = lds_base + vk * ROWB + (tile >> 2) * 128 + ((2 * (tile & 3) + ((n & 3) >> 1)) ^ turn(vk)) * 16 + (n & 1) * 8;
    }
    int buf = 0;
    for (int b = b0; b < b1; b += 2) {
        __builtin_amdgcn_s_waitcnt(0x0F70);                // vmcnt(0): the blocks have landed
        __syncthreads();                                   // (the other buffer was last read before this barrier)
        if (b + 2 < b1) request(b + 2, buf ^ 1);
        const uint8_t* blk = lds + (buf * 2 + ph) * BLKB;
        t12_f32x4 S[2];
        S[0] = S[1] = (t12_f32x4)(0.0f);
        constexpr int G = DT % 3 == 0 ? 3 : 2;             // steps whose keys are read together, one group ahead
        t12_bf16x8 K[2][G][2];
        auto keys = [&](int g) {
#pragma unroll
            for (int s = 0; s < G; s++)
#pragma unroll
                for (int u = 0; u < 2; u++) K[g & 1][s][u] = *(const t12_bf16x8*)(blk + ko[(g * G + s) & 1] + ((g * G + s) >> 1) * 128 + u * 16 * ROWB);
        };
        keys(0);
#pragma unroll
        for (int g = 0; g < DT / G; g++) {
            if (g + 1 < DT / G) keys(g + 1);
            __builtin_amdgcn_sched_barrier(0);
#pragma unroll
            for (int s = 0; s < G; s++)
#pragma unroll
                for (int u = 0; u < 2; u++) S[u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(K[g & 1][s][u], Q[g * G + s], S[u], 0, 0, 0);
        }
        // keys past the column's position, and a whole block past the stretch, get no weight
        const int left = b + ph < b1 ? pos - (b + ph) * BLK - 4 * g4 : -1;
#pragma unroll
        for (int u = 0; u < 2; u++) {
#pragma unroll
            for (int i = 0; i < 4; i++) S[u][i] = u * 16 + i <= left ? S[u][i] * scale : -INFINITY;
            told[(wave * 2 + u) * 64 + lane] = S[u];
        }
        __syncthreads();
        const int other = (wave + CT) % NW;
        float w[2][8], best = top;
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const t12_f32x4 theirs = told[(other * 2 + u) * 64 + lane];
#pragma unroll
            for (int i = 0; i < 4; i++) {
                w[0][u * 4 + i] = ph == 0 ? S[u][i] : theirs[i];
                w[1][u * 4 + i] = ph == 0 ? theirs[i] : S[u][i];
                best = fmaxf(best, fmaxf(S[u][i], theirs[i]));
            }
        }
        best = fmaxf(best, __shfl_xor(best, 16, 64));
        best = fmaxf(best, __shfl_xor(best, 32, 64));
        const float back = __builtin_amdgcn_exp2f(top - best);
        const bool grew = __any(best > top);
        top = best;
        sum *= back;
        t12_bf16x8 hi8[2], lo8[2];
#pragma unroll
        for (int z = 0; z < 2; z++) {
            uint32_t hi[4], lo[4];
#pragma unroll
            for (int i = 0; i < 8; i++) {
                w[z][i] = __builtin_amdgcn_exp2f(w[z][i] - best);
                sum += w[z][i];
            }
#pragma unroll
            for (int i = 0; i < 4; i++) {
                hi[i] = pack_bf16(w[z][2 * i], w[z][2 * i + 1]);
                lo[i] = pack_bf16(w[z][2 * i] - __builtin_bit_cast(float, hi[i] << 16),
                                  w[z][2 * i + 1] - __builtin_bit_cast(float, hi[i] & 0xFFFF0000u));
            }
            hi8[z] = __builtin_bit_cast(t12_bf16x8, make_uint4(hi[0], hi[1], hi[2], hi[3]));
            lo8[z] = __builtin_bit_cast(t12_bf16x8, make_uint4(lo[0], lo[1], lo[2], lo[3]));
        }
        if (grew) {
#pragma unroll
            for (int e = 0; e < EH; e++) acc[e] *= back;
        }
#pragma unroll
        for (int z = 0; z < 2; z++) {
            uint32_t at[N];
#pragma unroll
            for (int e = 0; e < N; e++) at[e] = vo[e] + (buf * 2 + z) * BLKB;
            add_block<EH, N, ROWB>(at, hi8[z], lo8[z], acc);
        }
        buf ^= 1;
    }
    sum += __shfl_xor(sum, 16, 64);
    sum += __shfl_xor(sum, 32, 64);
    if (col >= ncol) return;
    const float inv = p.parts ? 1.0f : 1.0f / sum;
#pragma unroll
    for (int e = 0; e < EH; e++) {
        const int c = (ph * EH + e) * 16 + 4 * g4;
        const t12_f32x4 s = acc[e] * inv;
        if (p.parts) *(t12_f32x4*)((float*)p.mean + (unit * p.splits + blockIdx.y) * a.rank_p + c) = s;
        else *(uint2*)((uint16_t*)p.mean + unit * a.rank_p + c) = make_uint2(pack_bf16(s[0], s[1]), pack_bf16(s[2], s[3]));
    }
    if (p.parts && ph == 0 && g4 == 0) p.parts[unit * p.splits + blockIdx.y] = make_float2(top, sum);
}

constexpr int PART_UNITS = 16384;          // (row, head, stretch) sums a pass keeps when it keeps more than one stretch

template <int RP, int CT>
int launch_matrix(const LatentParams& p, int columns, hipStream_t st)
{
    constexpr size_t lds = (size_t)4 * BLK * (RP + 2) * 64 + CT * 4096;
    if (lds > 64 * 1024) {
        static std::once_flag once[16];                    // the attribute is per device
        int dev = 0;
        if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 16) dev = 0;
        hipError_t e = hipSuccess;
        std::call_once(once[dev], [&] { e = hipFuncSetAttribute((const void*)latent_matrix_kernel<RP, CT>, hipFuncAttributeMaxDynamicSharedMemorySize, (int)lds); });
        if (e != hipSuccess) {
            t12_set_error("t12_latent_attention: cannot reserve %zu bytes of LDS", lds);
            return T12_ELAUNCH;
        }
    }
    hipLaunchKernelGGL((latent_matrix_kernel<RP, CT>), dim3((columns + CT * 16 - 1) / (CT * 16), p.splits, p.run ? 1 : p.n), dim3(CT * 128), lds, st, p);
    return T12_OK;
}

template <int CT>
int launch_matrix_rank(const LatentParams& p, int columns, hipStream_t st)
{
    switch (p.a.rank_p) {
        case 64: return launch_matrix<2, CT>(p, columns, st);
        case 128: return launch_matrix<4, CT>(p, columns, st);
        case 256: return launch_matrix<8, CT>(p, columns, st);
        default: return launch_matrix<16, CT>(p, columns, st);
    }
}

int launch_fast(LatentParams p, int max_position, void* out, int out_ld, hipStream_t st)
{
    const T12LatentAttn& a = p.a;
    const int qd = a.dim + a.rot_dim;
    const bool wide = (p.ld | a.q_off | qd) % 4 == 0 && (uintptr_t)p.in % 16 == 0;
    const FromProjection q = {p.in, p.ld, a.q_off, qd, true, wide};
    const ToQuery<uint16_t> to = {(uint16_t*)p.q, a.heads, a.row_p};
    const bool product = matrix_product(*a.k_up, a.dim);
    if (product && p.n <= 16) launch_heads<true>(*a.k_up, a.rank, a.dim, q, to, 1, p, st);
    else {
        hipLaunchKernelGGL(latent_store_kernel<uint16_t>, dim3(p.n), dim3(256), 0, st, p);
        if (product) launch_heads<false>(*a.k_up, a.rank, a.dim, q, to, 1, p, st);
        else hipLaunchKernelGGL((heads_general_kernel<FromProjection, ToQuery<uint16_t>>), dim3(p.n, a.heads, (a.rank + 63) / 64), dim3(256), 0, st,
                           *a.k_up, a.heads, a.rank, a.dim, q, to, p.n);
    }
    // stretches of keys: as many as it takes to give every CU a workgroup, each at least the two blocks of one step
    const int columns = p.run ? p.n * a.heads : a.heads, ct = columns > 32 ? 4 : columns > 16 ? 2 : 1;
    const int groups = (columns + ct * 16 - 1) / (ct * 16) * (p.run ? 1 : p.n), blocks = max_position / BLK + 1;
    p.splits = std::max(1, std::min({(256 + groups - 1) / groups, (blocks + 1) / 2, MAX_SPLITS, PART_UNITS / (p.n * a.heads)}));
    const bool parts = !p.run || p.splits > 1;
    if (!parts) p.parts = nullptr;
    const int rc = ct == 4 ? launch_matrix_rank<4>(p, columns, st) : ct == 2 ? launch_matrix_rank<2>(p, columns, st) : launch_matrix_rank<1>(p, columns, st);
    if (rc) return rc;
    const ToGated<uint16_t> gated = {(uint16_t*)out, out_ld, a.vdim, p.in, p.ld, a.g_off};
    const bool fast = matrix_product(*a.v_up, a.rank), aligned = a.vdim % 4 == 0 && out_ld % 4 == 0 && (uintptr_t)out % 8 == 0;
    const dim3 general(p.n, a.heads, (a.vdim + 63) / 64);
    if (parts) {
        const FromParts mean = {(const float*)p.mean, p.parts, a.heads, a.rank_p, p.splits};
        if (fast) launch_heads<false>(*a.v_up, a.vdim, a.rank, mean, gated, aligned, p, st);
        else
            hipLaunchKernelGGL((heads_general_kernel<FromParts, ToGated<uint16_t>>), general, dim3(256), 0, st, *a.v_up, a.heads, a.vdim, a.rank,
                               mean, gated, p.n);
    } else {
        const FromRows<uint16_t> mean = {(const uint16_t*)p.mean, a.heads, a.rank_p};
        if (fast) launch_heads<false>(*a.v_up, a.vdim, a.rank, mean, gated, aligned, p, st);
        else
            hipLaunchKernelGGL((heads_general_kernel<FromRows<uint16_t>, ToGated<uint16_t>>), general, dim3(256), 0, st, *a.v_up, a.heads, a.vdim,
                               a.rank, mean, gated, p.n);
    }
    return T12_OK;
}

template <typename T>
void launch_general(const LatentParams& p, void* out, int out_ld, hipStream_t st)
{
    const T12LatentAttn& a = p.a;
    const FromProjection q = {p.in, p.ld, a.q_off, a.dim + a.rot_dim, sizeof(T) == 2, false};
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
    a->matrix = a->elem_bytes == 2 && a->rank <= 512 && a->rot_dim <= 64;
    if (a->matrix) {
        a->rank_p = 64;
        while (a->rank_p < a->rank) a->rank_p *= 2;
        a->row_p = a->rank_p + 64;
    } else {
        a->rank_p = (a->rank + 31) / 32 * 32;
        a->row_p = a->rank_p + (a->rot_dim + 31) / 32 * 32;
    }
    const size_t blocks = (max_positions + BLK - 1) / BLK, el = a->elem_bytes;
    a->cache_elems = blocks * BLK * a->row_p;
    const size_t units = (size_t)rows * a->heads, q = units * a->row_p * el;
    size_t mean = (units * a->rank_p * el + 3) / 4;
    if (a->matrix) mean = std::max(units, (size_t)PART_UNITS) * (a->rank_p + 2);       // (fp32 sums of stretches, their weights)
    a->work_floats = (q + 15) / 16 * 4 + (mean + 3) / 4 * 4;
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
    if (a->matrix) {
        T12_REQUIRE(a->elem_bytes == 2 && (a->rank_p == 64 || a->rank_p == 128 || a->rank_p == 256 || a->rank_p == 512) && a->row_p == a->rank_p + 64 &&
                        (uintptr_t)a->cache % 16 == 0 && a->cache_elems % 8 == 0,
                    "t12_latent_attention: t12_latent_plan has not been called, or the cache is not aligned");
        p.parts = (float2*)((float*)p.mean + std::max((size_t)n * a->heads, (size_t)PART_UNITS) * a->rank_p);
        const int rc = launch_fast(p, max_position, out, out_ld, st);
        if (rc) return rc;
        T12_CHECK_LAUNCH("t12_latent_attention");
        return T12_OK;
    }
    if (a->elem_bytes == 4) hipLaunchKernelGGL(latent_store_kernel<float>, dim3(n), dim3(256), 0, st, p);
    else hipLaunchKernelGGL(latent_store_kernel<uint16_t>, dim3(n), dim3(256), 0, st, p);
    if (a->elem_bytes == 4) launch_general<float>(p, out, out_ld, st);
    else launch_general<uint16_t>(p, out, out_ld, st);
    T12_CHECK_LAUNCH("t12_latent_attention");
    return T12_OK;
}

}  // extern "C"
