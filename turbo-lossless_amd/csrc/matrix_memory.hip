// Matrix memory of mLSTM layers (T12MatrixMemory, t12_mixers.h): per head a [dim, vdim] fp32 state under exponential gates with
// a running maximum.  The normaliser n is one more value channel (index vdim) whose value is 1, so the state is
// [vdim + 1][dim_p] columns that never meet.
//
// Three ways through time, all over the same stored state:
//   * one token per row (decode): sixteen lanes own a column, the state streams through once;
//   * a run of tokens, exact: the same columns walked token by token in fp32;
//   * a run of tokens by chunks of 64 on the matrix cores: inside a chunk the recurrence is a causal product
//     (q k^T under the decays) v, across chunks a [dim, 16] strip of the state per workgroup is read out with q and
//     advanced with k^T (w v).  q, k and v are bf16 there; everything in 32 bits -- state, decay-weighted scores, weighted values --
//     enters a product as three bf16 limbs (24 bits), and is accumulated in fp32.

#include <mutex>

#include "t12_act.h"
#include "t12_device.h"
#include "t12_host.h"

namespace {

constexpr int CH = 64;                     // tokens per chunk

struct MemoryParams {
    T12MatrixMemory m;
    const float* in;
    const float* bias;
    int ld;
    const T12Row* rows;
    int n, nch;
    float4* gate;                          // [heads][nch * CH]; by chunks: F (log decay from the chunk's start), i, m, e^-m
                                           // exact: decay, entry weight, e^-m
    float* start;                          // [heads][nch + 1]: m at the chunks' starts
    uint16_t *qb, *kt, *vt, *aw;           // chunk form: q [64][DC] (value_slot order), k^T [DC][64], v^T [VP][64], scores [3][64][64]
    int dc, vp;
    float* o;                              // [n][heads][vdim + 1]
    void* out;
    int out_ld;
};

__device__ __forceinline__ float log_sigmoid(float z) { return fminf(z, 0.0f) - log1pf(expf(-fabsf(z))); }

__device__ __forceinline__ float input_gate(const MemoryParams& p, const float* x, int head)
{
    return p.m.gate_cap * tanhf((x[p.m.i_off + head] + p.bias[p.m.i_off + head]) / p.m.gate_cap);
}
__device__ __forceinline__ float forget_gate(const MemoryParams& p, const float* x, int head)
{
    return log_sigmoid(p.m.gate_cap * tanhf((x[p.m.f_off + head] + p.bias[p.m.f_off + head]) / p.m.gate_cap));
}

__device__ __forceinline__ const float* state_in(const T12MatrixMemory& m, T12Row r)
{
    return m.state + (size_t)(r.slot >> 1) * 2 * m.state_elems + (size_t)(r.slot & 1) * m.state_elems;
}
__device__ __forceinline__ float* state_out(const T12MatrixMemory& m, T12Row r)
{
    return m.state + (size_t)(r.slot >> 1) * 2 * m.state_elems + (size_t)((r.slot & 1) ^ 1) * m.state_elems;
}
__device__ __forceinline__ size_t maximum_at(const T12MatrixMemory& m, int head) { return (size_t)m.heads * (m.vdim + 1) * m.dim_p + head; }

// Sum over the sixteen lanes of a DPP row, in every lane of it.
__device__ __forceinline__ float row_sum16(float v)
{
#define T12_ROW_ADD(ctrl)                                                                      \
    v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), \
                                                               (ctrl), 0xF, 0xF, true))
    T12_ROW_ADD(0xB1);         // quad_perm [1,0,3,2]
    T12_ROW_ADD(0x4E);         // quad_perm [2,3,0,1]
    T12_ROW_ADD(0x141);        // row_half_mirror
    T12_ROW_ADD(0x140);        // row_mirror
#undef T12_ROW_ADD
    return v;
}

// ---- the gates of a run: one workgroup per head, a wave per 64 tokens.  (F, M) = (sum of f, largest i + the f behind it) of a
// stretch compose, so m of every token comes from a scan over a wave's lanes and one over the waves.  Tokens past the end: f = 0,
// i = -1e30.
constexpr int GATE_WAVES = 8;
template <bool CHUNKED>
__global__ __launch_bounds__(GATE_WAVES * 64) void memory_gates_kernel(const MemoryParams p)
{
    __shared__ float2 total[GATE_WAVES];
    const int head = blockIdx.x, lane = threadIdx.x & 63, wave = threadIdx.x >> 6;
    const T12Row row = p.rows[0];
    float m0 = row.position == 0 ? 0.0f : state_in(p.m, row)[maximum_at(p.m, head)];
    float4* gate = p.gate + (size_t)head * p.nch * CH;
    for (int c0 = 0; c0 < p.nch; c0 += GATE_WAVES) {
        const int c = c0 + wave, t = c * CH + lane;
        const float* x = p.in + (size_t)min(t, p.n - 1) * p.ld;
        const bool live = t < p.n;
        const float i = live ? input_gate(p, x, head) : -1e30f, f = live ? forget_gate(p, x, head) : 0.0f;
        float F = f, M = i;
#pragma unroll
        for (int off = 1; off < 64; off <<= 1) {
            const float F1 = __shfl_up(F, off, 64), M1 = __shfl_up(M, off, 64);
            if (lane >= off) {
                M = fmaxf(M1 + F, M);
                F += F1;
            }
        }
        if (lane == 63) total[wave] = make_float2(F, M);
        __syncthreads();
        float mine = m0, next = m0;                        // m ahead of this wave's tokens, and behind all waves'
#pragma unroll
        for (int w = 0; w < GATE_WAVES; w++) {
            if (w == wave) mine = next;
            next = fmaxf(next + total[w].x, total[w].y);
        }
        const float m = fmaxf(F + mine, M);
        float before = __shfl_up(m, 1, 64);
        if (lane == 0) before = mine;
        if (c < p.nch) {
            if (CHUNKED) {
                gate[t] = make_float4(F, i, m, expf(-m));
                if (lane == 0) p.start[head * (p.nch + 1) + c] = mine;
            } else {
                gate[t] = make_float4(expf(f + before - m), expf(i - m), expf(-m), 0.0f);
            }
        }
        m0 = next;
        __syncthreads();                                   // (total is written again)
    }
    if (threadIdx.x == 0) state_out(p.m, row)[maximum_at(p.m, head)] = m0;
}

// ---- exact: one wave = four columns of a head, lane l of a DPP row the key channels RL l .. RL l + RL - 1.
template <int RL>
__global__ __launch_bounds__(64) void memory_exact_kernel(const MemoryParams p)
{
    constexpr int DP = RL * 16, V4 = RL / 4;
    const T12MatrixMemory& m = p.m;
    const int head = blockIdx.x, lane = threadIdx.x, l = lane & 15, j = blockIdx.y * 4 + (lane >> 4);
    const bool live = j <= m.vdim, ones = j >= m.vdim;
    const T12Row row = p.rows[0];
    const size_t cell = ((size_t)head * (m.vdim + 1) + min(j, m.vdim)) * DP + l * RL;
    const float* s = state_in(m, row) + cell;
    t12_f32x4 S[V4];
#pragma unroll
    for (int q = 0; q < V4; q++) S[q] = row.position == 0 ? (t12_f32x4)(0.0f) : *(const t12_f32x4*)(s + q * 4);
    const int qc = m.q_off + head * m.dim, kc = m.k_off + head * m.dim, vc = m.v_off + head * m.vdim + min(j, m.vdim - 1);
    const float4* gate = p.gate + (size_t)head * p.nch * CH;
    for (int t = 0; t < p.n; t++) {
        const float* x = p.in + (size_t)t * p.ld;
        const float4 g = gate[t];
        const float v = (ones ? 1.0f : x[vc] + p.bias[vc]) * g.y;
        float y = 0.0f;
#pragma unroll
        for (int q = 0; q < V4; q++)
#pragma unroll
            for (int e = 0; e < 4; e++) {
                const int d = l * RL + q * 4 + e, dd = min(d, m.dim - 1);
                const float kk = d < m.dim ? x[kc + dd] + p.bias[kc + dd] : 0.0f, qq = d < m.dim ? x[qc + dd] + p.bias[qc + dd] : 0.0f;
                S[q][e] = g.x * S[q][e] + kk * v;
                y += qq * S[q][e];
            }
        y = row_sum16(y);
        if (l == 0 && live) p.o[((size_t)t * m.heads + head) * (m.vdim + 1) + j] = y * m.q_scale;
    }
    if (!live) return;
    float* out = state_out(m, row) + cell;
#pragma unroll
    for (int q = 0; q < V4; q++) *(t12_f32x4*)(out + q * 4) = S[q];
}

// ---- one token per row: workgroup = 256 threads = 16 NP columns of one head of one row.
template <int RL, int NP>
__global__ __launch_bounds__(256) void memory_token_kernel(const MemoryParams p)
{
    constexpr int DP = RL * 16, V4 = RL / 4;
    __shared__ float4 lds4[2 * DP / 4];
    float *q = (float*)lds4, *k = q + DP;
    const T12MatrixMemory& m = p.m;
    const int r = blockIdx.x, head = blockIdx.y, tid = threadIdx.x, l = tid & 15, j0 = blockIdx.z * 16 * NP + (tid >> 4);
    const T12Row row = p.rows[r];
    const float* x = p.in + (size_t)r * p.ld;
    const size_t cell = (size_t)head * (m.vdim + 1) * DP + l * RL;
    const float* s = state_in(m, row) + cell;
    float* out = state_out(m, row) + cell;
    t12_f32x4 S[NP][V4];
#pragma unroll
    for (int c = 0; c < NP; c++)
#pragma unroll
        for (int e = 0; e < V4; e++) S[c][e] = *(const t12_f32x4*)(s + (size_t)min(j0 + c * 16, m.vdim) * DP + e * 4);
    float v[NP];
#pragma unroll
    for (int c = 0; c < NP; c++) {
        const int j = min(j0 + c * 16, m.vdim), vc = m.v_off + head * m.vdim + min(j, m.vdim - 1);
        v[c] = j == m.vdim ? 1.0f : x[vc] + p.bias[vc];
    }
    for (int d = tid; d < DP; d += 256) {
        const int qc = m.q_off + head * m.dim + min(d, m.dim - 1), kc = m.k_off + head * m.dim + min(d, m.dim - 1);
        q[d] = d < m.dim ? (x[qc] + p.bias[qc]) * m.q_scale : 0.0f;
        k[d] = d < m.dim ? x[kc] + p.bias[kc] : 0.0f;
    }
    const float m0 = row.position == 0 ? 0.0f : state_in(m, row)[maximum_at(m, head)];
    const float i = input_gate(p, x, head), f = forget_gate(p, x, head), m1 = fmaxf(f + m0, i);
    const float keep = row.position == 0 ? 0.0f : expf(f + m0 - m1), enter = expf(i - m1);
    if (blockIdx.z == 0 && tid == 0) {
        state_out(m, row)[maximum_at(m, head)] = m1;
        p.gate[(size_t)r * m.heads + head] = make_float4(keep, enter, expf(-m1), 0.0f);
    }
    __syncthreads();
    t12_f32x4 Q[V4], K[V4];
#pragma unroll
    for (int e = 0; e < V4; e++) {
        Q[e] = *(const t12_f32x4*)(q + l * RL + e * 4);
        K[e] = *(const t12_f32x4*)(k + l * RL + e * 4) * enter;
    }
#pragma unroll
    for (int c = 0; c < NP; c++) {
        const int j = j0 + c * 16;
        if (j > m.vdim) continue;                          // uniform over the sixteen lanes
        float y = 0.0f;
#pragma unroll
        for (int e = 0; e < V4; e++) {
            t12_f32x4 w;
#pragma unroll
            for (int b = 0; b < 4; b++) {
                // (position 0: whatever the region holds is left out, also what is no number)
                w[b] = (row.position == 0 ? 0.0f : keep * S[c][e][b]) + K[e][b] * v[c];
                y += Q[e][b] * w[b];
            }
            *(t12_f32x4*)(out + (size_t)j * DP + e * 4) = w;
        }
        y = row_sum16(y);
        if (l == 0) p.o[((size_t)r * m.heads + head) * (m.vdim + 1) + j] = y;
    }
}

// ---- by chunks ----------------------------------------------------------------------------------------------------
// Place of a channel inside a block of 32: lane group g of the matrix cores takes channels 4 g .. 4 g + 3 of both halves, which
// is how an accumulator tile of the state holds them.
__device__ __forceinline__ int channel_slot(int d) { return (d & ~31) + ((d & 15) >> 2) * 8 + ((d >> 4) & 1) * 4 + (d & 3); }

__device__ __forceinline__ uint32_t pack_bf16(float lo, float hi)
{
    typedef __attribute__((ext_vector_type(2))) float f2;
    return __builtin_bit_cast(uint32_t, __builtin_convertvector((f2){lo, hi}, t12_bf16x2));
}
// Eight floats as three bf16 limbs each (24 significant bits).
__device__ __forceinline__ void limbs8(const float (&v)[8], t12_bf16x8 (&l)[3])
{
    float r[8];
#pragma unroll
    for (int e = 0; e < 8; e++) r[e] = v[e];
#pragma unroll
    for (int k = 0; k < 3; k++) {
        uint32_t w[4];
#pragma unroll
        for (int e = 0; e < 4; e++) {
            w[e] = pack_bf16(r[2 * e], r[2 * e + 1]);
            r[2 * e] -= __builtin_bit_cast(float, w[e] << 16);
            r[2 * e + 1] -= __builtin_bit_cast(float, w[e] & 0xFFFF0000u);
        }
        l[k] = __builtin_bit_cast(t12_bf16x8, make_uint4(w[0], w[1], w[2], w[3]));
    }
}

// Four consecutive projections with their bias, of which `left` exist (the others zero).
__device__ __forceinline__ t12_f32x4 projected4(const MemoryParams& p, const float* x, int at, int left)
{
    if (left >= 4 && ((uintptr_t)(x + at) | (uintptr_t)(p.bias + at)) % 16 == 0) return *(const t12_f32x4*)(x + at) + *(const t12_f32x4*)(p.bias + at);
    t12_f32x4 v;
#pragma unroll
    for (int e = 0; e < 4; e++) v[e] = e < left ? x[at + e] + p.bias[at + e] : 0.0f;
    return v;
}

// Operands of a chunk.  blockIdx.z == 0: q, k^T and the decay-weighted scores; z > 0: 64 value channels of v^T.
// Dynamic LDS: q and k [64][dc + 8] bf16.
__global__ __launch_bounds__(256) void memory_prep_kernel(const MemoryParams p)
{
    extern __shared__ uint4 lds4[];
    const T12MatrixMemory& m = p.m;
    const int c = blockIdx.x, head = blockIdx.y, tid = threadIdx.x;
    const size_t unit = (size_t)head * p.nch + c;
    const int nt = min(CH, p.n - c * CH);
    const float* x0 = p.in + (size_t)c * CH * p.ld;
    if (blockIdx.z > 0) {
        uint16_t* tile = (uint16_t*)lds4;                  // [64 tokens][66]
        const int j0 = (blockIdx.z - 1) * 64;
#pragma unroll
        for (int i = 0; i < 4; i++) {                      // (token, four channels)
            const int t = (tid >> 4) + i * 16, j = j0 + (tid & 15) * 4;
            t12_f32x4 v = (t12_f32x4)(0.0f);
            if (t < nt) {
                v = projected4(p, x0 + (size_t)t * p.ld, m.v_off + head * m.vdim + j, m.vdim - j);
#pragma unroll
                for (int e = 0; e < 4; e++)
                    if (j + e == m.vdim) v[e] = 1.0f;
            }
            *(uint32_t*)(tile + t * 66 + (tid & 15) * 4) = pack_bf16(v[0], v[1]);
            *(uint32_t*)(tile + t * 66 + (tid & 15) * 4 + 2) = pack_bf16(v[2], v[3]);
        }
        __syncthreads();
        for (int i = tid; i < 64 * 8; i += 256) {          // (channel, eight tokens)
            const int jj = i >> 3, t8 = (i & 7) * 8;
            if (j0 + jj >= p.vp) continue;
            uint32_t w[4];
#pragma unroll
            for (int e = 0; e < 4; e++) w[e] = tile[(t8 + 2 * e) * 66 + jj] | ((uint32_t)tile[(t8 + 2 * e + 1) * 66 + jj] << 16);
            *(uint4*)(p.vt + (unit * p.vp + j0 + jj) * CH + t8) = make_uint4(w[0], w[1], w[2], w[3]);
        }
        return;
    }
    const int DC = p.dc, pitch = DC + 8;
    uint16_t *qs = (uint16_t*)lds4, *ks = qs + CH * pitch;
#pragma unroll 4
    for (int i = tid; i < CH * DC / 4; i += 256) {
        const int t = i / (DC / 4), d = i % (DC / 4) * 4;
        t12_f32x4 q = (t12_f32x4)(0.0f), k = q;
        if (t < nt) {
            q = projected4(p, x0 + (size_t)t * p.ld, m.q_off + head * m.dim + d, m.dim - d);
            k = projected4(p, x0 + (size_t)t * p.ld, m.k_off + head * m.dim + d, m.dim - d);
        }
        const uint2 qw = make_uint2(pack_bf16(q[0], q[1]), pack_bf16(q[2], q[3]));
        *(uint2*)(qs + t * pitch + d) = qw;
        *(uint2*)(ks + t * pitch + d) = make_uint2(pack_bf16(k[0], k[1]), pack_bf16(k[2], k[3]));
        *(uint2*)(p.qb + (unit * CH + t) * DC + channel_slot(d)) = qw;
    }
    __syncthreads();
    for (int i = tid; i < DC * 8; i += 256) {              // (channel, eight tokens)
        const int d = i % DC, t8 = i / DC * 8;
        uint32_t w[4];
#pragma unroll
        for (int e = 0; e < 4; e++) w[e] = ks[(t8 + 2 * e) * pitch + d] | ((uint32_t)ks[(t8 + 2 * e + 1) * pitch + d] << 16);
        *(uint4*)(p.kt + (unit * DC + d) * CH + t8) = make_uint4(w[0], w[1], w[2], w[3]);
    }
    // scores: a wave takes sixteen queries
    const int lane = tid & 63, wave = tid >> 6, n = lane & 15, g4 = lane >> 4;
    const float4* gate = p.gate + ((size_t)head * p.nch + c) * CH;
    float4 gq[4], gk[4];
#pragma unroll
    for (int i = 0; i < 4; i++) {
        gq[i] = gate[wave * 16 + 4 * g4 + i];
        gk[i] = gate[i * 16 + n];
    }
    t12_f32x4 acc[4];
#pragma unroll
    for (int s = 0; s < 4; s++) acc[s] = (t12_f32x4)(0.0f);
    for (int d = 0; d < DC; d += 32) {
        const t12_bf16x8 a = *(const t12_bf16x8*)(qs + (wave * 16 + n) * pitch + d + 8 * g4);
#pragma unroll
        for (int s = 0; s < 4; s++) {
            const t12_bf16x8 b = *(const t12_bf16x8*)(ks + (s * 16 + n) * pitch + d + 8 * g4);
            acc[s] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a, b, acc[s], 0, 0, 0);
        }
    }
    uint16_t* aw = p.aw + unit * 3 * CH * CH;
#pragma unroll
    for (int s = 0; s < 4; s++)
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = wave * 16 + 4 * g4 + i, u = s * 16 + n;
            const float w = expf(gq[i].x - gk[s].x + gk[s].y - gq[i].z);
            float v = u <= t ? acc[s][i] * m.q_scale * w : 0.0f;
#pragma unroll
            for (int k = 0; k < 3; k++) {
                const uint16_t b = t12_f32_to_bf16(v);
                aw[(k * CH + t) * CH + u] = b;
                v -= t12_bf16_to_f32(b);
            }
        }
}

// The chunks one after the other for sixteen value channels of a head.  Wave w holds key channels 32 NS w .. 32 NS (w + 1) - 1 of
// the strip in its accumulators; what q reads out of the four parts is added up through LDS.
template <int NS>
__global__ __launch_bounds__(256) void memory_scan_kernel(const MemoryParams p)
{
    __shared__ t12_f32x4 red[2][4][4][64];
    __shared__ float wtab[2][CH], etab[2][CH];
    const T12MatrixMemory& m = p.m;
    constexpr int DC = NS * 128;
    const int head = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int n = lane & 15, g4 = lane >> 4, j = blockIdx.y * 16 + n;
    const bool live = j <= m.vdim;
    const T12Row row = p.rows[0];
    const size_t column = ((size_t)head * (m.vdim + 1) + min(j, m.vdim)) * m.dim_p;
    t12_f32x4 S[NS][2];
#pragma unroll
    for (int s = 0; s < NS; s++)
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const int d = (wave * NS + s) * 32 + 16 * u + 4 * g4;
            S[s][u] = (t12_f32x4)(0.0f);
            if (row.position != 0 && live && d < m.dim_p) S[s][u] = *(const t12_f32x4*)(state_in(m, row) + column + d);
        }
    struct Frags {
        t12_bf16x8 q[4][NS], k[NS][2][2], v[2], a[2][3];
        float4 gate, end;
        float start;
    };
    auto load = [&](Frags& f, int c) {
        const size_t unit = (size_t)head * p.nch + c;
        const float4* gate = p.gate + unit * CH;
        f.gate = gate[lane];
        f.end = gate[CH - 1];
        f.start = p.start[head * (p.nch + 1) + c];
#pragma unroll
        for (int s = 0; s < NS; s++) {
#pragma unroll
            for (int t = 0; t < 4; t++)
                f.q[t][s] = *(const t12_bf16x8*)(p.qb + (unit * CH + t * 16 + n) * DC + (wave * NS + s) * 32 + 8 * g4);
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int z = 0; z < 2; z++)
                    f.k[s][u][z] = *(const t12_bf16x8*)(p.kt + (unit * DC + (wave * NS + s) * 32 + 16 * u + n) * CH + z * 32 + 8 * g4);
        }
#pragma unroll
        for (int z = 0; z < 2; z++) {
            f.v[z] = *(const t12_bf16x8*)(p.vt + (unit * p.vp + j) * CH + z * 32 + 8 * g4);
#pragma unroll
            for (int k = 0; k < 3; k++)
                f.a[z][k] = *(const t12_bf16x8*)(p.aw + ((unit * 3 + k) * CH + wave * 16 + n) * CH + z * 32 + 8 * g4);
        }
    };
    // a chunk on f; the next one's operands are on their way meanwhile
    auto chunk = [&](const Frags& f, Frags& next, int c) {
        load(next, min(c + 1, p.nch - 1));
        const int buf = c & 1;
        if (wave == 0) {
            wtab[buf][lane] = expf(f.end.x - f.gate.x + f.gate.y - f.end.z);
            etab[buf][lane] = expf(f.gate.x + f.start - f.gate.z) * m.q_scale;
        }
        const float keep = expf(f.end.x + f.start - f.end.z);
        // what the queries read out of this wave's part of the old state
        t12_f32x4 acc[4];
#pragma unroll
        for (int t = 0; t < 4; t++) acc[t] = (t12_f32x4)(0.0f);
#pragma unroll
        for (int s = 0; s < NS; s++) {
            float v[8];
#pragma unroll
            for (int e = 0; e < 8; e++) v[e] = S[s][e >> 2][e & 3];
            t12_bf16x8 l[3];
            limbs8(v, l);
#pragma unroll
            for (int k = 2; k >= 0; k--)
#pragma unroll
                for (int t = 0; t < 4; t++) acc[t] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.q[t][s], l[k], acc[t], 0, 0, 0);
        }
#pragma unroll
        for (int t = 0; t < 4; t++) red[buf][wave][t][lane] = acc[t];
        // this chunk's own tokens, sixteen queries per wave
        t12_f32x4 own = (t12_f32x4)(0.0f);
#pragma unroll
        for (int z = 0; z < 2; z++)
#pragma unroll
            for (int k = 2; k >= 0; k--) own = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.a[z][k], f.v[z], own, 0, 0, 0);
        __syncthreads();                                   // (the other buffer was last read before the previous barrier)
        t12_f32x4 sum = red[buf][0][wave][lane];
#pragma unroll
        for (int w = 1; w < 4; w++) sum += red[buf][w][wave][lane];
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = wave * 16 + 4 * g4 + i;
            if (live && c * CH + t < p.n)
                p.o[((size_t)(c * CH + t) * m.heads + head) * (m.vdim + 1) + j] = sum[i] * etab[buf][t] + own[i];
        }
        // the state behind the chunk
#pragma unroll
        for (int s = 0; s < NS; s++)
#pragma unroll
            for (int u = 0; u < 2; u++) S[s][u] *= keep;
#pragma unroll
        for (int z = 0; z < 2; z++) {
            float v[8];
            const uint4 raw = __builtin_bit_cast(uint4, f.v[z]);
            const uint32_t w4[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
            for (int e = 0; e < 8; e++)
                v[e] = __builtin_bit_cast(float, e & 1 ? w4[e >> 1] & 0xFFFF0000u : w4[e >> 1] << 16) * wtab[buf][z * 32 + 8 * g4 + e];
            t12_bf16x8 l[3];
            limbs8(v, l);
#pragma unroll
            for (int k = 2; k >= 0; k--)
#pragma unroll
                for (int s = 0; s < NS; s++)
#pragma unroll
                    for (int u = 0; u < 2; u++) S[s][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.k[s][u][z], l[k], S[s][u], 0, 0, 0);
        }
    };
    Frags even, odd;
    load(even, 0);
    for (int c = 0; c < p.nch; c += 2) {
        chunk(even, odd, c);
        if (c + 1 < p.nch) chunk(odd, even, c + 1);
    }
    if (!live) return;
#pragma unroll
    for (int s = 0; s < NS; s++)
#pragma unroll
        for (int u = 0; u < 2; u++) {
            const int d = (wave * NS + s) * 32 + 16 * u + 4 * g4;
            if (d < m.dim_p) *(t12_f32x4*)(state_out(m, row) + column + d) = S[s][u];
        }
}

// ---- normaliser, RMS over the head, plain weight, sigmoid gate: WAVES waves per (row, head), their values in registers.  run:
// floors lie by head.
template <bool F32, int WAVES>
__global__ __launch_bounds__(256) void memory_out_kernel(const MemoryParams p, int run, int chunked)
{
    constexpr int KEEP = 8, LANES = WAVES * 64;
    __shared__ float red[4];
    const T12MatrixMemory& m = p.m;
    const int item = blockIdx.x * (4 / WAVES) + (threadIdx.x >> 6) / WAVES, i0 = threadIdx.x % LANES;
    const bool live = item < p.n * m.heads;
    const int r = min(item, p.n * m.heads - 1) / m.heads, head = min(item, p.n * m.heads - 1) % m.heads, V = m.vdim;
    const float4 g = run ? p.gate[(size_t)head * p.nch * CH + r] : p.gate[(size_t)r * m.heads + head];
    const float* o = p.o + ((size_t)r * m.heads + head) * (V + 1);
    const float* gates = p.in + (size_t)r * p.ld + m.g_off + head * V;
    float v[KEEP], z[KEEP];
#pragma unroll
    for (int q = 0; q < KEEP; q++) {
        const int i = min(i0 + q * LANES, V - 1);
        v[q] = o[i];
        z[q] = gates[i] + p.bias[m.g_off + head * V + i];
    }
    const float inv = 1.0f / (fmaxf(fabsf(o[V]), chunked ? g.w : g.z) + m.den_eps);
    float ss = 0.0f;
#pragma unroll
    for (int q = 0; q < KEEP; q++) {
        v[q] *= inv;
        ss += i0 + q * LANES < V ? v[q] * v[q] : 0.0f;
    }
    for (int i = i0 + KEEP * LANES; i < V; i += LANES) ss += o[i] * inv * (o[i] * inv);
    ss = t12_wave_sum(ss);
    if (WAVES > 1) {
        if ((threadIdx.x & 63) == 0) red[threadIdx.x >> 6] = ss;
        __syncthreads();
        ss = 0.0f;
#pragma unroll
        for (int w = 0; w < WAVES; w++) ss += red[(threadIdx.x >> 6) / WAVES * WAVES + w];
    }
    const float rn = 1.0f / sqrtf(ss / (float)V + m.out_eps);
    auto put = [&](int i, float x, float gate) {
        const int hc = head * V + i;
        x *= rn * m.norm_w[hc] * t12_sigmoid(gate);
        if (F32) ((float*)p.out)[(size_t)r * p.out_ld + hc] = x;
        else ((uint16_t*)p.out)[(size_t)r * p.out_ld + hc] = t12_f32_to_bf16(x);
    };
    if (!live) return;
#pragma unroll
    for (int q = 0; q < KEEP; q++)
        if (i0 + q * LANES < V) put(i0 + q * LANES, v[q], z[q]);
    for (int i = i0 + KEEP * LANES; i < V; i += LANES) put(i, o[i] * inv, gates[i] + p.bias[m.g_off + head * V + i]);
}

template <bool F32>
void launch_out(const MemoryParams& p, int run, int chunked, hipStream_t st)
{
    const int items = p.n * p.m.heads;
    if (items >= 2048 || p.m.vdim <= 128)
        hipLaunchKernelGGL((memory_out_kernel<F32, 1>), dim3((items + 3) / 4), dim3(256), 0, st, p, run, chunked);
    else
        hipLaunchKernelGGL((memory_out_kernel<F32, 4>), dim3(items), dim3(256), 0, st, p, run, chunked);
}

int chunk_channels(int dim) { return dim <= 128 ? 128 : dim <= 256 ? 256 : 512; }

template <int RL>
void launch_token(const MemoryParams& p, hipStream_t st)
{
    const int cols = p.m.vdim + 1;
    // few rows: as many workgroups as there are columns to give out; many: four columns per thread in flight
    if ((size_t)p.n * p.m.heads * ((cols + 63) / 64) >= 512 && RL <= 16)
        hipLaunchKernelGGL((memory_token_kernel<RL, RL <= 16 ? 4 : 1>), dim3(p.n, p.m.heads, (cols + 63) / 64), dim3(256), 0, st, p);
    else
        hipLaunchKernelGGL((memory_token_kernel<RL, 1>), dim3(p.n, p.m.heads, (cols + 15) / 16), dim3(256), 0, st, p);
}

}  // namespace

extern "C" {

int t12_memory_plan(T12MatrixMemory* m, int rows)
{
    T12_REQUIRE(m && m->heads >= 1 && m->dim >= 1 && m->dim <= 512 && m->vdim >= 1 && m->vdim <= 65536 && rows >= 1,
                "t12_memory_plan: heads %d, dim %d (1..512), vdim %d or %d rows out of range", m ? m->heads : 0, m ? m->dim : 0,
                m ? m->vdim : 0, rows);
    m->dim_p = 64;
    while (m->dim_p < m->dim) m->dim_p *= 2;
    m->state_elems = (size_t)m->heads * (m->vdim + 1) * m->dim_p + (m->heads + 3) / 4 * 4;
    const size_t nch = (rows + CH - 1) / CH, H = m->heads, dc = chunk_channels(m->dim), vp = (m->vdim + 16) / 16 * 16;
    m->work_floats = H * nch * CH * 4 + (H * (nch + 1) + 3) / 4 * 4 + H * nch * (CH * dc + CH * vp / 2 + 3 * CH * CH / 2) +
                     (size_t)rows * H * (m->vdim + 1);
    return T12_OK;
}

int t12_matrix_memory(const T12MatrixMemory* m, const float* in, const float* bias, int ld, const T12Row* rows, int n, int run, int exact,
                      float* work, void* out, int out_f32, int out_ld, void* stream)
{
    T12_REQUIRE(m && in && bias && rows && work && out && m->state && m->norm_w && n >= 1, "t12_matrix_memory: null operand or no rows");
    T12_REQUIRE(m->dim_p >= m->dim && m->dim_p >= 64 && m->state_elems == (size_t)m->heads * (m->vdim + 1) * m->dim_p + (m->heads + 3) / 4 * 4,
                "t12_matrix_memory: t12_memory_plan has not been called");
    const int HD = m->heads * m->dim, HV = m->heads * m->vdim;
    T12_REQUIRE(m->q_off >= 0 && m->q_off + HD <= ld && m->k_off >= 0 && m->k_off + HD <= ld && m->v_off >= 0 && m->v_off + HV <= ld &&
                    m->g_off >= 0 && m->g_off + HV <= ld && m->i_off >= 0 && m->i_off + m->heads <= ld && m->f_off >= 0 &&
                    m->f_off + m->heads <= ld && out_ld >= HV,
                "t12_matrix_memory: a projection lies outside a row of %d, or output rows of %d are too short", ld, out_ld);
    T12_REQUIRE((uintptr_t)work % 16 == 0 && (uintptr_t)m->state % 16 == 0 && m->gate_cap > 0.0f,
                "t12_matrix_memory: workspace or state not aligned, or a cap that is not positive");
    hipStream_t st = (hipStream_t)stream;
    const size_t H = m->heads;
    MemoryParams p = {};
    p.m = *m;
    p.in = in;
    p.bias = bias;
    p.ld = ld;
    p.rows = rows;
    p.n = n;
    p.nch = (n + CH - 1) / CH;
    p.dc = chunk_channels(m->dim);
    p.vp = (m->vdim + 16) / 16 * 16;
    float* w = work;
    auto take = [&](size_t floats) {
        float* q = w;
        w += floats;
        return q;
    };
    p.gate = (float4*)take(H * p.nch * CH * 4);
    p.start = take((H * (p.nch + 1) + 3) / 4 * 4);
    p.qb = (uint16_t*)take(H * p.nch * CH * p.dc / 2);
    p.kt = (uint16_t*)take(H * p.nch * CH * p.dc / 2);
    p.vt = (uint16_t*)take(H * p.nch * CH * p.vp / 2);
    p.aw = (uint16_t*)take(H * p.nch * 3 * CH * CH / 2);
    p.o = w;
    p.out = out;
    p.out_ld = out_ld;
    const int cols = m->vdim + 1;
    if (!run) {
        switch (m->dim_p) {
            case 64: launch_token<4>(p, st); break;
            case 128: launch_token<8>(p, st); break;
            case 256: launch_token<16>(p, st); break;
            default: launch_token<32>(p, st); break;
        }
    } else if (exact) {
        hipLaunchKernelGGL(memory_gates_kernel<false>, dim3(m->heads), dim3(GATE_WAVES * 64), 0, st, p);
        const dim3 grid(m->heads, (cols + 3) / 4);
        switch (m->dim_p) {
            case 64: hipLaunchKernelGGL(memory_exact_kernel<4>, grid, dim3(64), 0, st, p); break;
            case 128: hipLaunchKernelGGL(memory_exact_kernel<8>, grid, dim3(64), 0, st, p); break;
            case 256: hipLaunchKernelGGL(memory_exact_kernel<16>, grid, dim3(64), 0, st, p); break;
            default: hipLaunchKernelGGL(memory_exact_kernel<32>, grid, dim3(64), 0, st, p); break;
        }
    } else {
        hipLaunchKernelGGL(memory_gates_kernel<true>, dim3(m->heads), dim3(GATE_WAVES * 64), 0, st, p);
        const size_t lds = (size_t)2 * CH * (p.dc + 8) * 2;
        if (lds > 64 * 1024) {
            static std::once_flag once[16];                // the attribute is per device
            int dev = 0;
            if (hipGetDevice(&dev) != hipSuccess || dev < 0 || dev >= 16) dev = 0;
            hipError_t e = hipSuccess;
            std::call_once(once[dev], [&] {
                e = hipFuncSetAttribute((const void*)memory_prep_kernel, hipFuncAttributeMaxDynamicSharedMemorySize, 2 * CH * (512 + 8) * 2);
            });
            if (e != hipSuccess) {
                t12_set_error("t12_matrix_memory: cannot reserve %zu bytes of LDS", lds);
                return T12_ELAUNCH;
            }
        }
        hipLaunchKernelGGL(memory_prep_kernel, dim3(p.nch, m->heads, 1 + (p.vp + 63) / 64), dim3(256), lds, st, p);
        // (the head is the fast axis: workgroups go to the chip's XCDs in turn, so an XCD's L2 holds few heads' operands)
        const dim3 grid(m->heads, p.vp / 16);
        switch (p.dc) {
            case 128: hipLaunchKernelGGL(memory_scan_kernel<1>, grid, dim3(256), 0, st, p); break;
            case 256: hipLaunchKernelGGL(memory_scan_kernel<2>, grid, dim3(256), 0, st, p); break;
            default: hipLaunchKernelGGL(memory_scan_kernel<4>, grid, dim3(256), 0, st, p); break;
        }
    }
    T12_CHECK_LAUNCH("t12_matrix_memory");
    if (out_f32) launch_out<true>(p, run, run && !exact, st);
    else launch_out<false>(p, run, run && !exact, st);
    T12_CHECK_LAUNCH("t12_matrix_memory(out)");
    return T12_OK;
}

}  // extern "C"
