// Matrix memory of mLSTM layers (T12MatrixMemory, t12_mixers.h): per head a [dim, vdim] fp32 state under exponential gates with
// a running maximum.  The normaliser n is one more value channel (index vdim) whose value is 1, so the state is
// [vdim + 1][dim_p] columns that never meet.
//
// Three ways through time, all over the same stored state:
//   * one token per row (decode): sixteen lanes own a column, the state streams through once;
//   * a run of tokens, exact: the same columns walked token by token in fp32;
//   * a run of tokens by chunks of 64 on the matrix cores: inside a chunk the recurrence is a causal product
//     (q k^T under the decays) v, across chunks a [dim, 32] strip of the state per workgroup is read out with q and
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
    uint16_t *qb, *kt, *vt, *aw;           // chunk form: q, k^T, v^T and scores of every chunk, in fragments (below)
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
// Operands lie as the matrix cores take them: fragments of 64 lanes x eight bf16, lane (n, g) = (lane % 16, lane / 16), so that a wave
// loads a fragment as one contiguous kilobyte.
//   q       [token tile][32-channel step]       lane: token n of the tile, channels 4 g .. 4 g + 3 of both halves of the step -- the
//                                               order in which an accumulator tile of the state holds them
//   k^T     [16-channel tile][32-token half]    lane: channel n, tokens 8 g .. 8 g + 7
//   v^T     [16-channel tile][32-token half]    the same
//   scores  [token tile][32-token half][limb]   lane: query n of the tile, tokens 8 g .. 8 g + 7
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

// Four consecutive projections with their bias, columns at .. at + 3 of which those below `end` exist (the others zero).  No branch:
// the loads of an unrolled loop stay in flight together.
template <bool WIDE>
__device__ __forceinline__ t12_f32x4 projected4(const MemoryParams& p, const float* x, int at, int end)
{
    t12_f32x4 v;
    if (WIDE) {                                            // everything aligned, sizes multiples of four
        const int c = min(at, end - 4);
        v = *(const t12_f32x4*)(x + c) + *(const t12_f32x4*)(p.bias + c);
        return at < end ? v : (t12_f32x4)(0.0f);
    }
#pragma unroll
    for (int e = 0; e < 4; e++) {
        const int c = min(at + e, end - 1);
        v[e] = at + e < end ? x[c] + p.bias[c] : 0.0f;
    }
    return v;
}

// Operands of a chunk.  blockIdx.z == 0: q, k^T and the decay-weighted scores; z > 0: 64 value channels of v^T.
// Dynamic LDS: q and k [64][dc + 8] bf16.
template <bool WIDE>
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
        const int j0 = (blockIdx.z - 1) * 64, from = m.v_off + head * m.vdim, jj = (tid & 15) * 4;
        t12_f32x4 v[4];
#pragma unroll
        for (int i = 0; i < 4; i++)                        // (token, four channels)
            v[i] = projected4<WIDE>(p, x0 + (size_t)min((tid >> 4) + i * 16, nt - 1) * p.ld, from + j0 + jj, from + m.vdim);
#pragma unroll
        for (int i = 0; i < 4; i++) {
            const int t = (tid >> 4) + i * 16;
#pragma unroll
            for (int e = 0; e < 4; e++) v[i][e] = t >= nt ? 0.0f : j0 + jj + e == m.vdim ? 1.0f : v[i][e];
            *(uint32_t*)(tile + t * 66 + jj) = pack_bf16(v[i][0], v[i][1]);
            *(uint32_t*)(tile + t * 66 + jj + 2) = pack_bf16(v[i][2], v[i][3]);
        }
        __syncthreads();
        uint4* out = (uint4*)p.vt + unit * p.vp * CH / 8;
        for (int i = tid; i < 64 * 8; i += 256) {          // (tile, half, lane)
            const int n = i & 15, g = i >> 4 & 3, z = i >> 6 & 1, jt = i >> 7, ch = jt * 16 + n, t8 = z * 32 + g * 8;
            if (j0 + ch >= p.vp) continue;
            uint32_t w[4];
#pragma unroll
            for (int e = 0; e < 4; e++) w[e] = tile[(t8 + 2 * e) * 66 + ch] | ((uint32_t)tile[(t8 + 2 * e + 1) * 66 + ch] << 16);
            out[((j0 / 16 + jt) * 2 + z) * 64 + (i & 63)] = make_uint4(w[0], w[1], w[2], w[3]);
        }
        return;
    }
    const int DC = p.dc, pitch = DC + 8, per_row = DC / 4;
    uint16_t *qs = (uint16_t*)lds4, *ks = qs + CH * pitch;
    const int qf = m.q_off + head * m.dim, kf = m.k_off + head * m.dim;
    constexpr int U = 4;                                   // pieces whose loads are in flight together
    for (int i0 = tid; i0 < CH * per_row; i0 += 256 * U) {
        t12_f32x4 q[U], k[U];
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int i = i0 + u * 256, d = i % per_row * 4;
            const float* x = x0 + (size_t)min(i / per_row, nt - 1) * p.ld;
            q[u] = projected4<WIDE>(p, x, qf + d, qf + m.dim);
            k[u] = projected4<WIDE>(p, x, kf + d, kf + m.dim);
        }
#pragma unroll
        for (int u = 0; u < U; u++) {
            const int i = i0 + u * 256, t = i / per_row, d = i % per_row * 4;
            const bool live = t < nt;
            *(uint2*)(qs + t * pitch + d) = live ? make_uint2(pack_bf16(q[u][0], q[u][1]), pack_bf16(q[u][2], q[u][3])) : make_uint2(0, 0);
            *(uint2*)(ks + t * pitch + d) = live ? make_uint2(pack_bf16(k[u][0], k[u][1]), pack_bf16(k[u][2], k[u][3])) : make_uint2(0, 0);
        }
    }
    __syncthreads();
    {
        uint4* out = (uint4*)p.qb + unit * DC * CH / 8;
        const int steps = DC / 32;
        for (int i = tid; i < steps * 4 * 64; i += 256) {
            const int n = i & 15, g = i >> 4 & 3, f = i >> 6, step = f % steps, tile = f / steps;
            const uint16_t* q = qs + (tile * 16 + n) * pitch + step * 32 + 4 * g;
            const uint2 lo = *(const uint2*)q, hi = *(const uint2*)(q + 16);
            out[i] = make_uint4(lo.x, lo.y, hi.x, hi.y);
        }
        out = (uint4*)p.kt + unit * DC * CH / 8;
        for (int i = tid; i < DC / 16 * 2 * 64; i += 256) {
            const int n = i & 15, g = i >> 4 & 3, z = i >> 6 & 1, d = (i >> 7) * 16 + n, t8 = z * 32 + g * 8;
            uint32_t w[4];
#pragma unroll
            for (int e = 0; e < 4; e++) w[e] = ks[(t8 + 2 * e) * pitch + d] | ((uint32_t)ks[(t8 + 2 * e + 1) * pitch + d] << 16);
            out[i] = make_uint4(w[0], w[1], w[2], w[3]);
        }
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
                aw[((((wave * 2 + (s >> 1)) * 3 + k) * 64 + ((s & 1) * 2 + (n >> 3)) * 16 + 4 * g4 + i) * 8) + (n & 7)] = b;
                v -= t12_bf16_to_f32(b);
            }
        }
}

// The chunks one after the other for 16 NJ value channels of a head.  Wave w holds key channels 32 NS w .. 32 NS (w + 1) - 1 of
// the strip in its accumulators; what q reads out of the four parts is added up through LDS.
template <int NS>
__global__ __launch_bounds__(256) void memory_scan_kernel(const MemoryParams p)
{
    constexpr int DC = NS * 128, NJ = 2;
    __shared__ t12_f32x4 red[4][4][NJ][64];
    __shared__ float wtab[CH], etab[CH];
    const T12MatrixMemory& m = p.m;
    const int head = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    const int n = lane & 15, g4 = lane >> 4, tiles = p.vp / 16;
    const T12Row row = p.rows[0];
    int jt[NJ], j[NJ];                                     // (a strip past the last one works on that one and stores nothing)
    bool live[NJ];
    size_t column[NJ];
    t12_f32x4 S[NJ][NS][2];
#pragma unroll
    for (int c = 0; c < NJ; c++) {
        jt[c] = min((int)blockIdx.y * NJ + c, tiles - 1);
        j[c] = jt[c] * 16 + n;
        live[c] = (int)blockIdx.y * NJ + c < tiles && j[c] <= m.vdim;
        column[c] = ((size_t)head * (m.vdim + 1) + min(j[c], m.vdim)) * m.dim_p;
#pragma unroll
        for (int s = 0; s < NS; s++)
#pragma unroll
            for (int u = 0; u < 2; u++) {
                const int d = (wave * NS + s) * 32 + 16 * u + 4 * g4;
                S[c][s][u] = (t12_f32x4)(0.0f);
                if (row.position != 0 && live[c] && d < m.dim_p) S[c][s][u] = *(const t12_f32x4*)(state_in(m, row) + column[c] + d);
            }
    }
    struct Frags {
        t12_bf16x8 q[4][NS], k[NS][2][2], v[NJ][2], a[2][3];
        float4 gate, end;
        float start;
    };
    auto load = [&](Frags& f, int c) {
        const size_t unit = (size_t)head * p.nch + c;
        const float4* gate = p.gate + unit * CH;
        f.gate = gate[lane];
        f.end = gate[CH - 1];
        f.start = p.start[head * (p.nch + 1) + c];
        const t12_bf16x8* q = (const t12_bf16x8*)p.qb + unit * (DC * CH / 8) + lane;
        const t12_bf16x8* k = (const t12_bf16x8*)p.kt + unit * (DC * CH / 8) + lane;
        const t12_bf16x8* v = (const t12_bf16x8*)p.vt + unit * p.vp * (CH / 8) + lane;
        const t12_bf16x8* a = (const t12_bf16x8*)p.aw + (unit * 4 + wave) * 6 * 64 + lane;
#pragma unroll
        for (int s = 0; s < NS; s++) {
#pragma unroll
            for (int t = 0; t < 4; t++) f.q[t][s] = q[(t * (DC / 32) + wave * NS + s) * 64];
#pragma unroll
            for (int u = 0; u < 2; u++)
#pragma unroll
                for (int z = 0; z < 2; z++) f.k[s][u][z] = k[(((wave * NS + s) * 2 + u) * 2 + z) * 64];
        }
#pragma unroll
        for (int z = 0; z < 2; z++) {
#pragma unroll
            for (int i = 0; i < NJ; i++) f.v[i][z] = v[(jt[i] * 2 + z) * 64];
#pragma unroll
            for (int l = 0; l < 3; l++) f.a[z][l] = a[(z * 3 + l) * 64];
        }
    };
    // a chunk on f; the next one's operands are on their way meanwhile
    auto chunk = [&](const Frags& f, Frags& next, int c) {
        load(next, min(c + 1, p.nch - 1));
        const float keep = expf(f.end.x + f.start - f.end.z);
        // what the queries read out of this wave's part of the old state
        t12_f32x4 acc[4][NJ];
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int i = 0; i < NJ; i++) acc[t][i] = (t12_f32x4)(0.0f);
#pragma unroll
        for (int s = 0; s < NS; s++) {
            t12_bf16x8 l[NJ][3];
#pragma unroll
            for (int i = 0; i < NJ; i++) {
                float v[8];
#pragma unroll
                for (int e = 0; e < 8; e++) v[e] = S[i][s][e >> 2][e & 3];
                limbs8(v, l[i]);
            }
#pragma unroll
            for (int k = 2; k >= 0; k--)
#pragma unroll
                for (int t = 0; t < 4; t++)
#pragma unroll
                    for (int i = 0; i < NJ; i++) acc[t][i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.q[t][s], l[i][k], acc[t][i], 0, 0, 0);
        }
        // this chunk's own tokens, sixteen queries per wave
        t12_f32x4 own[NJ];
#pragma unroll
        for (int i = 0; i < NJ; i++) own[i] = (t12_f32x4)(0.0f);
#pragma unroll
        for (int z = 0; z < 2; z++)
#pragma unroll
            for (int k = 2; k >= 0; k--)
#pragma unroll
                for (int i = 0; i < NJ; i++) own[i] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.a[z][k], f.v[i][z], own[i], 0, 0, 0);
        __syncthreads();                                   // (what the last chunk left in LDS has been read)
        if (wave == 0) {
            wtab[lane] = expf(f.end.x - f.gate.x + f.gate.y - f.end.z);
            etab[lane] = expf(f.gate.x + f.start - f.gate.z) * m.q_scale;
        }
#pragma unroll
        for (int t = 0; t < 4; t++)
#pragma unroll
            for (int i = 0; i < NJ; i++) red[wave][t][i][lane] = acc[t][i];
        __syncthreads();
        const t12_f32x4 e4 = *(const t12_f32x4*)(etab + wave * 16 + 4 * g4);
#pragma unroll
        for (int i = 0; i < NJ; i++) {
            t12_f32x4 sum = red[0][wave][i][lane];
#pragma unroll
            for (int w = 1; w < 4; w++) sum += red[w][wave][i][lane];
            float* o = p.o + ((size_t)(c * CH + wave * 16 + 4 * g4) * m.heads + head) * (m.vdim + 1) + j[i];
#pragma unroll
            for (int r = 0; r < 4; r++)
                if (live[i] && c * CH + wave * 16 + 4 * g4 + r < p.n) o[(size_t)r * m.heads * (m.vdim + 1)] = sum[r] * e4[r] + own[i][r];
        }
        // the state behind the chunk
#pragma unroll
        for (int i = 0; i < NJ; i++)
#pragma unroll
            for (int s = 0; s < NS; s++)
#pragma unroll
                for (int u = 0; u < 2; u++) S[i][s][u] *= keep;
#pragma unroll
        for (int z = 0; z < 2; z++) {
            const t12_f32x4 w0 = *(const t12_f32x4*)(wtab + z * 32 + 8 * g4), w1 = *(const t12_f32x4*)(wtab + z * 32 + 8 * g4 + 4);
            t12_bf16x8 l[NJ][3];
#pragma unroll
            for (int i = 0; i < NJ; i++) {
                const uint4 raw = __builtin_bit_cast(uint4, f.v[i][z]);
                const uint32_t r4[4] = {raw.x, raw.y, raw.z, raw.w};
                float v[8];
#pragma unroll
                for (int e = 0; e < 8; e++)
                    v[e] = __builtin_bit_cast(float, e & 1 ? r4[e >> 1] & 0xFFFF0000u : r4[e >> 1] << 16) * (e < 4 ? w0[e & 3] : w1[e & 3]);
                limbs8(v, l[i]);
            }
#pragma unroll
            for (int k = 2; k >= 0; k--)
#pragma unroll
                for (int s = 0; s < NS; s++)
#pragma unroll
                    for (int u = 0; u < 2; u++)
#pragma unroll
                        for (int i = 0; i < NJ; i++)
                            S[i][s][u] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(f.k[s][u][z], l[i][k], S[i][s][u], 0, 0, 0);
        }
    };
    Frags even, odd;
    load(even, 0);
    for (int c = 0; c < p.nch; c += 2) {
        chunk(even, odd, c);
        if (c + 1 < p.nch) chunk(odd, even, c + 1);
    }
#pragma unroll
    for (int i = 0; i < NJ; i++) {
        if (!live[i]) continue;
#pragma unroll
        for (int s = 0; s < NS; s++)
#pragma unroll
            for (int u = 0; u < 2; u++) {
                const int d = (wave * NS + s) * 32 + 16 * u + 4 * g4;
                if (d < m.dim_p) *(t12_f32x4*)(state_out(m, row) + column[i] + d) = S[i][s][u];
            }
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
                for (const void* k : {(const void*)memory_prep_kernel<true>, (const void*)memory_prep_kernel<false>})
                    if (e == hipSuccess) e = hipFuncSetAttribute(k, hipFuncAttributeMaxDynamicSharedMemorySize, 2 * CH * (512 + 8) * 2);
            });
            if (e != hipSuccess) {
                t12_set_error("t12_matrix_memory: cannot reserve %zu bytes of LDS", lds);
                return T12_ELAUNCH;
            }
        }
        bool wide = ld % 4 == 0 && m->dim % 4 == 0 && m->vdim % 4 == 0 && ((uintptr_t)in | (uintptr_t)bias) % 16 == 0;
        for (int off : {m->q_off, m->k_off, m->v_off}) wide = wide && off % 4 == 0;
        const dim3 prep(p.nch, m->heads, 1 + (p.vp + 63) / 64);
        if (wide) hipLaunchKernelGGL(memory_prep_kernel<true>, prep, dim3(256), lds, st, p);
        else hipLaunchKernelGGL(memory_prep_kernel<false>, prep, dim3(256), lds, st, p);
        // (the head is the fast axis: workgroups go to the chip's XCDs in turn, so an XCD's L2 holds few heads' operands)
        const dim3 grid(m->heads, (p.vp / 16 + 1) / 2);
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
