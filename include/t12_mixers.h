/* C ABI of the sequence mixers and layer pieces that hybrid decoders use (libturbo12.so): windowed attention with
 * sigmoid weights over a ring cache, the generalized delta rule, matrix memory (mLSTM), latent attention, learned
 * positions, norms around sublayers, unary activations, gated linear units, logit capping.
 * No counterpart in the reference, whose one family is Llama.  Device pointers, asynchronous on `stream`, T12_* return
 * codes (t12_abi.h).
 *
 * A launch works on `n` ROWS, one token each.  Row r sits at rows[r].position of its sequence and belongs to cache
 * region rows[r].slot >> 1; the low bit of slot names which of the region's two recurrent states is read (the other one
 * is written, so that the last step can be taken back).  Either every row is a sequence of its own (a decode step), or
 * all rows are consecutive tokens of one sequence (a prompt pass): `run` says which.
 */
#ifndef T12_MIXERS_H
#define T12_MIXERS_H

#include <stddef.h>
#include <stdint.h>

#ifdef __cplusplus
extern "C" {
#endif

typedef struct T12Row {
    int position;
    int slot;
} T12Row;

/* Fills a row table on the device: n consecutive positions of one region, or a host list (it travels as a kernel
 * argument: no copy is enqueued). */
int t12_rows_run(T12Row* rows, int first_position, int slot, int n, void* stream);
int t12_rows_list(T12Row* rows, const T12Row* host_rows, int n, void* stream);

/* out[r, :] = table[tokens[r], :] + pos_table[rows[r].position, :] in fp32, bf16 tables; a token or position outside its
 * table contributes zeros. */
int t12_embed_positions(const void* table_bf16, int n_vocab, const void* pos_bf16, int n_positions, const int* tokens,
                        const T12Row* rows, float* out, int width, int n, void* stream);

/* out[r, :] = e / sqrt(mean(e^2) + eps) * weight in fp32, e = table[tokens[r], :] (bf16 table; a token outside it: zeros). */
int t12_embed_norm(const void* table_bf16, int n_vocab, const int* tokens, const float* weight, float eps, float* out, int width,
                   int n, void* stream);

/* A sublayer's output through its own norm, onto the residual, and the next norm:
 *     x_out[r] = residual[r] + y[r] / sqrt(mean(y[r]^2) + eps) * post_w,   h[r] = x_out[r] / sqrt(mean(x_out[r]^2) + eps) * norm_w
 * y: fp32 [n, width], or, with part, the K-split partial sums t12_gemm_deferred left (their first `width` columns).  x_out
 * fp32 (may be y itself, not residual); h bf16, or fp32 with h_f32. */
struct T12GemmPartials;
int t12_post_norm_add(const float* y, const struct T12GemmPartials* part, const float* residual, const float* post_w,
                      const float* norm_w, float eps, float* x_out, void* h, int h_f32, int width, int n, void* stream);

/* y[r] = x[r] / sqrt(mean(x[r]^2) + eps) * weight, all fp32. */
int t12_rms_norm_f32(const float* x, const float* weight, float* y, int width, float eps, int n, void* stream);

/* ---- unary functions of a projection ---------------------------------------------------------------------------
 * T12_ACT_XIELU: z > 0: a z^2 + z/2;  z <= 0: b (exp(z) - 1 - z) + z/2   (a, b already softplus'ed by the caller)
 * T12_ACT_SOFTCAP: a tanh(z / a) */
enum { T12_ACT_NONE = 0, T12_ACT_XIELU = 1, T12_ACT_SOFTCAP = 2 };
typedef struct T12Act {
    int   kind;
    float a, b;
} T12Act;
/* out[i] = act(x[i]), i < n; out_f32: fp32 (may be x itself), else bf16. */
int t12_act(const float* x, const T12Act* act, void* out, int out_f32, size_t n, void* stream);

/* t12_gemv with the function in its epilogue, one tensor: T12_ACT_XIELU stores bf16 to out_bf16, T12_ACT_SOFTCAP fp32 to
 * seg->out.  act_bf16 given: the activations; NULL: bf16(x / sqrt(mean(x^2) + eps) * norm_w) of the fp32 x, computed in the
 * prologue (K <= 8192).  K % 16 == 0, base_exp in 0..240. */
struct T12Segment;
int t12_gemv_act(const struct T12Segment* seg, const void* act_bf16, const float* x, const float* norm_w, float eps, int K,
                 const T12Act* act, void* out_bf16, void* stream);

/* t12_gemm with the function in its epilogue, one tensor, T12_ACT_XIELU: out_bf16[b*out_stride + m] = bf16(act(W[m,:] . X[b,:])).
 * Returns 1 when the shape has no such kernel (B <= 64, a K split, K not a multiple of 64, base_exp outside 0..240): run
 * t12_gemm and t12_act then -- or t12_gemm_deferred and t12_act_partials, which adds up the partial sums of a K-split
 * launch (*part) while it applies the function: out_bf16 [B, M]. */
int t12_gemm_act(const struct T12Segment* seg, const void* act_bf16, int act_stride, int K, int B, const T12Act* act,
                 void* out_bf16, int out_stride, void* stream);
int t12_act_partials(const struct T12GemmPartials* part, const T12Act* act, void* out_bf16, int M, int B, void* stream);

/* ---- gated linear units ------------------------------------------------------------------------------------------
 *     g' = min(g, limit),  u' = clamp(u, -limit, limit),  out = g' * sigmoid(slope g') * (u' + offset)
 * limit = infinity, slope 1, offset 0: SwiGLU. */
typedef struct T12Glu {
    float limit, slope, offset;
} T12Glu;
/* out[i] = glu(gate[i], up[i]), i < n; out_f32: fp32, else bf16. */
int t12_glu(const float* gate, const float* up, const T12Glu* glu, void* out, int out_f32, size_t n, void* stream);
/* t12_gemm_swiglu and t12_gemv_swiglu (t12_abi.h) with any unit. */
int t12_gemm_glu(const struct T12Segment* gate, const struct T12Segment* up, const T12Glu* glu, const void* act_bf16, int act_stride,
                 int K, int B, void* out_bf16, int out_stride, void* stream);
int t12_gemv_glu(const struct T12Segment* gate, const struct T12Segment* up, const T12Glu* glu, const void* act_bf16, int K,
                 void* out_bf16, void* stream);

/* The decode-GEMV behind a sublayer whose output goes through a norm of its own, norms with one gain for all columns:
 *     s = residual + rmsnorm(x) gain_post  (-> hidden_out when given; it may not alias x or residual),
 *     activations = bf16(rmsnorm(s) gain),
 * x, residual fp32 [K]; K % 16 == 0, K <= 8192, base_exp in 0..240.  t12_gemv_norm (t12_abi.h), and t12_gemv_glu, on these. */
int t12_gemv_gain_norm(const struct T12Segment* segs, int nseg, const float* x, const float* residual, float gain_post, float gain,
                       float eps, float* hidden_out, int K, void* stream);
int t12_gemv_glu_gain_norm(const struct T12Segment* gate, const struct T12Segment* up, const T12Glu* glu, const float* x,
                           const float* residual, float gain_post, float gain, float eps, float* hidden_out, int K, void* out_bf16,
                           void* stream);

/* ---- windowed attention with sigmoid weights -------------------------------------------------------------------
 * Query head h reads key/value head h / (heads / kv_heads).  The query at position i sees the key at j <= i when
 * i - j < window or j < keep_first, with weight sigmoid(scale * q.k + head_bias[h]); weights are not normalised.
 *
 * The cache of a region holds the first keep_first positions for good and the others in a ring of whole 32-position
 * blocks that is large enough for the window of every row of a pass.  Per kv head and block: keys [32][dim_p], then
 * (another array) values [vdim_p][32] with the block's positions in the order 0-3, 16-19, 4-7, 20-23, ... that the
 * matrix cores consume; dim_p, vdim_p = the sizes padded (with zeros) to 64, 128 or 256, the sizes of the matrix-core
 * instances, in a bf16 cache when both fit, else to a multiple of 32. */
typedef struct T12WindowAttn {
    int   heads, kv_heads, dim, vdim;
    int   window, keep_first;
    float scale;
    int   elem_bytes;                   /* cache element: 2 bf16, 4 fp32 */
    /* set by t12_window_plan: */
    int   dim_p, vdim_p, kept_blocks, ring_blocks;
    size_t k_elems, v_elems;            /* cache elements per region */
    /* the cache, regions back to back; zeroed before first use */
    void* k;
    void* v;
    /* where a row's projections lie in the fp32 input: q [heads*dim], k [kv_heads*dim], v [kv_heads*vdim] */
    int   q_off, k_off, v_off;
    const float* head_bias;             /* [heads] */
} T12WindowAttn;
/* Sizes the cache for `max_positions` positions and passes of up to `rows` rows of one sequence. */
int t12_window_plan(T12WindowAttn* a, int max_positions, int rows);
/* Stores k + bias and v + bias of every row in its region (before any row of the pass attends).  in: fp32 [n, ld],
 * bias: fp32 [ld], added to every row. */
int t12_window_store(const T12WindowAttn* a, const float* in, const float* bias, int ld, const T12Row* rows, int n,
                     int run, void* stream);
/* out[r * out_ld + h * vdim + c] = out_scale * (head h's weighted value sum); out bf16, or fp32 with out_f32. */
int t12_window_attention(const T12WindowAttn* a, const float* in, const float* bias, int ld, const T12Row* rows, int n,
                         int run, float out_scale, void* out, int out_f32, int out_ld, void* stream);

/* ---- generalized delta rule --------------------------------------------------------------------------------------
 * Per head, with u = k / sqrt(sum k^2 + unit_eps), removal rate a = sigmoid(a_in), decay
 * w = exp(-decay_rate * sigmoid(W2 tanh(w1_in) + w0)), all per key channel, 32-bit throughout:
 *     S <- diag(w) S - (a u) (u^T S) + k v^T   (both terms read the old S),    o = S^T r
 *     out = out_scale * norm_w * (o / sqrt(mean(o^2) + out_eps)) * sigmoid(g)
 * A row at position 0 starts from S = 0, whatever its region holds. */
typedef struct T12DeltaRule {
    int   heads, dim, rank;
    float unit_eps, decay_rate, out_eps;
    const float* w2t;                   /* [rank, heads*dim]: W2 transposed */
    const float* w0;                    /* [heads*dim] */
    const float* norm_w;                /* [heads*dim] */
    int   r_off, k_off, v_off, a_off, g_off, w1_off;   /* in a row of the fp32 input: [heads*dim] each, w1: [rank] */
    /* set by t12_delta_plan: */
    int   dim_p;                        /* key channels padded (zero) to a multiple of 16 lanes */
    size_t state_elems;                 /* floats per state: [heads][value channel][dim_p] */
    size_t work_elems;                  /* floats of workspace per row */
    float* state;                       /* [region][2][state_elems] */
} T12DeltaRule;
int t12_delta_plan(T12DeltaRule* d);
int t12_delta_rule(const T12DeltaRule* d, const float* in, const float* bias, int ld, const T12Row* rows, int n, int run,
                   float out_scale, float* work, void* out, int out_f32, int out_ld, void* stream);

/* ---- matrix memory (mLSTM) -----------------------------------------------------------------------------------------
 * Per head, with log gates i = cap tanh(i_in / cap), f = log sigmoid(cap tanh(f_in / cap)), running maximum m, 32-bit:
 *     m' = max(f + m, i)     S <- e^(f+m-m') S + e^(i-m') k v^T     n <- e^(f+m-m') n + e^(i-m') k
 *     o = S^T q q_scale / (max(|n . q q_scale|, e^(-m')) + den_eps)
 *     out = norm_w * (o / sqrt(mean(o^2) + out_eps)) * sigmoid(g)
 * n is held as one more value channel whose value is always 1.  A row at position 0 starts from S = n = 0, m = 0. */
typedef struct T12MatrixMemory {
    int   heads, dim, vdim;
    float q_scale, gate_cap, den_eps, out_eps;
    const float* norm_w;                /* [heads*vdim] */
    int   q_off, k_off, v_off, g_off, i_off, f_off;   /* in a row of the fp32 input: q, k [heads*dim]; v, g [heads*vdim]; i, f [heads] */
    /* set by t12_memory_plan: */
    int   dim_p;                        /* key channels padded (zero) to 64, 128, 256 or 512 */
    size_t state_elems;                 /* floats per state: [heads][vdim + 1][dim_p], then m [heads] */
    size_t work_floats;                 /* workspace for passes of up to `rows` rows */
    float* state;                       /* [region][2][state_elems] */
} T12MatrixMemory;
int t12_memory_plan(T12MatrixMemory* m, int rows);
/* exact: prompt runs take the recurrence token by token in fp32 instead of the matrix-core form by chunks (whose keys,
 * queries and values are bf16).  in: fp32 [n, ld], bias: fp32 [ld], added to every row. */
int t12_matrix_memory(const T12MatrixMemory* m, const float* in, const float* bias, int ld, const T12Row* rows, int n, int run,
                      int exact, float* work, void* out, int out_f32, int out_ld, void* stream);

/* ---- latent attention ----------------------------------------------------------------------------------------------
 * Keys and values of all heads come from one cached vector per token: the latent c (RMS norm of `rank` projections) and a
 * rotated key part of rot_dim channels.  Per head, with up-projections U_k [dim, rank] and U_v [vdim, rank]:
 *     score(i, j) = scale (q_i . U_k c_j + rot(q^r_i) . rot(k^r_j)), j <= i;   out_i = sigmoid(g) sum_j softmax_j U_v c_j
 * Channel i of a rotated part is paired with channel i + rot_dim / 2 and turned by position * freqs[i].
 * The up-projections are taken out of the sum over keys: q is multiplied with U_k, the mean latent with U_v, so scores and
 * values read the cached vectors alone.
 *
 * The cache of a region: blocks of 32 positions, position p in row p % 32; a row holds c [rank] padded (zeros) to rank_p, then
 * the rotated part padded to row_p - rank_p.  bf16 caches of sizes that have a matrix-core instance (rank_p 64, 128, 256
 * or 512, row_p = rank_p + 64) keep the row's 16-byte pieces in an order that spreads equal pieces of neighbouring positions over the banks. */
typedef struct T12LatentAttn {
    int   heads, dim, rot_dim, vdim, rank;
    float scale, eps;
    int   elem_bytes;                   /* cache element: 2 bf16, 4 fp32 */
    struct T12Segment const* k_up;      /* host; [heads*rank, dim]: U_k transposed, head by head */
    struct T12Segment const* v_up;      /* host; [heads*vdim, rank] */
    const float* norm_w;                /* [rank] */
    const float* freqs;                 /* [rot_dim / 2] */
    int   q_off, c_off, g_off;          /* in a row of the fp32 input: q [heads][dim + rot_dim], c | k^r [rank + rot_dim], g [heads] */
    /* set by t12_latent_plan: */
    int   rank_p, row_p, matrix;
    size_t cache_elems;                 /* per region */
    size_t work_floats;                 /* workspace for passes of up to `rows` rows */
    void* cache;                        /* regions back to back; zeroed before first use */
} T12LatentAttn;
int t12_latent_plan(T12LatentAttn* a, int max_positions, int rows);
/* Stores every row's latent, then attends.  max_position: no row stands beyond it. */
int t12_latent_attention(const T12LatentAttn* a, const float* in, int ld, const T12Row* rows, int n, int run, int max_position,
                         float* work, void* out, int out_f32, int out_ld, void* stream);

/* ---- decode step of the two mixers in one launch ------------------------------------------------------------------
 * For rows that are sequences of their own: t12_window_store + t12_window_attention (into attn_out) and, when d is given,
 * t12_delta_rule (into delta_out), bf16 outputs of row stride out_ld, every row's key and value stored by the launch
 * itself.  max_position: no row stands beyond it (a hint for how the keys are split over workgroups).  ws
 * (t12_parallel_step_ws_floats() floats) and counters (T12_STEP_MAX_ITEMS ints, zero before the first launch and zero
 * again after every one) carry partial sums of long windows; both may be NULL.  Returns 1 when the shape has no such
 * kernel (fp32 cache, dim or vdim above 256, a delta head above 128, more than T12_STEP_MAX_ITEMS rows x delta heads --
 * without d this last one does not count): use the separate calls. */
#define T12_STEP_MAX_ITEMS 512
size_t t12_parallel_step_ws_floats(void);
int t12_parallel_step(const T12WindowAttn* a, const T12DeltaRule* d, const float* in, const float* bias, int ld,
                      const T12Row* rows, int n, int max_position, float attn_scale, float delta_scale, void* attn_out,
                      void* delta_out, int out_ld, float* ws, int* counters, void* stream);

#ifdef __cplusplus
}
#endif
#endif /* T12_MIXERS_H */
