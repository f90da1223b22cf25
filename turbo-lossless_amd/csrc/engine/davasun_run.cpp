// The layer stack of Davasun models (davasun.h): what a state holds, and a pass of rows through the layer runs.
//
// A state owns for every layer run a latent cache or a pair of matrix memories per sequence region (t12_mixers.h).  Regions,
// rows and the turning of the pair: regions.h.
#include <algorithm>
#include <cmath>
#include <cstdio>

#include "davasun.h"
#include "regions.h"
#include "t12_glue.h"

namespace davasun {
namespace {

constexpr int kPromptRows = 512;                 // tokens per prompt pass unless the caller chooses
constexpr float kDenominatorEps = 1e-6f;         // beside the normaliser of a matrix memory
constexpr float kGateSlope = 1.702f, kUpOffset = 1.0f;   // feed-forward: g sigmoid(slope g) (u + offset)

// A layer run: the layer, and the past of this run.
struct Run {
    const Layer* layer;
    T12MatrixMemory memory;
    T12LatentAttn latent;
    T12Segment k_up, v_up;
};

struct State : RegionState {
    std::vector<Run> runs;
    float* in = nullptr;                         // [rows, in_ld]
    float *gate = nullptr, *up = nullptr;        // [rows, ff]
    float* y = nullptr;                          // a sublayer's output [rows, width]
    float* work = nullptr;                       // mixers
    void* h = nullptr;                           // normed input of a sublayer: bf16 (fp32 in 32-bit states) [rows, width]
    void* mix = nullptr;                         // the mixer's output [rows, out_cols]
    void* act = nullptr;                         // feed-forward activations [rows, ff]
    bool no_fuse = false;                        // debugging: no products with prologues or epilogues
    bool fused_b1 = false;                       // one sequence, bf16: norms in the prologues of the projections
};

State* state_of(const InferenceState* s) { return (State*)(StateCommon*)s->impl; }

// Every tensor behind a norm can take the decode-GEMV with the norms in its prologue.
bool fused_b1_eligible(const Model* model)
{
    const Data& d = *data_of(model);
    if (!region_norm_width(d.config.width) || !exp_ok(model->output_proj)) return false;
    for (const Layer& L : d.layers)
        if (!exp_ok(L.w_in) || (L.c.ff && (!exp_ok(L.gate) || !exp_ok(L.up)))) return false;
    return true;
}

T12MatrixMemory memory_of(const Layer& L, float eps)
{
    const LayerConfig& k = L.c;
    T12MatrixMemory m = {};
    m.heads = k.heads;
    m.dim = k.dim;
    m.vdim = k.vdim;
    m.q_scale = (float)(1.0 / sqrt((double)k.dim));
    m.gate_cap = k.gate_cap;
    m.den_eps = kDenominatorEps;
    m.out_eps = eps;
    m.norm_w = L.o_norm;
    m.q_off = 0;
    m.k_off = k.k_off();
    m.v_off = k.v_off();
    m.g_off = k.m_g_off();
    m.i_off = k.i_off();
    m.f_off = k.f_off();
    return m;
}

T12LatentAttn latent_of(const Layer& L, float eps, int elem_bytes)
{
    const LayerConfig& k = L.c;
    T12LatentAttn a = {};
    a.heads = k.heads;
    a.dim = k.dim;
    a.rot_dim = k.rot_dim;
    a.vdim = k.vdim;
    a.rank = k.rank;
    a.scale = k.scale;
    a.eps = eps;
    a.elem_bytes = elem_bytes;
    a.norm_w = L.o_norm;
    a.freqs = L.freqs;
    a.q_off = 0;
    a.c_off = k.c_off();
    a.g_off = k.a_g_off();
    return a;
}

InferenceState* create(Model* model, const StateOptions& o)
{
    const Data& d = *data_of(model);
    const Config& c = d.config;
    auto* st = new State();
    st->shape(o, model->max_seq_len, kPromptRows);
    const int regions = st->regions();
    const size_t R = (size_t)st->rows, el = st->f32 ? 4 : 2;

    // sizes first: refuse what does not fit
    size_t need = 0, in = 0, ff = 0, work = 0, mix = 0;
    for (int i : c.runs()) {
        Run r = {};
        r.layer = &d.layers[i];
        const LayerConfig& k = r.layer->c;
        if (k.kind == MLSTM) {
            r.memory = memory_of(*r.layer, c.eps);
            must(t12_memory_plan(&r.memory, st->rows), "memory plan");
            need += regions * 2 * r.memory.state_elems * sizeof(float);
            work = std::max(work, r.memory.work_floats);
        } else {
            r.latent = latent_of(*r.layer, c.eps, (int)el);
            must(t12_latent_plan(&r.latent, st->max_seq, st->rows), "latent plan");
            need += regions * r.latent.cache_elems * el;
            work = std::max(work, r.latent.work_floats);
            r.k_up = seg_of(r.layer->k_up, nullptr, 0);
            r.v_up = seg_of(r.layer->v_up, nullptr, 0);
        }
        in = std::max(in, (size_t)k.in_ld());
        ff = std::max(ff, (size_t)k.ff);
        mix = std::max(mix, (size_t)k.out_cols());
        st->runs.push_back(r);
    }
    size_t free_b = 0, total_b = 0;
    (void)hipMemGetInfo(&free_b, &total_b);
    const size_t acts = R * ((in + 2 * ff + 3 * (size_t)c.width) * 4 + (c.width + mix + ff) * el) + work * 4;
    if (need + acts > free_b) {
        fprintf(stderr, "ERROR: %d sequence regions need %.1f GB, %.1f GB free\n", regions, (need + acts) / 1e9, free_b / 1e9);
        delete st;
        return nullptr;
    }
    InferenceState* s = new_state(model, o.batch_size, st->rows, st);
    for (Run& r : st->runs) {
        if (r.layer->c.kind == MLSTM) {
            r.memory.state = (float*)st->own_zeroed(regions * 2 * r.memory.state_elems * sizeof(float), s->stream);
        } else {
            r.latent.cache = st->own_zeroed(regions * r.latent.cache_elems * el, s->stream);
            r.latent.k_up = &r.k_up;
            r.latent.v_up = &r.v_up;
        }
    }
    st->d_rows = (T12Row*)st->own(R * sizeof(T12Row));
    st->in = (float*)st->own(R * in * 4);
    st->gate = (float*)st->own(R * ff * 4);
    st->up = (float*)st->own(R * ff * 4);
    st->y = (float*)st->own(R * c.width * 4);
    st->work = (float*)st->own(work * 4);
    st->h = st->own(R * c.width * el);
    st->mix = st->own(R * mix * el);
    st->act = st->own(R * ff * el);
    st->no_fuse = region_no_fuse();
    st->fused_b1 = !st->f32 && !st->no_fuse && o.batch_size == 1 && fused_b1_eligible(model);
    check_gpu(hipMalloc((void**)&s->hidden, R * c.width * 4), "hipMalloc");
    check_gpu(hipMalloc((void**)&s->hidden2, R * c.width * 4), "hipMalloc");
    printf("  Sequence regions: %d, %.3f GB, %d rows per pass\n", regions, need / 1e9, st->rows);
    return s;
}

void release_state(InferenceState* s)
{
    for (void* p : state_of(s)->owned) (void)hipFree(p);
}

T12Glu unit_of(const LayerConfig& k) { return {k.limit, kGateSlope, kUpOffset}; }

// The mixer of a run on the projections in st->in, into st->mix.
void mixer(State* st, const Run& r, int R, int run, int max_position, hipStream_t q)
{
    const LayerConfig& k = r.layer->c;
    if (k.kind == MLSTM)
        must(t12_matrix_memory(&r.memory, st->in, r.layer->in_bias, k.in_ld(), st->d_rows, R, run, st->f32, st->work, st->mix, st->f32,
                               k.out_cols(), q), "matrix memory");
    else
        must(t12_latent_attention(&r.latent, st->in, k.in_ld(), st->d_rows, R, run, max_position, st->work, st->mix, st->f32, k.out_cols(), q),
             "latent attention");
}

// cur += norm(w . act) with gain `post`, then h = norm(cur) with gain `next`: what ends a sublayer.
void close_sublayer(const CompressedWeight& w, const void* act, int K, const float* post, const float* next, float eps, int R, State* st,
                    float*& cur, float*& other, hipStream_t q)
{
    const int n = w.M;
    T12GemmPartials part = {nullptr, 1, 0, 0};
    if (!st->f32 && R > 1) {
        T12Segment g = seg_of(w, st->y, n);
        must(t12_gemm_deferred(&g, 1, (const int16_t*)act, K, n, K, R, &part, q), "output projection");
    } else {
        region_linear(w, st->y, n, act, K, R, st->f32, q);
    }
    must(t12_post_norm_add(st->y, part.nsplit > 1 ? &part : nullptr, cur, post, next, eps, other, st->h, st->f32, n, R, q), "norms");
    std::swap(cur, other);
}

// act = unit(gate . h, up . h): in the product's epilogue where the shape has such a kernel.
void gated_up(State* st, const Layer& L, int n, int R, hipStream_t q)
{
    const int ff = L.c.ff;
    const T12Glu unit = unit_of(L.c);
    T12Segment g = seg_of(L.gate, st->gate, ff), u = seg_of(L.up, st->up, ff);
    if (!st->f32 && R > 1 && !st->no_fuse) {
        const int rc = t12_gemm_glu(&g, &u, &unit, st->h, n, n, R, st->act, ff, q);
        if (rc < 0) must(rc, "gate|up projection");
        if (rc == T12_OK) return;
    }
    const bool whole = n % 16 == 0 && n <= 81920 && exp_ok(L.gate) && exp_ok(L.up);
    if (!st->f32 && R == 1 && whole && !st->no_fuse) {
        must(t12_gemv_glu(&g, &u, &unit, st->h, n, st->act, q), "gate|up decode-GEMV");
        return;
    }
    T12Segment both[2] = {g, u};
    if (st->f32) must(t12_gemm_f32(both, 2, (const float*)st->h, n, ff, n, R, 0, q), "32-bit linear");
    else run_linear(both, 2, (const int16_t*)st->h, n, R, q);
    must(t12_glu(st->gate, st->up, &unit, st->act, st->f32, (size_t)R * ff, q), "gated unit");
}

// One row.  A sublayer's output waits in st->y: the prologue of the next projection puts it through its norm, adds it to the
// residual and norms the sum.  mLSTM: projections, memory, its output, output projection; latent attention: projections, key
// projection beside the cache store, attention, value projection, output projection; feed-forward: gate|up with the unit, down.
void pass_b1_fused(InferenceState* s, int position)
{
    State* st = state_of(s);
    const Data& d = *data_of(s->model);
    const Config& c = d.config;
    const int n = c.width;
    hipStream_t q = s->stream;
    must(t12_embed_norm(s->model->token_embd, c.vocab, s->d_tokens, d.embed_norm, c.eps, s->hidden, n, 1, q), "embedding");
    float *cur = s->hidden, *other = s->hidden2;
    bool waits = false;                                            // st->y goes through a norm of gain `post`
    float post = 1.0f;
    auto project = [&](T12Segment g, const float* norm, float gain) {
        if (!waits) {
            must(t12_gemv_norm(&g, 1, cur, nullptr, norm, c.eps, nullptr, n, q), "decode-GEMV");
            return;
        }
        must(t12_gemv_gain_norm(&g, 1, st->y, cur, post, gain, c.eps, other, n, q), "decode-GEMV");
        std::swap(cur, other);
    };
    for (const Run& r : st->runs) {
        const Layer& L = *r.layer;
        project(seg_of(L.w_in, st->in, L.c.in_ld()), L.norm1, L.gain1);
        mixer(st, r, 1, 0, position, q);
        region_linear(L.w_out, st->y, n, st->mix, L.c.out_cols(), 1, false, q);
        waits = true;
        post = L.gain1b;
        if (!L.c.ff) continue;
        const T12Glu unit = unit_of(L.c);
        T12Segment g = seg_of(L.gate, nullptr, L.c.ff), u = seg_of(L.up, nullptr, L.c.ff);
        must(t12_gemv_glu_gain_norm(&g, &u, &unit, st->y, cur, post, L.gain2, c.eps, other, n, st->act, q), "gate|up decode-GEMV");
        std::swap(cur, other);
        region_linear(L.down, st->y, n, st->act, L.c.ff, 1, false, q);
        post = L.gain2b;
    }
    T12Segment g = seg_of(s->model->output_proj, s->logits, c.vocab);
    if (c.vocab >= 8192) {      // thousands of workgroups would each rebuild the normed input: one small kernel does it once
        const Layer& L = *st->runs.back().layer;
        must(t12_post_norm_add(st->y, nullptr, cur, L.c.ff ? L.norm2b : L.norm1b, s->model->output_norm, c.eps, other, st->h, 0, n, 1, q), "norms");
        must(t12_gemv(&g, 1, st->h, n, q), "head decode-GEMV");
    } else {
        project(g, s->model->output_norm, d.final_gain);
    }
}

void pass(InferenceState* s, int R, int run, int max_position, const LogitsRequest& lr)
{
    State* st = state_of(s);
    if (!run && st->fused_b1) {
        pass_b1_fused(s, max_position);
        return;
    }
    const Data& d = *data_of(s->model);
    const Config& c = d.config;
    const int n = c.width;
    hipStream_t q = s->stream;
    must(t12_embed_norm(s->model->token_embd, c.vocab, s->d_tokens, d.embed_norm, c.eps, s->hidden, n, R, q), "embedding");
    float *cur = s->hidden, *other = s->hidden2;
    const float* first = st->runs[0].layer->norm1;
    if (st->f32) must(t12_rms_norm_f32(cur, first, (float*)st->h, n, c.eps, R, q), "norm");
    else launch_rms_norm_bf16_batch(cur, first, (int16_t*)st->h, n, c.eps, R, q);
    for (size_t i = 0; i < st->runs.size(); i++) {
        const Run& r = st->runs[i];
        const Layer& L = *r.layer;
        const LayerConfig& k = L.c;
        region_linear(L.w_in, st->in, k.in_ld(), st->h, n, R, st->f32, q);
        mixer(st, r, R, run, max_position, q);
        const float* next = i + 1 < st->runs.size() ? st->runs[i + 1].layer->norm1 : s->model->output_norm;
        close_sublayer(L.w_out, st->mix, k.out_cols(), L.norm1b, k.ff ? L.norm2 : next, c.eps, R, st, cur, other, q);
        if (!k.ff) continue;
        gated_up(st, L, n, R, q);
        close_sublayer(L.down, st->act, k.ff, L.norm2b, next, c.eps, R, st, cur, other, q);
    }
    auto head = [&](const void* act, int rows, float* out) { region_linear(s->model->output_proj, out, c.vocab, act, n, rows, st->f32, q); };
    const size_t row_bytes = (size_t)n * (st->f32 ? 4 : 2);
    if (lr.mode == LOGITS_ALL) {
        head(st->h, R, s->logits);
    } else if (lr.mode == LOGITS_LAST_ROW) {
        head((char*)st->h + (R - 1) * row_bytes, 1, lr.out);
    } else if (lr.mode == LOGITS_ROWS && lr.n_rows > 0) {
        // (the residual stream's other buffer is free again)
        must(t12_util_gather_rows(other, st->h, row_bytes, lr.rows, lr.n_rows, q), "row gather");
        head(other, lr.n_rows, lr.out);
    }
}

void forward(InferenceState* s, const int* token_ids) { region_forward(s, token_ids, pass); }
void prompt(InferenceState* s, const PromptPass& p) { region_prompt(s, p, pass); }

}  // namespace
}  // namespace davasun

FamilyRun kDavasunRun = {
    davasun::create, davasun::release_state, region_max_positions, davasun::forward, davasun::prompt, region_retract,
    nullptr,                                     // a recurrent state holds its whole past
};
