// The layer stack of Gamilorn models (gamilorn.h): what a state holds, and a pass of rows through the layers.
//
// A state owns per layer a ring cache of keys and values and a pair of recurrent states for every sequence region
// (t12_mixers.h).  Regions, rows and the turning of the pair: regions.h.
#include <algorithm>
#include <cstdio>

#include "gamilorn.h"
#include "regions.h"
#include "t12_glue.h"

namespace gamilorn {
namespace {

constexpr int kPromptRows = 512;                 // tokens per prompt pass unless the caller chooses
constexpr int kOverlapRows = 128;                // from this many prompt rows on the two mixers run side by side on two streams
constexpr float kUnitEps = 1e-6f;                // under the root of a key's length
constexpr float kDecayRate = 0.60653065971263342f;   // exp(-1/2)

struct State : RegionState {
    std::vector<T12WindowAttn> attn;             // per layer, with the cache
    std::vector<T12DeltaRule> delta;             // per layer, with the states
    float* in = nullptr;                         // [rows, in_rows]
    float* up = nullptr;                         // [rows, ff]
    float* work = nullptr;                       // delta rule
    void* h = nullptr;                           // normed input of a block: bf16 (fp32 in 32-bit states) [rows, width]
    void* cat = nullptr;                         // both mixers' outputs [rows, out_cols]
    void* act = nullptr;                         // feed-forward activations [rows, ff]
    float* step_ws = nullptr;                    // decode step: partial sums of long windows, arrival counters
    int* step_count = nullptr;
    hipEvent_t fork = nullptr, join = nullptr;   // prompt passes: the recurrent half runs on the state's second stream
    bool fused_b1 = false;                       // one sequence, bf16: a decode step in five launches per layer
};

State* state_of(const InferenceState* s) { return (State*)(StateCommon*)s->impl; }

bool fused_b1_eligible(const Model* model)
{
    const Data& d = *data_of(model);
    if (!region_norm_width(d.config.width) || !exp_ok(model->output_proj)) return false;
    for (const Layer& L : d.layers) {
        if (!region_fused_tensor(L.w_in) || !region_fused_tensor(L.w_out)) return false;
        if (L.c.ff && (!region_fused_tensor(L.up) || !region_fused_tensor(L.down))) return false;
    }
    return true;
}

InferenceState* create(Model* model, const StateOptions& o)
{
    const Data& d = *data_of(model);
    const Config& c = d.config;
    if (o.max_seq_len > c.max_positions) {
        fprintf(stderr, "ERROR: %d positions asked for, the model has %d\n", o.max_seq_len, c.max_positions);
        return nullptr;
    }
    auto* st = new State();
    st->shape(o, model->max_seq_len, kPromptRows);
    const int regions = st->regions();
    const size_t R = (size_t)st->rows, el = st->f32 ? 4 : 2;

    // sizes first: refuse what does not fit
    size_t need = 0, in = 0, ff = 0, work = 0, cat = 0;
    for (const Layer& L : d.layers) {
        const LayerConfig& k = L.c;
        T12WindowAttn a = {};
        a.heads = k.heads;
        a.kv_heads = k.kv_heads;
        a.dim = k.dim;
        a.vdim = k.vdim;
        a.window = k.window;
        a.keep_first = k.keep_first;
        a.scale = k.scale;
        a.elem_bytes = (int)el;
        a.q_off = k.q_off();
        a.k_off = k.k_off();
        a.v_off = k.v_off();
        a.head_bias = L.head_bias;
        must(t12_window_plan(&a, st->max_seq, st->rows), "window plan");
        T12DeltaRule r = {};
        r.heads = k.d_heads;
        r.dim = k.d_dim;
        r.rank = k.rank;
        r.unit_eps = kUnitEps;
        r.decay_rate = kDecayRate;
        r.out_eps = c.eps;
        r.w2t = L.w2t;
        r.w0 = L.w0;
        r.norm_w = L.o_norm;
        r.r_off = k.r_off();
        r.k_off = k.dk_off();
        r.v_off = k.dv_off();
        r.a_off = k.a_off();
        r.g_off = k.g_off();
        r.w1_off = k.w1_off();
        must(t12_delta_plan(&r), "delta plan");
        st->attn.push_back(a);
        st->delta.push_back(r);
        need += regions * ((a.k_elems + a.v_elems) * el + 2 * r.state_elems * sizeof(float));
        in = std::max(in, (size_t)k.in_rows());
        ff = std::max(ff, (size_t)k.ff);
        cat = std::max(cat, (size_t)k.out_cols());
        work = std::max(work, r.work_elems);
    }
    size_t free_b = 0, total_b = 0;
    (void)hipMemGetInfo(&free_b, &total_b);
    const size_t acts = R * ((in + ff + work + 2 * (size_t)c.width) * 4 + (c.width + cat + ff) * el);
    if (need + acts > free_b) {
        fprintf(stderr, "ERROR: %d sequence regions need %.1f GB, %.1f GB free\n", regions, (need + acts) / 1e9, free_b / 1e9);
        delete st;
        return nullptr;
    }
    InferenceState* s = new_state(model, o.batch_size, st->rows, st);
    auto own = [&](size_t bytes) { return st->own(bytes); };
    auto zeroed = [&](size_t bytes) { return st->own_zeroed(bytes, s->stream); };
    for (size_t i = 0; i < d.layers.size(); i++) {
        st->attn[i].k = zeroed(regions * st->attn[i].k_elems * el);
        st->attn[i].v = zeroed(regions * st->attn[i].v_elems * el);
        st->delta[i].state = (float*)zeroed(regions * 2 * st->delta[i].state_elems * sizeof(float));
    }
    check_gpu(hipEventCreateWithFlags(&st->fork, hipEventDisableTiming), "event");
    check_gpu(hipEventCreateWithFlags(&st->join, hipEventDisableTiming), "event");
    st->d_rows = (T12Row*)own(R * sizeof(T12Row));
    st->in = (float*)own(R * in * 4);
    st->up = (float*)own(R * ff * 4);
    st->work = (float*)own(R * work * 4);
    st->h = own(R * c.width * el);
    st->cat = own(R * cat * el);
    st->act = own(R * ff * el);
    if (!st->f32) {
        st->step_ws = (float*)own(t12_parallel_step_ws_floats() * sizeof(float));
        st->step_count = (int*)zeroed(T12_STEP_MAX_ITEMS * sizeof(int));
        st->fused_b1 = !region_no_fuse() && o.batch_size == 1 && fused_b1_eligible(model);
    }
    check_gpu(hipMalloc((void**)&s->hidden, R * c.width * 4), "hipMalloc");
    check_gpu(hipMalloc((void**)&s->hidden2, R * c.width * 4), "hipMalloc");
    printf("  Sequence regions: %d, %.3f GB, %d rows per pass\n", regions, need / 1e9, st->rows);
    return s;
}

void release_state(InferenceState* s)
{
    State* st = state_of(s);
    for (void* p : st->owned) (void)hipFree(p);
    for (hipEvent_t e : {st->fork, st->join})
        if (e) (void)hipEventDestroy(e);
}

// act = xIELU(up . h): in the GEMM's epilogue, in the sum over its K splits, or on its own.
void up_activation(State* st, const Layer& L, int n, int R, hipStream_t q)
{
    const int ff = L.c.ff;
    if (!st->f32 && R > 1) {
        T12Segment g = seg_of(L.up, st->up, ff);
        const int rc = t12_gemm_act(&g, st->h, n, n, R, &L.xielu, st->act, ff, q);
        if (rc < 0) must(rc, "up projection");
        if (rc == T12_OK) return;
        T12GemmPartials part;
        must(t12_gemm_deferred(&g, 1, st->h, n, ff, n, R, &part, q), "up projection");
        if (part.nsplit > 1) {
            must(t12_act_partials(&part, &L.xielu, st->act, ff, R, q), "activation");
            return;
        }
    } else {
        region_linear(L.up, st->up, ff, st->h, n, R, st->f32, q);
    }
    must(t12_act(st->up, &L.xielu, st->act, st->f32, (size_t)R * ff, q), "activation");
}

// cur += w . act, then h = norm(cur): what ends the mixer and the feed-forward of a layer.
void close_block(const CompressedWeight& w, const void* act, int K, const float* norm, float eps, int R, State* st, float*& cur,
                 float*& other, hipStream_t q)
{
    const int n = w.M;
    if (st->f32) {
        region_linear_add_f32(w, cur, act, K, R, q);
        must(t12_rms_norm_f32(cur, norm, (float*)st->h, n, eps, R, q), "norm");
        return;
    }
    T12Segment g = seg_of(w, other, n);
    if (R > 1) {
        run_linear_add_norm(&g, (const int16_t*)act, K, R, cur, norm, eps, (int16_t*)st->h, q);
    } else {
        run_linear(&g, 1, (const int16_t*)act, K, 1, q);
        launch_add_rms_norm_bf16_batch(other, cur, norm, (int16_t*)st->h, n, eps, 1, q);
    }
    std::swap(cur, other);
}

void head(InferenceState* s, State* st, const Config& c, const void* act, int R, float* out)
{
    region_linear(s->model->output_proj, out, c.vocab, act, c.width, R, st->f32, s->stream);
    const T12Act cap = {T12_ACT_SOFTCAP, c.softcap, 0.0f};
    if (c.softcap > 0.0f)
        must(t12_act(out, &cap, out, 1, (size_t)R * c.vocab, s->stream), "logit cap");
}

// Both mixers of layer i on the projections in st->in, into st->cat.
void mixers(InferenceState* s, const Layer& L, size_t i, int R, int run, int max_position)
{
    State* st = state_of(s);
    hipStream_t q = s->stream;
    const LayerConfig& k = L.c;
    const int ld = k.in_rows(), oc = k.out_cols();
    char* right = (char*)st->cat + (size_t)k.att() * (st->f32 ? 4 : 2);
    int rc = 1;
    if (!run && !st->f32) {
        // few rows: both mixers in one launch; many: the attention's own, and the rule's kernels, which share more of a token
        for (T12DeltaRule* d : {&st->delta[i], (T12DeltaRule*)nullptr}) {
            rc = t12_parallel_step(&st->attn[i], d, st->in, L.in_bias, ld, st->d_rows, R, max_position, k.left_scale, k.right_scale, st->cat,
                                   d ? right : nullptr, oc, st->step_ws, st->step_count, q);
            if (rc < 0) must(rc, "mixer step");
            if (rc == T12_OK && d) return;
            if (rc == T12_OK) break;
        }
    }
    // (the attention fills the chip and the recurrence, whose time axis is a chain, does not)
    const bool apart = run && R >= kOverlapRows;
    hipStream_t q2 = apart ? s->stream2 : q;
    if (apart) {
        check_gpu(hipEventRecord(st->fork, q), "hipEventRecord");
        check_gpu(hipStreamWaitEvent(q2, st->fork, 0), "hipStreamWaitEvent");
    }
    must(t12_delta_rule(&st->delta[i], st->in, L.in_bias, ld, st->d_rows, R, run, k.right_scale, st->work, right, st->f32, oc, q2),
         "delta rule");
    if (apart) check_gpu(hipEventRecord(st->join, q2), "hipEventRecord");
    if (rc != T12_OK) {
        must(t12_window_store(&st->attn[i], st->in, L.in_bias, ld, st->d_rows, R, run, q), "cache store");
        must(t12_window_attention(&st->attn[i], st->in, L.in_bias, ld, st->d_rows, R, run, k.left_scale, st->cat, st->f32, oc, q),
             "window attention");
    }
    if (apart) check_gpu(hipStreamWaitEvent(q, st->join, 0), "hipStreamWaitEvent");
}

// One row in five launches per layer:
//   RMSNorm + all projections of both mixers                 t12_gemv_norm
//   cache store + attention + recurrent step                 t12_parallel_step
//   both output projections + residual add                   t12_gemv_add
//   RMSNorm + up + xIELU                                     t12_gemv_act
//   down + residual add                                      t12_gemv_add
void pass_b1_fused(InferenceState* s, int position)
{
    State* st = state_of(s);
    const Data& d = *data_of(s->model);
    const Config& c = d.config;
    const int n = c.width;
    hipStream_t q = s->stream;
    must(t12_embed_positions(s->model->token_embd, c.vocab, d.pos_table, c.max_positions, s->d_tokens, st->d_rows, s->hidden, n, 1, q),
         "embedding");
    float *cur = s->hidden, *other = s->hidden2;
    for (size_t i = 0; i < d.layers.size(); i++) {
        const Layer& L = d.layers[i];
        const LayerConfig& k = L.c;
        T12Segment g = seg_of(L.w_in, st->in, k.in_rows());
        must(t12_gemv_norm(&g, 1, cur, nullptr, L.norm1, c.eps, nullptr, n, q), "mixer decode-GEMV");
        mixers(s, L, i, 1, 0, position);
        g = seg_of(L.w_out, other, n);
        must(t12_gemv_add(&g, st->cat, k.out_cols(), cur, q), "output decode-GEMV");
        std::swap(cur, other);
        if (!k.ff) continue;
        g = seg_of(L.up, nullptr, k.ff);
        must(t12_gemv_act(&g, nullptr, cur, L.norm2, c.eps, n, &L.xielu, st->act, q), "up decode-GEMV");
        g = seg_of(L.down, other, n);
        must(t12_gemv_add(&g, st->act, k.ff, cur, q), "down decode-GEMV");
        std::swap(cur, other);
    }
    T12Segment g = seg_of(s->model->output_proj, s->logits, c.vocab);
    const T12Act cap = {T12_ACT_SOFTCAP, c.softcap, 0.0f};
    // thousands of workgroups would each rebuild the normed input: from there on one small kernel does it once
    const bool apart = c.vocab >= 32768;
    if (apart) launch_rms_norm_bf16_batch(cur, s->model->output_norm, (int16_t*)st->h, n, c.eps, 1, q);
    if (c.softcap > 0.0f) must(t12_gemv_act(&g, apart ? st->h : nullptr, cur, s->model->output_norm, c.eps, n, &cap, nullptr, q), "head decode-GEMV");
    else if (apart) must(t12_gemv(&g, 1, st->h, n, q), "head decode-GEMV");
    else must(t12_gemv_norm(&g, 1, cur, nullptr, s->model->output_norm, c.eps, nullptr, n, q), "head decode-GEMV");
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
    must(t12_embed_positions(s->model->token_embd, c.vocab, d.pos_table, c.max_positions, s->d_tokens, st->d_rows, s->hidden, n, R, q),
         "embedding");
    float *cur = s->hidden, *other = s->hidden2;
    if (st->f32) must(t12_rms_norm_f32(cur, d.layers[0].norm1, (float*)st->h, n, c.eps, R, q), "norm");
    else launch_rms_norm_bf16_batch(cur, d.layers[0].norm1, (int16_t*)st->h, n, c.eps, R, q);
    for (size_t i = 0; i < d.layers.size(); i++) {
        const Layer& L = d.layers[i];
        const LayerConfig& k = L.c;
        const int ld = k.in_rows(), oc = k.out_cols();
        region_linear(L.w_in, st->in, ld, st->h, n, R, st->f32, q);
        mixers(s, L, i, R, run, max_position);
        const float* next = i + 1 < d.layers.size() ? d.layers[i + 1].norm1 : s->model->output_norm;
        close_block(L.w_out, st->cat, oc, k.ff ? L.norm2 : next, c.eps, R, st, cur, other, q);
        if (!k.ff) continue;
        up_activation(st, L, n, R, q);
        close_block(L.down, st->act, k.ff, next, c.eps, R, st, cur, other, q);
    }
    const size_t row_bytes = (size_t)n * (st->f32 ? 4 : 2);
    if (lr.mode == LOGITS_ALL) {
        head(s, st, c, st->h, R, s->logits);
    } else if (lr.mode == LOGITS_LAST_ROW) {
        head(s, st, c, (char*)st->h + (R - 1) * row_bytes, 1, lr.out);
    } else if (lr.mode == LOGITS_ROWS && lr.n_rows > 0) {
        // (the residual stream's other buffer is free again)
        must(t12_util_gather_rows(other, st->h, row_bytes, lr.rows, lr.n_rows, q), "row gather");
        head(s, st, c, other, lr.n_rows, lr.out);
    }
}

void forward(InferenceState* s, const int* token_ids) { region_forward(s, token_ids, pass); }
void prompt(InferenceState* s, const PromptPass& p) { region_prompt(s, p, pass); }

}  // namespace
}  // namespace gamilorn

FamilyRun kGamilornRun = {
    gamilorn::create, gamilorn::release_state, region_max_positions, gamilorn::forward, gamilorn::prompt, region_retract,
    nullptr,                                     // a recurrent state holds its whole past
};
