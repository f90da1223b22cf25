// Sequence regions with recurrent states, and the passes of rows over them (regions.h).
#include "regions.h"

#include <algorithm>
#include <cstdlib>

namespace {
RegionState* state_of(const InferenceState* s) { return (RegionState*)(StateCommon*)s->impl; }

// A region's recurrent states only go forward: the next token must be the one after what they have absorbed, or the
// first of a new sequence (which the kernels start from zero).
void enter(RegionState* st, int region, int position)
{
    if (position == 0) st->absorbed[region] = 0;
    if (st->absorbed[region] != position)
        engine_fail("position %d: the recurrent state of this sequence stands at %d (it continues there or restarts at 0)", position,
                    st->absorbed[region]);
}
}  // namespace

void* RegionState::own(size_t bytes)
{
    void* p = nullptr;
    check_gpu(hipMalloc(&p, std::max<size_t>(bytes, 16)), "hipMalloc");
    owned.push_back(p);
    return p;
}

void* RegionState::own_zeroed(size_t bytes, hipStream_t st)
{
    void* p = own(bytes);
    check_gpu(hipMemsetAsync(p, 0, bytes, st), "hipMemsetAsync");
    return p;
}

void RegionState::shape(const StateOptions& o, int context, int default_rows)
{
    f32 = o.precision == PRECISION_FP32;
    per_seq = o.per_sequence;
    max_seq = o.per_sequence && o.max_seq_len > 0 ? o.max_seq_len : context;
    rows = std::max(o.batch_size, std::min(o.prompt_rows > 0 ? o.prompt_rows : default_rows, max_seq));
    absorbed.assign(o.per_sequence ? o.batch_size : 1, 0);
    parity.assign(absorbed.size(), 0);
}

void region_forward(InferenceState* s, const int* token_ids, RegionPass pass)
{
    RegionState* st = state_of(s);
    const int B = s->batch_size;
    std::vector<T12Row> rows(B);
    for (int b = 0; b < B; b++) {
        const int region = st->per_seq ? b : 0;
        if (!st->per_seq && s->positions[b] != s->positions[0])
            engine_fail("the rows of a lock-step state must stand at one position");
        enter(st, region, s->positions[b]);
        rows[b] = {s->positions[b], region * 2 + st->parity[region]};
    }
    if (token_ids) check_gpu(hipMemcpyAsync(s->d_tokens, token_ids, B * sizeof(int), hipMemcpyHostToDevice, s->stream), "token copy");
    must(t12_rows_list(st->d_rows, rows.data(), B, s->stream), "row table");
    int max_position = 0;
    for (const T12Row& r : rows) max_position = std::max(max_position, r.position);
    LogitsRequest lr;
    lr.mode = LOGITS_ALL;
    pass(s, B, 0, max_position, lr);
    for (int& a : st->absorbed) a++;
    for (int& p : st->parity) p ^= 1;
    for (int b = 0; b < B; b++) s->positions[b]++;
}

void region_retract(InferenceState* s)
{
    RegionState* st = state_of(s);
    for (int& a : st->absorbed) a--;
    for (int& p : st->parity) p ^= 1;
    for (int b = 0; b < s->batch_size; b++) s->positions[b]--;
}

int region_max_positions(const InferenceState* s) { return state_of(s)->max_seq; }

void region_prompt(InferenceState* s, const PromptPass& p, RegionPass pass)
{
    RegionState* st = state_of(s);
    const int region = st->per_seq ? p.seq : 0, vocab = s->model->config.n_vocab;
    const size_t V = (size_t)vocab;
    if (s->batch_size == 1 && p.n == 1) {                     // one token: the decode step
        region_forward(s, p.tokens, pass);
        if (p.n_want > 0)
            check_gpu(hipMemcpyAsync(p.logits, s->logits, V * sizeof(float), hipMemcpyDeviceToDevice, s->stream), "logits copy");
        return;
    }
    const int rows = p.rows > 0 ? std::min(p.rows, st->rows) : st->rows;
    float* last_row = s->logits + V * (st->per_seq ? p.seq : 0);
    int taken = 0;
    std::vector<int> picked;
    for (int done = 0; done < p.n;) {
        const int R = std::min(rows, p.n - done), pos = s->positions[p.seq];
        enter(st, region, pos);
        check_gpu(hipMemcpyAsync(s->d_tokens, p.tokens + done, R * sizeof(int), hipMemcpyHostToDevice, s->stream), "token copy");
        must(t12_rows_run(st->d_rows, pos, region * 2 + st->parity[region], R, s->stream), "row table");
        pass(s, R, 1, pos + R - 1, pass_logits(p, done, R, taken, vocab, last_row, picked));
        st->absorbed[region] += R;
        st->parity[region] ^= 1;
        if (st->per_seq) s->positions[p.seq] += R;
        else
            for (int b = 0; b < s->batch_size; b++) s->positions[b] += R;
        done += R;
    }
    for (int b = 1; !st->per_seq && p.n_want < 0 && b < s->batch_size; b++)
        check_gpu(hipMemcpyAsync(s->logits + V * b, last_row, V * sizeof(float), hipMemcpyDeviceToDevice, s->stream), "logits copy");
}

void region_linear(const CompressedWeight& w, float* out, int out_stride, const void* act, int K, int R, bool f32, hipStream_t q)
{
    T12Segment g = seg_of(w, out, out_stride);
    if (f32) must(t12_gemm_f32(&g, 1, (const float*)act, K, out_stride, K, R, 0, q), "32-bit linear");
    else run_linear(&g, 1, (const int16_t*)act, K, R, q);
}

void region_linear_add_f32(const CompressedWeight& w, float* cur, const void* act, int K, int R, hipStream_t q)
{
    T12Segment g = seg_of(w, cur, w.M);
    must(t12_gemm_f32(&g, 1, (const float*)act, K, w.M, K, R, 1, q), "32-bit linear");
}

bool region_fused_tensor(const CompressedWeight& w) { return exp_ok(w) && w.K % 16 == 0 && w.K <= 81920; }

bool region_no_fuse()
{
    const char* s = getenv("TURBO_NO_FUSE");
    return s && s[0] == '1';
}
