// Model families (engine-internal).  A family says which directories are its models, loads and saves them, and runs its
// layer stack; everything above -- sampling, the pipelined decode loop, generate, chat turns, the C face -- is shared.
#pragma once
#include <string>
#include <vector>

#include "turbo/inference.h"

// What every state carries for the shared decode loop; a family derives its own state from it (InferenceState::impl).
struct StateCommon {
    virtual ~StateCommon() = default;
    // pipelined greedy decoding: sampled tokens land in pinned host memory, two slots in rotation
    int* h_tokens[2] = {nullptr, nullptr};
    hipEvent_t sampled[2] = {nullptr, nullptr};
    // pipelined decoding: the second logits buffer (the forward enqueued ahead of the host's look at a token writes
    // there, so the logits that produced an end-of-stream token are still in place when the loop stops)
    float* logits_alt = nullptr;
    bool no_pipeline = false;      // read once, when the state is created
    float* picked = nullptr;       // logits of picked places on their way to the host (C face), grown on demand
    size_t picked_floats = 0;
};

// A stretch of one sequence's tokens that enters at state->positions[seq].
struct PromptPass {
    int seq = 0;
    const int* tokens = nullptr;   // host
    int n = 0;
    int rows = 0;                  // tokens per pass of the layer stack; 0: what the state was made for
    // n_want < 0: the last token's logits go into the sequence's row of state->logits.  Otherwise the logits of the
    // tokens want[0..n_want) (places in `tokens`, ascending) go to logits, fp32 [n_want, n_vocab] on the device.
    const int* want = nullptr;
    int n_want = -1;
    float* logits = nullptr;
};

// Which rows of a pass of the layer stack get logits: all of them (into state->logits), the last one, the listed ones
// (ascending), or none.
enum LogitsMode { LOGITS_ALL, LOGITS_LAST_ROW, LOGITS_ROWS, LOGITS_NONE };
struct LogitsRequest {
    LogitsMode mode = LOGITS_NONE;
    float* out = nullptr;                // LOGITS_LAST_ROW, LOGITS_ROWS: [rows, n_vocab]
    const int* rows = nullptr;
    int n_rows = 0;
};
// The request of the pass that runs tokens done .. done + R - 1 of p; `taken` counts the wanted places already served,
// `rows` backs the request's list, last_row receives the last token's logits when none are picked.
LogitsRequest pass_logits(const PromptPass& p, int done, int R, int& taken, int n_vocab, float* last_row, std::vector<int>& rows);

struct FamilyRun {
    InferenceState* (*create)(Model*, const StateOptions&);       // nullptr: the caches do not fit, or the precision is not offered
    void (*release)(InferenceState*);                             // the family's own buffers; the shared ones follow
    int (*max_positions)(const InferenceState*);
    void (*forward)(InferenceState*, const int* token_ids);
    void (*prompt)(InferenceState*, const PromptPass&);
    void (*retract)(InferenceState*);                             // takes the last forward back (one step at most)
    void (*shift)(InferenceState*, int seq, int current_pos, int discard);   // null: a context cannot be shifted
};

struct ModelFamily {
    const char* name;
    bool (*owns)(const std::string& dir);                         // is the directory one of its models?
    bool (*check)(const std::string& dir, std::string& err);      // host only; what load_model starts with
    Model* (*load)(const std::string& dir);
    bool (*save)(const Model*, const std::string& dir);
    void (*release)(Model*);
    const FamilyRun* run;
};

// (not const: hipcc would make constant-initialised host tables part of the device code as well)
extern ModelFamily kLlamaFamily, kGamilornFamily, kDavasunFamily;
extern FamilyRun kLlamaRun, kGamilornRun, kDavasunRun;

const ModelFamily& family_of(const Model* m);

// ---- shared by the families' layer stacks (inference.cpp) ------------------------------------------------------
struct T12Segment;
void check_gpu(hipError_t e, const char* what);                   // throws EngineError
void must(int rc, const char* what);                              // the same for a library call's return code
T12Segment seg_of(const CompressedWeight& w, float* out, int out_stride);
void run_linear(const T12Segment* segs, int nseg, const int16_t* act, int K, int B, hipStream_t st);
void run_linear_add_norm(const T12Segment* seg, const int16_t* act, int K, int B, const float* residual, const float* norm_w,
                         float eps, int16_t* y, hipStream_t st);
bool exp_ok(const CompressedWeight& w);                           // the fused B = 1 kernels take this tensor
// A state with its streams, ids, positions and logits (batch_size rows); impl is adopted.
InferenceState* new_state(Model* model, int batch_size, int rows, StateCommon* impl);
