// States of families whose layers hold a past that only goes forward (engine-internal): sequence regions with a pair of
// recurrent states each, and the passes of rows over them.
//
// A pass works on rows: one token of every sequence (decode), or consecutive tokens of one sequence (prompt).  The
// recurrent states of a region are read from one of the pair and written to the other, so the newest step can be taken
// back by turning the pair around (the pipelined decode loop runs one step past an end-of-stream token).
#pragma once
#include <vector>

#include "family.h"
#include "t12_abi.h"
#include "t12_mixers.h"

struct RegionState : StateCommon {
    bool f32 = false;
    bool per_seq = false;                        // false: all rows of the batch share region 0 (lock-step copies)
    int rows = 0;                                // rows a pass can carry
    int max_seq = 0;
    std::vector<int> absorbed;                   // per region: tokens its recurrent states have seen
    std::vector<int> parity;                     // per region: which of the pair is current
    std::vector<void*> owned;                    // device buffers that go with the state
    T12Row* d_rows = nullptr;

    int regions() const { return (int)absorbed.size(); }
    void* own(size_t bytes);
    void* own_zeroed(size_t bytes, hipStream_t st);
    // Precision, kind and sizes the options ask for, and the empty regions.
    void shape(const StateOptions& o, int context, int default_rows);
};

// R rows whose tokens are in s->d_tokens and whose row table is in d_rows; run: consecutive tokens of one sequence; no row
// stands beyond max_position.
typedef void (*RegionPass)(InferenceState* s, int R, int run, int max_position, const LogitsRequest& lr);

// The shared halves of FamilyRun::forward, prompt, retract and max_positions.
void region_forward(InferenceState* s, const int* token_ids, RegionPass pass);
void region_prompt(InferenceState* s, const PromptPass& p, RegionPass pass);
void region_retract(InferenceState* s);
int region_max_positions(const InferenceState* s);

// out[r, :] = w . act[r, :] in the state's precision (act fp32 or bf16).
void region_linear(const CompressedWeight& w, float* out, int out_stride, const void* act, int K, int R, bool f32, hipStream_t q);
// cur += w . act in 32 bits, which ends a block of a 32-bit state.
void region_linear_add_f32(const CompressedWeight& w, float* cur, const void* act, int K, int R, hipStream_t q);
// Every tensor can take the decode-GEMV with fused prologues and epilogues (K of a norm prologue: region_norm_width).
bool region_fused_tensor(const CompressedWeight& w);
inline bool region_norm_width(int K) { return K % 16 == 0 && K <= 8192; }
// The debugging switch that turns the fused decode paths off.
bool region_no_fuse();
