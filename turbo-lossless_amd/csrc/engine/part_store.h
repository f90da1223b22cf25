// Models whose tensors are a list of named parts (engine-internal): one walk over the list serves checking, loading,
// saving, filling and freeing.
//
// Two directory forms, both with the model's config.json:
//   * a checkpoint, config.json + model.safetensors: the family fuses and packs the tensors while they are loaded;
//   * what save_model writes: the packed tensors as the seven files every split-12 tensor of this build has, fp32 vectors
//     as <name>.f32.bin, bf16 tables as <name>.bf16.bin.
#pragma once
#include <functional>
#include <string>
#include <vector>

#include "checkpoint.h"
#include "model_store.h"

namespace part_store {

struct Parts {
    // fused or single matrix [M, K]
    std::function<void(const std::string&, CompressedWeight&, int M, int K)> weight;
    std::function<void(const std::string&, float*&, size_t n)> vector;
    std::function<void(const std::string&, int16_t*&, size_t n)> table;
};
typedef std::function<void(const Parts&)> Walk;

std::string layer_name(size_t i, const char* what);               // l<i>.<what>
bool ends_with(const std::string& s, const char* end);

// ---- directories
bool read_config_text(const std::string& dir, std::string& text); // config.json
bool has_architecture(const std::string& dir, const char* name);  // config.json names it
bool is_checkpoint(const std::string& dir);
std::string vector_file(const std::string& dir, const std::string& name);
std::string table_file(const std::string& dir, const std::string& name);

// ---- the packed form
bool check_packed(const std::string& dir, const Walk& walk, std::string& err);   // host only
bool load_packed(const std::string& dir, const Walk& walk);
bool save_packed(const std::string& dir, const std::string& config_text, const Walk& walk);

// ---- checkpoints
float bf16_value(const uint8_t* p);
// A tensor as fp32 values, `add` added to each.
std::vector<float> values(const Checkpoint& ck, const std::string& name, float add = 0.0f);
// Matrices stacked below each other (equal K), or side by side along K (equal M), as bf16 bytes.
std::vector<uint8_t> below(const Checkpoint& ck, const std::vector<std::string>& names);
std::vector<uint8_t> beside(const Checkpoint& ck, const std::vector<std::string>& names, int M);
// bf16 bytes [M, K] -> a split-12 tensor packed on the GPU
void pack(const std::string& name, const std::vector<uint8_t>& bits, int M, int K, CompressedWeight& w);

// ---- on the device
void release(const Walk& walk);
// Matrices N(0, 0.02) with outliers N(0, 8) at rate p_outlier, tables N(0, 0.02), vectors filled with fill(name).
void synthesize(const Walk& walk, uint64_t seed, float p_outlier, const std::function<float(const std::string&)>& fill);

}  // namespace part_store
