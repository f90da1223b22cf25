// The Davasun family: a decoder with an RMS norm of one gain before and after every sublayer.  A layer's mixer is a matrix
// memory (mLSTM) or latent attention with a gate per head; some layers have a clamped gated feed-forward; a stretch of layers
// may be run several times in a row with the same weights, every run with a past of its own.  Every layer has its own sizes.
#pragma once
#include <string>
#include <vector>

#include "t12_abi.h"
#include "t12_mixers.h"
#include "turbo/model.h"

namespace davasun {

enum MixerKind { MLSTM, LATENT };

struct LayerConfig {
    MixerKind kind;
    int heads, dim, vdim;
    float gate_cap;                      // MLSTM
    int rot_dim, rank;                   // LATENT
    float rot_base, scale;
    int ff;                              // 0: no feed-forward
    float limit;

    // rows of the fused input projection.  MLSTM: q | k | v | g | i | f.  LATENT: q | c, rotated key part | g
    int k_off() const { return heads * dim; }
    int v_off() const { return 2 * heads * dim; }
    int m_g_off() const { return v_off() + heads * vdim; }
    int i_off() const { return m_g_off() + heads * vdim; }
    int f_off() const { return i_off() + heads; }
    int c_off() const { return heads * (dim + rot_dim); }
    int a_g_off() const { return c_off() + rank + rot_dim; }
    int in_rows() const { return kind == MLSTM ? f_off() + heads : a_g_off() + heads; }
    int in_ld() const { return (in_rows() + 3) / 4 * 4; }                  // floats between projected rows
    int out_cols() const { return heads * vdim; }
};

struct Config {
    int vocab = 0, width = 0;
    float eps = 0.0f, logit_scale = 1.0f;
    int loop_start = 0, loop_stop = 0, loop_times = 1;
    std::vector<LayerConfig> layers;
    std::string text;                    // config.json as read

    std::vector<int> runs() const;       // layers in the order they run
};

struct Layer {
    LayerConfig c;
    float *norm1, *norm1b;               // the gain, once per coordinate
    float *norm2, *norm2b;               // (null without a feed-forward)
    float gain1, gain1b, gain2, gain2b;  // the same gains, once
    CompressedWeight w_in;               // [in_rows, width]
    CompressedWeight w_out;              // [width, out_cols]
    float* in_bias;                      // MLSTM: [in_ld], gate biases, zeros elsewhere
    float* o_norm;                       // MLSTM: [out_cols]; LATENT: the latent's norm [rank]
    CompressedWeight k_up;               // LATENT: [heads*rank, dim], every head's key projection transposed
    CompressedWeight v_up;               // LATENT: [heads*vdim, rank]
    float* freqs;                        // LATENT: [rot_dim / 2]
    CompressedWeight gate, up, down;
};

struct Data {
    Config config;
    std::vector<Layer> layers;
    float* embed_norm = nullptr;         // [width]
    float final_gain = 1.0f;             // the final norm's, times the logit scale
};

Data* data_of(const Model* m);

}  // namespace davasun
