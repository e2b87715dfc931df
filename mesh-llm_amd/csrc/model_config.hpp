// A model described layer by layer, as read from the config.json of a model folder.
#pragma once

#include <cstdint>
#include <string>
#include <vector>

namespace mesh {

enum MixerKind {
    MIXER_ATTENTION = 0,     // grouped-query attention over a window of keys; the values are the projected keys
    MIXER_MIN_GRU = 1,       // gated recurrence whose gates read the current token only
    MIXER_LATENT = 2,        // attention whose keys and values are projections of one cached latent per token
    MIXER_DELTA = 3,         // matrix state per head, corrected towards each token's value (gated delta rule)
    MIXER_GLA = 4            // matrix state per head, decayed per key channel (gated linear attention)
};

// Angles of rotary positions: pair i of `dims` entries turns by position * freq(i).
struct RotarySpec {
    int dims = 0;
    double base = 0.0;
    bool scaled = false;     // frequencies blended between f and f / factor by how often a pair turns over `original` tokens
    double factor = 1.0, original = 0.0, fast = 0.0, slow = 0.0;

    double freq(int pair) const;
    float gain() const;      // of cosine and sine
    bool operator==(const RotarySpec &o) const {
        return dims == o.dims && base == o.base && scaled == o.scaled && factor == o.factor && original == o.original && fast == o.fast && slow == o.slow;
    }
};

struct MixerSpec {
    MixerKind kind = MIXER_ATTENTION;
    // every kind with heads; dim: of queries and keys (latent: their unrotated part), vdim: of values
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    // attention
    int window = 0;          // a token sees itself and window - 1 tokens before it; 0: every earlier token
    float scale = 1.f;       // of the scores
    // latent attention
    int q_rank = 0, kv_rank = 0, rot_dim = 0;
    int kv_from = -1;        // reads the cache of this earlier layer instead of having one
    RotarySpec rot;
    // recurrence
    int width = 0;           // minGRU
    int taps = 0;            // delta: of the short convolutions
    float tau = 1.f;         // GLA: decay = sigmoid(.)^(1 / tau)

    bool has_matrix_state() const { return kind == MIXER_DELTA || kind == MIXER_GLA; }
    bool has_state() const { return kind == MIXER_MIN_GRU || has_matrix_state(); }
};

struct LayerSpec {
    MixerSpec mixer;
    int ff = 0;              // rows of the feed-forward; 0: the layer has none
};

enum NormKind { NORM_NONE = 0, NORM_RMS = 1, NORM_LAYER = 2 };         // x / rms(x) * gain | (x - mean) / deviation * gain + bias
enum FfKind { FF_POLY_NORM = 0, FF_RELU2 = 1 };

struct ModelSpec {
    std::string arch;
    int vocab = 0, width = 0;
    int side_dim = 0;        // width of a layer's part of the per-token side embedding; 0: the layers do not read the token ids
    float eps = 0.f, embed_scale = 1.f;
    bool sinusoid = false;   // a position vector is added to the embedding
    NormKind in_norm = NORM_NONE, out_norm = NORM_RMS;       // before and after every sublayer
    FfKind ff = FF_POLY_NORM;
    float residual_mult = 1.f, logit_scale = 1.f;
    bool tied_head = false;  // logits from the embedding table
    std::vector<LayerSpec> layers;
};

bool is_model_folder(const char *path);
// <folder>/config.json -> spec; MESH_OK or a negative mesh_status with the message set.  Every size is checked for sanity,
// so that the products of two of them fit 32 bits.
int model_spec_from_folder(const char *folder, ModelSpec &out);

}  // namespace mesh
