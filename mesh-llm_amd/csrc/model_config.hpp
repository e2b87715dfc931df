// A model described layer by layer, as read from the config.json of a model folder.
#pragma once

#include <cstdint>
#include <string>
#include <vector>

namespace mesh {

enum MixerKind {
    MIXER_ATTENTION = 0,     // grouped-query attention over a window of keys; the values are the projected keys
    MIXER_MIN_GRU = 1        // gated recurrence whose gates read the current token only
};

struct MixerSpec {
    MixerKind kind = MIXER_ATTENTION;
    // attention
    int heads = 0, kv_heads = 0, dim = 0;
    int window = 0;          // a token sees itself and window - 1 tokens before it; 0: every earlier token
    float scale = 1.f;       // of the scores
    // recurrence
    int width = 0;
};

struct LayerSpec {
    MixerSpec mixer;
    int ff = 0;              // rows of the feed-forward; 0: the layer has none
};

struct ModelSpec {
    std::string arch;
    int vocab = 0, width = 0;
    int side_dim = 0;        // width of a layer's part of the per-token side embedding
    float eps = 0.f, embed_scale = 1.f;
    std::vector<LayerSpec> layers;
};

bool is_model_folder(const char *path);
// <folder>/config.json -> spec; MESH_OK or a negative mesh_status with the message set.  Every size is checked for sanity,
// so that the products of two of them fit 32 bits.
int model_spec_from_folder(const char *folder, ModelSpec &out);

}  // namespace mesh
