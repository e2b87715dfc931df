// The runner of models whose layers are described one by one (model_config.hpp): attention and recurrent mixers over bf16
// weights, each layer with sizes of its own.  Shares the stage / session surface with the K-quant runner (stage.hpp).
#pragma once

#include <string>
#include <vector>

#include "linear.hpp"
#include "model_config.hpp"
#include "rowops.hpp"

struct mesh_stage;
struct mesh_session;

namespace mesh {

// Device-resident layer.  q and k (or the recurrence's z, x, g) are one stacked matrix `in`; attention heads are padded to
// head_pad entries, with zero rows in `in`, zero columns in `out` and zero norm weights.
struct HybridLayer {
    LayerSpec spec;
    int head_pad = 0;
    LinearWeight in, out, up, down, side_gate, side_proj;
    float *q_norm = nullptr, *k_norm = nullptr, *bias_z = nullptr, *bias_x = nullptr;
    float *coef = nullptr;                              // the activation's four numbers
    float *gain1 = nullptr, *gain2 = nullptr, *gain_side = nullptr;   // per element: the sublayer's output norm times its layer scale
};

struct HybridModel {
    ModelSpec spec;
    ActType act = ACT_BF16;
    std::vector<HybridLayer> layers;                    // of this stage
    uint16_t *embed = nullptr, *side = nullptr;
    float *freq = nullptr, *final_gain = nullptr;
    LinearWeight head;
    bool has_state = false;                             // some layer carries a state from token to token
    bool step_ok = true;                                // every product fits the single-token kernel
    int width_pad = 0, in_max = 0, act_max = 0, q_max = 0, state_max = 0;       // largest rows of the buffers below
};

// What the single-token step leaves to be added to the residual by whatever reads it next.
struct HybridPending {
    float *x = nullptr;
    const float *y = nullptr, *gain = nullptr, *part = nullptr;
    int n_part = 0;
};

struct HybridSession {
    void *xa = nullptr, *acta = nullptr;                // activations of the products: the residual stream, and a sublayer's inside
    float *big = nullptr, *y = nullptr, *q = nullptr, *ws = nullptr, *x2 = nullptr;
    float *part = nullptr;                              // two sets of STEP_PARTS_MAX x 3 partial sums
    std::vector<uint8_t *> k, v;                        // per local layer (attention)
    std::vector<float *> state;                         // per local layer (recurrence): [n_seq][width]
    std::vector<int32_t> seq_len;                       // tokens each sequence holds; -1: a failed call left it undefined
    HybridPending tail;                                 // of the last single-token step
};

int hybrid_open(const char *folder, int layer_begin, int layer_end, const mesh_stage_opts *opts, mesh_stage *st);
int hybrid_session_alloc(mesh_session *s);
// Positions of a call against what the sequences hold: tokens of a sequence are neighbours in the call and ascend by one;
// with a recurrent layer in the stage they start where the sequence stands, or at 0 (the sequence starts anew).
int hybrid_check_batch(const mesh_session *s, const mesh_batch *b);
void hybrid_note_batch(mesh_session *s, const mesh_batch *b, bool ok);
bool hybrid_single_step(const mesh_session *s, int T);
uint64_t hybrid_graph_key(const mesh_session *s, int T, int max_keys);
int hybrid_embed(mesh_session *s, int T);
int hybrid_run_layers(mesh_session *s, int T, int max_keys);
// after the layers: the residual stream complete (returned in *x), or logits of n_rows rows (rows null: the first n_rows)
int hybrid_finish(mesh_session *s, int T, float **x);
int hybrid_logits(mesh_session *s, int T, const int32_t *d_rows, int n_rows, float *d_out);

}  // namespace mesh
