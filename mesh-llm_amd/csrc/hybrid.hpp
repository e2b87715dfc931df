// The runner of models whose layers are described one by one (model_config.hpp): attention and recurrent mixers over bf16
// weights, each layer with sizes of its own (hybrid_load.hip: weights; hybrid.hip: sessions and layers).  Shares the stage / session surface with the K-quant runner (stage.hpp).
#pragma once

#include <string>
#include <vector>

#include "gated_state.hpp"
#include "latent.hpp"
#include "linear.hpp"
#include "model_config.hpp"
#include "rowops.hpp"

struct mesh_stage;
struct mesh_session;

namespace mesh {

// Device-resident layer.  The projections that read the mixer's input are one stacked matrix `in`: q, k (attention); z, x, g
// (minGRU); latents of queries, of keys with the rotated part, gates (latent attention); q, k, v, g, then b, a (delta) or a1 (GLA).
// Attention heads are padded to head_pad entries, with zero rows in `in`, zero columns in `out` and zero norm weights.
struct HybridLayer {
    LayerSpec spec;
    int head_pad = 0;
    LinearWeight in, out, up, down, side_gate, side_proj;
    float *q_norm = nullptr, *k_norm = nullptr, *bias_z = nullptr, *bias_x = nullptr;
    float *coef = nullptr;                              // the activation's four numbers
    RowNorm pre1, pre2, post1, post2, post_side;        // post: the sublayer's output norm times its layer scale / residual factor
    // latent attention
    LatentShape latent;
    LinearWeight uq, ukv;                               // ukv: keys' rows, then values' (chunks of many tokens)
    uint16_t *w_uk_t = nullptr, *w_uv = nullptr;        // per head, for few tokens (latent.hpp)
    float *cq_norm = nullptr, *c_norm = nullptr;
    LatentRotary rot;
    int cache_layer = -1;                               // local index of the layer whose cache it reads (its own, or an earlier one's)
    // matrix states: weights and column offsets of a GatedStateArgs, completed per call
    GatedStateArgs gated;
    bool own_cache(int il) const { return cache_layer == il; }
};

struct HybridModel {
    ModelSpec spec;
    ActType act = ACT_BF16;
    std::vector<HybridLayer> layers;                    // of this stage
    uint16_t *embed = nullptr, *side_embed = nullptr;
    float *freq = nullptr, *final_gain = nullptr;       // position vectors; a final norm with one number
    RowNorm final_norm;                                 // or per element, times the logits' scale
    int embed_ld = 0;                                   // row length of `embed`
    LinearWeight head;
    bool has_state = false, has_chunks = false;         // some layer carries a state from token to token; some of these take tokens in chunks
    bool step_ok = true;                                // every product fits the single-token kernel
    int width_pad = 0, in_max = 0, act_max = 0, q_max = 0, state_max = 0;       // largest rows of the buffers below
    size_t qx_max = 0, part_max = 0, kvx_max = 0, kv16_max = 0, gated_ws_max = 0;   // bytes, floats, floats, f16 values per context position, floats per chunk
    bool side() const { return spec.side_dim > 0; }
};

// What the single-token step leaves to be added to the residual by whatever reads it next.
struct HybridPending {
    float *x = nullptr;
    const float *y = nullptr, *part = nullptr;
    RowNorm post;
    int n_part = 0;
};

struct HybridSession {
    void *xa = nullptr, *acta = nullptr;                // activations of the products: the residual stream, and a sublayer's inside
    float *big = nullptr, *y = nullptr, *q = nullptr, *ws = nullptr, *x2 = nullptr;
    float *part = nullptr;                              // two sets of STEP_PARTS_MAX x 3 partial sums
    std::vector<uint8_t *> k, v;                        // per local layer (attention; latent attention: k, its rows)
    std::vector<float *> state, tail;                   // per local layer (recurrence): [n_seq][width] or [n_seq][heads][dim][vdim]; convolution inputs
    void *qx = nullptr;                                 // latent attention: queries as its kernels take them
    float *kvx = nullptr, *gated_ws = nullptr;          // projected keys and values of some positions; what chunks leave for the scan
    uint16_t *kv16 = nullptr;                           // projected keys and values of one sequence
    int chunk_cap = 0;
    StateChunks chunks;                                 // of this call
    std::vector<int32_t> seq_len;                       // tokens each sequence holds; -1: a failed call left it undefined
    HybridPending tail_step;                               // of the last single-token step
};

int hybrid_open(const char *folder, int layer_begin, int layer_end, const mesh_stage_opts *opts, mesh_stage *st);
int hybrid_session_alloc(mesh_session *s);
// Positions of a call against what the sequences hold: tokens of a sequence are neighbours in the call and ascend by one;
// with a recurrent layer in the stage they start where the sequence stands, or at 0 (the sequence starts anew).
int hybrid_check_batch(const mesh_session *s, const mesh_batch *b);
void hybrid_note_batch(mesh_session *s, const mesh_batch *b, bool ok);
// Layers that read the token ids of the call.
bool hybrid_needs_ids(const mesh_stage *st);
// The tables of StateChunks for a call, into `table` (3 * n_batch_max + 2 entries; the device copy is at d_table); entries used,
// 0 if the call needs none.
size_t hybrid_chunk_table(mesh_session *s, const mesh_batch *b, int32_t *table, const int32_t *d_table);
bool hybrid_single_step(const mesh_session *s, int T);
uint64_t hybrid_graph_key(const mesh_session *s, int T, int max_keys);
int hybrid_embed(mesh_session *s, int T);
int hybrid_run_layers(mesh_session *s, int T, int max_keys);
// after the layers: the residual stream complete (returned in *x), or logits of n_rows rows (rows null: the first n_rows)
int hybrid_finish(mesh_session *s, int T, float **x);
int hybrid_logits(mesh_session *s, int T, const int32_t *d_rows, int n_rows, float *d_out);

}  // namespace mesh
