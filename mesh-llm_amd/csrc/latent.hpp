// Attention over latents (latent.hip): per token the cache holds one row [latent, rotated key part] that all heads share;
// a head's unrotated key and its value are projections of the latent.
//
// Few tokens per call: the key projection is moved to the query side (q . W_uk c = W_uk^T q . c) and the value projection
// behind the softmax, so that the cache rows themselves are keys and values and are read once for all heads.  Many tokens
// of one sequence: keys and values are projected once and the chunk kernel of attn.hpp runs over them.
#pragma once

#include "linear.hpp"

namespace mesh {

// Sizes of a layer.  Cache rows are rank_pad + rot_pad elements: the latent, zeros, the rotated part, zeros; f16, or f32 in
// 32-bit stages.
struct LatentShape {
    int heads = 0, dim = 0, rot_dim = 0, vdim = 0, rank = 0;
    int rank_pad = 0, rot_pad = 0, dim_pad = 0;       // dim_pad: row length of w_uk_t
    int chunk_k = 0, chunk_v = 0;                     // row lengths of projected keys and values for the chunk kernel (0: it has none for them)
    int v_pad = 0;                                    // entries of a head in the output
    __host__ __device__ int row() const { return rank_pad + rot_pad; }
};
// fills the padded sizes; false if the kernels have none large enough
bool latent_shape(LatentShape &s);
constexpr int LATENT_HEADS_TILE = 16;                 // heads a workgroup of the attention kernel takes
inline int latent_head_tiles(const LatentShape &s) { return (s.heads + LATENT_HEADS_TILE - 1) / LATENT_HEADS_TILE; }

struct LatentRotary {
    const double *freq = nullptr;                     // device, [rot_dim / 2]
    float gain = 1.f;
};

// Where the rows of a layer are, [n_seq][n_ctx], and whose projections fill them (in null: another layer's)
struct LatentCache {
    void *rows = nullptr;
    int n_ctx = 0;
    const float *in = nullptr;                        // [T][ld], the projection's kv_rank + rot_dim columns
    int ld = 0;
    const float *gain = nullptr;                      // [rank]
    LatentRotary rot;
    const int32_t *pos = nullptr, *seq = nullptr;     // device, [T]
    unsigned *sat = nullptr;
    float eps = 0.f;
};

// act[t] = in[t][0 .. n) / rms * gain, rows of ld_out; and the cache rows of the call's tokens (cache.in set)
int latent_rows(const LatentShape &s, const LatentCache &cache, ActType act, const float *in, int ld, const float *gain, int n, void *out, int ld_out, int T, hipStream_t stream);

// Queries against cache rows: qa[t][h] = (W_uk^T q, rotated part) * scale in log2 units, rows of s.row() elements of the
// cache's type.  q: [T][heads * (dim + rot_dim)].  append: one more workgroup per token writes the cache rows.
int latent_query(const LatentShape &s, const LatentCache &cache, ActType act, const float *q, const uint16_t *w_uk_t, float scale, bool append, void *qa, int T, hipStream_t stream);

struct LatentAttnArgs {
    const void *qa = nullptr, *rows = nullptr;
    const int32_t *pos = nullptr, *seq = nullptr;
    float *part = nullptr;             // [T][heads][n_splits][rank_pad]
    float *ml = nullptr;               // [T][heads][n_splits][2]: maximum (log2 units) and sum
    int n_ctx = 0, n_splits = 1;
    int group = 1;                     // tokens a workgroup takes: 1, or LATENT_GROUP where the call is one run of positions of a sequence
    // latent_out
    const uint16_t *w_uv = nullptr;    // [heads][vdim][rank_pad]
    const float *gate = nullptr;       // [T][gate_ld], one per head, through a sigmoid
    int gate_ld = 0;
    float *out = nullptr;              // [T][heads * v_pad], or
    uint16_t *out_bf16 = nullptr;
};
constexpr int LATENT_GROUP = 4;
int latent_group(const LatentShape &s, int T, bool one_run);
// key splits of a launch that aims at `target` workgroups (0: one per compute unit); splits * T is at most LATENT_GROUP * target or T
int latent_splits(const LatentShape &s, int T, int group, int max_keys, int target);
// token t over positions [0, pos[t]] of sequence seq[t]: partial sums of latents per key split
int latent_attention(const LatentShape &s, const LatentAttnArgs &a, ActType act, int T, hipStream_t stream);
// splits merged, projected to values, times the head's gate
int latent_out(const LatentShape &s, const LatentAttnArgs &a, int T, hipStream_t stream);

// ---- many tokens of one sequence
// q [T][heads * (dim + rot_dim)] -> [T][heads][chunk_k], the second part rotated, zeros behind
int latent_chunk_query(const LatentShape &s, const LatentRotary &rot, const float *q, const int32_t *pos, float *out, int T, hipStream_t stream);
// latents of positions [k0, k0 + n) of sequence seq as bf16 rows of ld
int latent_chunk_rows(const LatentShape &s, const void *rows, int n_ctx, int seq, int k0, int n, uint16_t *out, int ld, hipStream_t stream);
// their projections kv [n][heads * (dim + vdim)] (all keys, then all values) and rotated parts -> f16 rows [heads][n_ctx][chunk_k] and [heads][n_ctx][chunk_v]
int latent_chunk_pack(const LatentShape &s, const void *rows, int n_ctx, int seq, int k0, int n, const float *kv, uint16_t *k16, uint16_t *v16, unsigned *sat, hipStream_t stream);

}  // namespace mesh
