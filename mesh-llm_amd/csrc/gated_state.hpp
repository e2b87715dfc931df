// Recurrences whose state is a matrix S [dim][vdim] per head (gated_state.hip), f32 throughout.  With queries q, keys k, values
// v and a decay between 0 and 1:
//   GLA     S <- diag(alpha) S + k v^T                      decay per key channel, alpha = sigmoid(z)^(1 / tau), z = W_a2 a1 + b
//   DELTA   S <- g S;  u = beta (v - S^T k);  S <- S + k u^T   decay per head, g = exp(-A softplus(a + dt)); q, k, v through a short
//           causal convolution and silu, q and k then as unit vectors; query heads share q / k heads in groups
// and the read-out o = S^T q, with q scaled by dim^(-1/2), after the token's write.  The layer's output is
// o / rms(o over vdim) * norm * silu(g_out).
//
// One token per sequence: one launch.  More: chunks of up to 32 tokens of a sequence.  Within a chunk the recurrence is a
// triangular system; solved for all chunks at once it leaves per chunk the matrices with which
//   u = U - W S,  o = Q S + A u,  S <- G S + K^T u
// carries the state over the whole chunk (GLA: W = 0, U = v), so that only these products run one chunk after the other
// (Yang et al., Parallelizing Linear Transformers with the Delta Rule over Sequence Length).
#pragma once

#include "linear.hpp"

namespace mesh {

constexpr int STATE_CHUNK = 32;
constexpr int STATE_DIM_MAX = 256;          // of dim and of vdim
constexpr int STATE_RANK_MAX = 256;         // of GLA's decay projection

// The calls' tokens by sequence: chunk i is tokens [chunk[i], chunk[i + 1]), all of one sequence, whose run of tokens begins
// at first[i]; sequence j of the call has chunks [run[j], run[j + 1]).  Device arrays.
struct StateChunks {
    const int32_t *chunk = nullptr, *first = nullptr, *run = nullptr;
    int n_chunks = 0, n_runs = 0;
};

struct GatedStateArgs {
    bool delta = false;                     // else GLA
    int heads = 0, kv_heads = 0, dim = 0, vdim = 0;
    const float *in = nullptr;              // [T][ld] projections; the columns each starts at:
    int ld = 0, at_q = 0, at_k = 0, at_v = 0, at_g = 0, at_a = 0, at_b = 0;      // GLA: at_a is a1 (rank columns); DELTA: a and b, one per head
    // GLA
    int rank = 0;
    const float *a2 = nullptr, *a2_bias = nullptr;      // [heads * dim][rank], [heads * dim]
    float inv_tau = 1.f;
    // DELTA
    int taps = 0;
    const float *conv_q = nullptr, *conv_k = nullptr, *conv_v = nullptr;       // [channels][taps], the last the current token's
    const float *A = nullptr, *dt_bias = nullptr;       // [heads]; A = exp(A_log)
    float *tail = nullptr;                  // [n_seq][taps][channels of q, k, v]: the convolutions' inputs by position modulo taps
    const float *norm = nullptr;            // [vdim]
    float eps = 0.f;
    float *state = nullptr;                 // [n_seq][heads][dim][vdim]
    const int32_t *pos = nullptr, *seq = nullptr;       // device; a sequence at position 0 starts from zero
    StateChunks chunks;
    float *ws = nullptr;                    // gated_state_workspace floats
    float *o = nullptr;                     // [T][heads * vdim]
    // output rows of ld_out, zeros behind heads * vdim: f32 or bf16
    void *out = nullptr;
    ActType act = ACT_BF16;
    int ld_out = 0;
};
inline bool gated_state_supported(int dim, int vdim) { return dim <= STATE_DIM_MAX && vdim <= STATE_DIM_MAX; }
inline int gated_state_channels(const GatedStateArgs &a) { return 2 * a.kv_heads * a.dim + a.heads * a.vdim; }
size_t gated_state_workspace(int n_chunks, int heads, int dim, int vdim);
// every token its own sequence
int gated_state_step(const GatedStateArgs &a, int T, hipStream_t stream);
// any call
int gated_state_chunks(const GatedStateArgs &a, int T, hipStream_t stream);

}  // namespace mesh
