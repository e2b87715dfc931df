// Element-wise and per-row work between the products of a hybrid model's layers (rowops.hip), many tokens at a time, and
// the gated recurrence (recurrent.hip).  "act" outputs are rows of ld elements of `act` type whose columns from n on are
// written as zeros (linear.hpp: the activations of a product).
#pragma once

#include "linear.hpp"
#include "model_config.hpp"

namespace mesh {

// A norm over a row, with what is folded into it: RMS takes gain, LAYER gain and bias.
struct RowNorm {
    NormKind kind = NORM_NONE;
    const float *gain = nullptr, *bias = nullptr;
};

// x[t] = table[tok[t]] * scale, table rows of ldt, plus (freq set) the position vector of pos[t]: entries 2i and 2i + 1 are
// sin and cos of pos * freq[i]
int embed_rows(const uint16_t *table, int ldt, const int32_t *tok, const int32_t *pos, const float *freq, float scale, int T, int n, float *x, hipStream_t stream);

// x[t] += post(y[t]) (y null: x as it is), and act[t] = pre(x[t]): post RMS with pre NONE, or both LAYER
int residual_norm_rows(float *x, const float *y, const RowNorm &post, const RowNorm &pre, float eps, int T, int n, void *out, ActType act, int ld, hipStream_t stream);

// act[i] = layer norm of x[row[i]] for i < n_rows (row null: i)
int layer_norm_rows(const float *x, const int32_t *row, const RowNorm &norm, float eps, int n_rows, int n, void *out, ActType act, int ld, hipStream_t stream);

// act[i] = x[row[i]] / rms * gain[0] for i < n_rows (row null: i)
int scalar_norm_rows(const float *x, const int32_t *row, const float *gain, float eps, int n_rows, int n, void *out, ActType act, int ld, hipStream_t stream);

// act[t] = c0 N(u) + c1 N(u^2) + c2 N(u^3) + c3 with u = u[t][0..n), powers element by element, N(v) = v / rms(v)
int poly_norm_rows(const float *u, const float *coef, float eps, int T, int n, void *out, ActType act, int ld, hipStream_t stream);

// act[t][i] = gelu_tanh(g[t][i]) * side[tok[t]][offset + i]; g as the sum of `slices` partial products (linear_sliced)
int side_gate_rows(const float *g, int slices, size_t slice_stride, const uint16_t *side, const int32_t *tok, int stride, int offset, int T, int n, void *out, ActType act, int ld, hipStream_t stream);

// Norm over a whole q / k projection and KV append for attention whose values are the un-normalised keys.  qk: [T][(n_head +
// n_kv) * hd], q first; each head's entries from dim on are zero.  q[t] = q / rms(q over all heads) * q_norm; the cache
// gets k / rms(k) * k_norm as the key and k as the value, rows of hd of kv_type (f16 or f32).
struct QkAppendArgs {
    const float *qk = nullptr;
    float *q = nullptr;                // [T][n_head * hd]
    uint8_t *kcache = nullptr, *vcache = nullptr;       // this layer's, [n_seq][n_kv][n_ctx] rows
    int kv_type = MESH_F16;
    const float *q_norm = nullptr, *k_norm = nullptr;   // [n_head * hd], [n_kv * hd], zero where the head is padded
    const int32_t *pos = nullptr, *seq = nullptr;
    unsigned *sat = nullptr;           // counts values clamped to the f16 range
    float eps = 0.f;
    int n_head = 0, n_kv = 0, dim = 0, hd = 0, n_ctx = 0;
};
int qk_norm_append(const QkAppendArgs &a, int T, hipStream_t stream);

// Gated recurrence over the tokens of a call, in order within each sequence:
//   z = sigmoid(pz + bias_z), u = px + bias_x, c = u + 1/2 where u >= 0 and sigmoid(u) elsewhere,
//   S = (1 - z) S + z c,  act[t] = S * silu(pg)
// with (pz, px, pg) = zxg[t] (three rows of width).  A sequence's tokens are neighbours in the call and ascend; its state is
// read from `state` [n_seq][width] unless its first token is at position 0, and the last one is left there.  ws:
// min_gru_workspace(T, width) floats.
struct MinGruArgs {
    const float *zxg = nullptr;
    const float *bias_z = nullptr, *bias_x = nullptr;
    float *state = nullptr;
    const int32_t *pos = nullptr, *seq = nullptr;
    float *ws = nullptr;
    void *out = nullptr;
    ActType act = ACT_BF16;
    int ld = 0, width = 0;
};
size_t min_gru_workspace(int T, int width);
int min_gru(const MinGruArgs &a, int T, hipStream_t stream);

}  // namespace mesh
