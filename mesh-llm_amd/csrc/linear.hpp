// Products with bf16 weight matrices: many tokens (linear.hip) and the single-token step with its fused ends
// (linear_step.hip).
#pragma once

#include "mesh_common.hpp"

namespace mesh {

// What the activations of a product are stored as, and with it the arithmetic: bf16 rows on the bf16 matrix cores with
// f32 sums, or f32 rows on the f32 matrix cores (weights widened exactly): every product and sum in 32 bits.
enum ActType { ACT_BF16 = 0, ACT_F32 = 1 };
inline size_t act_bytes(ActType a) { return a == ACT_BF16 ? 2 : 4; }

// A [M][K] matrix as bf16 rows of Kp elements, Mp rows; the padding holds zeros.
constexpr int LINEAR_ROW_PAD = 128, LINEAR_K_PAD = 64;
struct LinearWeight {
    const uint16_t *w = nullptr;
    int M = 0, K = 0, Mp = 0, Kp = 0;
    bool present() const { return w != nullptr; }
};
inline int linear_rows_padded(int M) { return (M + LINEAR_ROW_PAD - 1) / LINEAR_ROW_PAD * LINEAR_ROW_PAD; }
inline int linear_k_padded(int K) { return (K + LINEAR_K_PAD - 1) / LINEAR_K_PAD * LINEAR_K_PAD; }

// y[t][m] = sum_k W[m][k] x[t][k] for t < T.  x: rows of W.Kp elements of `act` (columns from K on hold zeros), 16-byte
// aligned; y: f32 rows of ldy.  big_from: bf16 calls of at least this many tokens take the large-tile kernel.
int linear(const LinearWeight &W, const void *x, ActType act, int T, float *y, int ldy, int big_from, hipStream_t stream);
// The same, leaving max(y, 0)^2 as rows of ld elements of `act` (W.M <= ld <= W.Mp; columns from W.M on are zeros) for the
// product that follows.
int linear_relu2(const LinearWeight &W, const void *x, ActType act, int T, void *out, int ld, int big_from, hipStream_t stream);

// The same for a matrix of few rows (hundreds), which leaves the large tile with few workgroups: K is cut into slices, each of
// which writes its own partial y, `stride` floats apart; the reader adds them in order.  Returns the slice count (1: y is
// the product) or a negative status.  y holds at least LINEAR_SLICES_MAX * T * W.M floats.
constexpr int LINEAR_SLICES_MAX = 8;
int linear_sliced(const LinearWeight &W, const void *x, ActType act, int T, float *y, size_t stride, int big_from, hipStream_t stream);

// ---- one token ------------------------------------------------------------------------------------------------
// A mat-vec whose workgroups derive the input vector themselves from what the launch before them left, and whose epilogue
// does the element-wise work that follows.  Activations are f32 throughout, so the results serve both ActTypes.
enum StepIn {
    STEP_IN_VEC = 0,          // x = in
    STEP_IN_RESIDUAL = 1,     // x = in + y / rms(y) * gain, rms from the partial sums its producer left; also written to x_out
    STEP_IN_RESIDUAL_NORM = 2,// the same, then x / rms(x) * norm_gain
    STEP_IN_POLY = 3,         // x = c0 N(u) + c1 N(u^2) + c2 N(u^3) + c3, u = in, N(v) = v / rms(v)
    STEP_IN_LAYER = 4,        // v = in + LN(y) gain + bias (y null: v = in), also written to x_out; x = LN(v) norm_gain + norm_bias, LN(v) = (v - mean) / deviation
    STEP_IN_UNIT_RMS = 5,     // x = in / rms(in) * gain
    STEP_IN_RELU2 = 6         // x = max(in, 0)^2
};
enum StepOut {
    STEP_OUT_PLAIN = 0,       // out = W x
    STEP_OUT_SUMSQ = 1,       // and the sum of squares of the workgroup's rows (for STEP_IN_RESIDUAL)
    STEP_OUT_POWERS = 2,      // and the sums of squares of u, u^2, u^3 (for STEP_IN_POLY)
    STEP_OUT_MIN_GRU = 3,     // W = three stacked matrices z, x, g of `width` rows: the state's update, out = state * silu(g)
    STEP_OUT_SIDE = 4         // out = gelu_tanh(W x) * side embedding of the token
};
constexpr int STEP_PARTS_MAX = 512;
struct StepArgs {
    LinearWeight W;
    StepIn in_kind = STEP_IN_VEC;
    StepOut out_kind = STEP_OUT_PLAIN;
    const float *in = nullptr;            // [K]
    const float *y = nullptr;             // RESIDUAL, LAYER: [K]
    const float *gain = nullptr;          // RESIDUAL, LAYER with y, UNIT_RMS: [K]
    const float *bias = nullptr;          // LAYER with y: [K]
    const float *part = nullptr;          // RESIDUAL: [n_part]; POLY: [3][n_part]
    int n_part = 0;
    float *x_out = nullptr;               // RESIDUAL, LAYER with y: [K], not `in`
    const float *norm_gain = nullptr;     // RESIDUAL_NORM: one number; LAYER: [K]
    const float *norm_bias = nullptr;     // LAYER: [K]
    const float *coef = nullptr;          // POLY: four numbers
    float eps = 0.f;
    float *out = nullptr;                 // [M] (MIN_GRU: [width])
    float *out_part = nullptr;            // SUMSQ: [grid]; POWERS: [3][grid]
    // MIN_GRU
    int width = 0;
    const float *bias_z = nullptr, *bias_x = nullptr;
    float *state = nullptr;               // [n_seq][width]
    const int32_t *pos = nullptr, *seq = nullptr;    // device, one entry; position 0 starts from a zero state
    // SIDE
    const uint16_t *side = nullptr;       // bf16 [vocab][side_stride], this layer's part at side_offset
    int side_stride = 0, side_offset = 0;
    const int32_t *tok = nullptr;         // device, one entry
};
bool linear_step_supported(const LinearWeight &W);
// grid of the launch = partial sums it writes
int linear_step_grid(const StepArgs &a);
int linear_step(const StepArgs &a, hipStream_t stream);

}  // namespace mesh
