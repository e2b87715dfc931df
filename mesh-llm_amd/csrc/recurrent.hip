// Gated recurrence over many tokens: a linear recurrence S = a S + b per channel, cut into windows of tokens.
//
// One thread owns one channel of one window.  The first launch composes each window's steps into (A, B), S_out = A S_in + B,
// or, when a sequence starts inside the window, into the state its last sequence leaves (A = 0).  The second walks the
// windows again, each starting from the composition of the windows before it, and writes the outputs.  Both read the
// projections coalesced along the channels.  A call of one window (decode batches) needs the second launch only.
//
// A sequence's starting state is read in the first launch where the sequence goes on into later windows: those may write
// its final state while this window still runs.
#include "act_math.hpp"
#include "rowops.hpp"

namespace mesh {

constexpr int GRU_WINDOW = 32, GRU_THREADS = 256;

__global__ __launch_bounds__(GRU_THREADS) void min_gru_compose_kernel(const MinGruArgs a, int T) {
    const int ch = blockIdx.x * GRU_THREADS + threadIdx.x, w = blockIdx.y, W = a.width;
    if (ch >= W) return;
    const int t0 = w * GRU_WINDOW, t1 = t0 + GRU_WINDOW < T ? t0 + GRU_WINDOW : T;
    const float bz = a.bias_z[ch], bx = a.bias_x[ch];
    float A = 1.f, B = 0.f, init = 0.f;
#pragma unroll 8
    for (int t = t0; t < t1; ++t) {
        if (t == 0 || a.seq[t] != a.seq[t - 1]) {
            A = 0.f;
            B = init = a.pos[t] == 0 ? 0.f : a.state[(size_t)a.seq[t] * W + ch];
        }
        const float *p = a.zxg + (size_t)t * 3 * W + ch;
        const MinGruGate g = min_gru_gate(p[0] + bz, p[W] + bx);
        A *= g.keep;
        B = fmaf(g.keep, B, g.in);
    }
    float *ws = a.ws + (size_t)w * 3 * W + ch;
    ws[0] = A; ws[W] = B; ws[2 * W] = init;
}

template <ActType ACT>
__global__ __launch_bounds__(GRU_THREADS) void min_gru_kernel(const MinGruArgs a, int T) {
    const int ch = blockIdx.x * GRU_THREADS + threadIdx.x, w = blockIdx.y, W = a.width;
    if (ch >= a.ld) return;
    const int t0 = w * GRU_WINDOW, t1 = t0 + GRU_WINDOW < T ? t0 + GRU_WINDOW : T;
    auto put = [&](int t, float v) {
        if constexpr (ACT == ACT_BF16) static_cast<uint16_t *>(a.out)[(size_t)t * a.ld + ch] = f32_to_bf16_bits(v);
        else static_cast<float *>(a.out)[(size_t)t * a.ld + ch] = v;
    };
    if (ch >= W) {
        for (int t = t0; t < t1; ++t) put(t, 0.f);
        return;
    }
    float S = 0.f;
#pragma unroll 8
    for (int v = 0; v < w; ++v) S = a.ws[(size_t)v * 3 * W + ch] * S + a.ws[((size_t)v * 3 + 1) * W + ch];
    int last_start = -1;                // the sequence that may go on past this window begins here
    for (int t = t0; t < t1; ++t)
        if (t == 0 || a.seq[t] != a.seq[t - 1]) last_start = t;
    const float bz = a.bias_z[ch], bx = a.bias_x[ch];
#pragma unroll 8
    for (int t = t0; t < t1; ++t) {
        const int seq = a.seq[t];
        if (t == 0 || seq != a.seq[t - 1]) {
            if (a.pos[t] == 0) S = 0.f;
            else S = gridDim.y > 1 && t == last_start ? a.ws[((size_t)w * 3 + 2) * W + ch] : a.state[(size_t)seq * W + ch];
        }
        const float *p = a.zxg + (size_t)t * 3 * W + ch;
        const MinGruGate g = min_gru_gate(p[0] + bz, p[W] + bx);
        S = fmaf(g.keep, S, g.in);
        put(t, S * act_silu(p[2 * W]));
        if (t + 1 == T || a.seq[t + 1] != seq) a.state[(size_t)seq * W + ch] = S;
    }
}

size_t min_gru_workspace(int T, int width) { return (size_t)((T + GRU_WINDOW - 1) / GRU_WINDOW) * 3 * width; }

int min_gru(const MinGruArgs &a, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    const int windows = (T + GRU_WINDOW - 1) / GRU_WINDOW;
    if (!a.zxg || !a.state || !a.out || a.ld < a.width || a.width < 1 || windows > 65535 || (windows > 1 && !a.ws)) return fail(MESH_ERR_INVALID, "min_gru: bad operands");
    const dim3 block(GRU_THREADS);
    if (windows > 1) {
        MESH_LAUNCH(min_gru_compose_kernel, dim3((unsigned)((a.width + GRU_THREADS - 1) / GRU_THREADS), (unsigned)windows), block, 0, stream, a, T);
        MESH_LAUNCH_CHECK();
    }
    const dim3 grid((unsigned)((a.ld + GRU_THREADS - 1) / GRU_THREADS), (unsigned)windows);
    if (a.act == ACT_BF16) MESH_LAUNCH((min_gru_kernel<ACT_BF16>), grid, block, 0, stream, a, T);
    else MESH_LAUNCH((min_gru_kernel<ACT_F32>), grid, block, 0, stream, a, T);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

}  // namespace mesh
