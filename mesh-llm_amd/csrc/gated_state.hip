// See gated_state.hpp.
//
// The products of the chunk path run on v_mfma_f32_16x16x4_f32: the state and everything that enters it stay f32.  That
// instruction contracts over four k, one per lane group g; step j of a float4 is taken as k = 16 n + 4 g + j, so that an operand
// is one 16-byte load per 16 k, and a result tile (lane group g holds rows 4g .. 4g + 3 of column c) is the right operand of
// the next product as it lies in the registers.  The scan therefore moves no state between lanes.
#include "gated_state.hpp"

#include <algorithm>

#include "act_math.hpp"

namespace mesh {

typedef float gs_f4 __attribute__((ext_vector_type(4)));

constexpr int C = STATE_CHUNK;
constexpr float UNIT_EPS = 1e-6f;               // inside the root of the unit vectors of DELTA

__device__ __forceinline__ float gs_wave_sum(float v) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    return v;
}
__device__ __forceinline__ float gs_softplus(float z) { return fmaxf(z, 0.f) + log1pf(expf(-fabsf(z))); }
__device__ __forceinline__ gs_f4 gs_mma(const float4 &a, const gs_f4 &b, gs_f4 acc) {
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.x, b[0], acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.y, b[1], acc, 0, 0, 0);
    acc = __builtin_amdgcn_mfma_f32_16x16x4f32(a.z, b[2], acc, 0, 0, 0);
    return __builtin_amdgcn_mfma_f32_16x16x4f32(a.w, b[3], acc, 0, 0, 0);
}
__device__ __forceinline__ gs_f4 gs_mma(const float4 &a, const float4 &b, gs_f4 acc) { return gs_mma(a, gs_f4{b.x, b.y, b.z, b.w}, acc); }

__device__ __forceinline__ float delta_log_decay(const GatedStateArgs &a, int t, int h) { return -a.A[h] * gs_softplus(a.in[(size_t)t * a.ld + a.at_a + h] + a.dt_bias[h]); }
__device__ __forceinline__ float delta_beta(const GatedStateArgs &a, int t, int h) { return act_sigmoid(a.in[(size_t)t * a.ld + a.at_b + h]); }

// Convolution and silu of one channel at token t.  at: its column of `in`; ch: its place in the tail; t_first: the call's first
// token of the sequence (inputs before it come from the tail).
__device__ __forceinline__ float delta_conv(const GatedStateArgs &a, const float *w, int t, int t_first, int at, int ch, int channels) {
    const int pos = a.pos[t];
    const float *tail = a.tail + (size_t)a.seq[t] * a.taps * channels + ch;
    float v = 0.f;
    for (int j = 0; j < a.taps; ++j) {
        const int back = a.taps - 1 - j;
        if (pos < back) continue;
        const float x = t - back >= t_first ? a.in[(size_t)(t - back) * a.ld + at] : tail[(size_t)((pos - back) % a.taps) * channels];
        v = fmaf(w[j], x, v);
    }
    return act_silu(v);
}

// The same for tokens t0 .. t0 + 15 (the first `live` of them; zeros behind), up to CONV_WINDOW taps: every input is read once.
constexpr int CONV_WINDOW = 4, CONV_RUN = 16;
__device__ __forceinline__ void delta_conv_run(const GatedStateArgs &a, const float *w, int t0, int live, int t_first, int pos0, const float *tail, int at, int channels, float (&y)[CONV_RUN]) {
    float x[CONV_RUN + CONV_WINDOW - 1], wt[CONV_WINDOW];
#pragma unroll
    for (int j = 0; j < CONV_WINDOW; ++j) {
        const int tap = a.taps - CONV_WINDOW + j;
        wt[j] = tap >= 0 ? w[tap] : 0.f;
    }
#pragma unroll
    for (int i = 0; i < CONV_RUN + CONV_WINDOW - 1; ++i) {
        const int k = i - (CONV_WINDOW - 1);              // token t0 + k at position pos0 + k
        x[i] = 0.f;
        if (k < 0) {
            if (-k < a.taps && pos0 + k >= 0) x[i] = t0 + k >= t_first ? a.in[(size_t)(t0 + k) * a.ld + at] : tail[(size_t)((unsigned)(pos0 + k) % (unsigned)a.taps) * channels];
        } else if (k < live) {
            x[i] = a.in[(size_t)(t0 + k) * a.ld + at];
        }
    }
#pragma unroll
    for (int k = 0; k < CONV_RUN; ++k) {
        float v = 0.f;
#pragma unroll
        for (int j = 0; j < CONV_WINDOW; ++j) v = fmaf(wt[j], x[k + j], v);
        y[k] = k < live ? act_silu(v) : 0.f;
    }
}

// ---- one token per sequence
// grid (heads, T).  Thread (row group, column): RPT rows of one column of the state in registers.
template <int THREADS, int RPT>
__global__ __launch_bounds__(THREADS) void gated_step_kernel(const GatedStateArgs a, int vt) {
    __shared__ float sq[STATE_DIM_MAX], sk[STATE_DIM_MAX], sd[STATE_DIM_MAX], sv[STATE_DIM_MAX], so[STATE_DIM_MAX];
    __shared__ float red[2][THREADS], s_qk, s_ss;
    const int h = blockIdx.x, t = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int D = a.dim, V = a.vdim, seq = a.seq[t], pos = a.pos[t];
    const int col = tid & (vt - 1), grp = tid / vt, groups = THREADS / vt;
    float *st = a.state + ((size_t)seq * a.heads + h) * D * V;
    // the state's rows are requested before anything is computed
    float S[RPT];
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int d = grp + i * groups;
        S[i] = pos > 0 && d < D && col < V ? st[(size_t)d * V + col] : 0.f;
    }
    const float *x = a.in + (size_t)t * a.ld;
    float decay = 1.f, beta = 1.f;
    // (so are the vectors that the token's output ends with: V <= THREADS)
    const int vi = tid < V ? tid : V - 1;
    const float out_norm = a.norm[vi], out_gate = x[a.at_g + h * V + vi];
    if (a.delta) {
        decay = expf(delta_log_decay(a, t, h));
        beta = delta_beta(a, t, h);
        const int kvh = h / (a.heads / a.kv_heads), channels = 2 * a.kv_heads * D + a.heads * V, taps = a.taps, now = pos % taps;
        float *tail = a.tail + (size_t)seq * taps * channels;
        const bool own = h % (a.heads / a.kv_heads) == 0;           // one head of a group keeps the shared channels' inputs
        for (int i = tid; i < 2 * D + V; i += THREADS) {
            const int part = i < D ? 0 : i < 2 * D ? 1 : 2, e = part == 0 ? i : part == 1 ? i - D : i - 2 * D;
            const int c = part == 2 ? h * V + e : kvh * D + e;
            const int at = (part == 0 ? a.at_q : part == 1 ? a.at_k : a.at_v) + c, ch = (part == 0 ? 0 : part == 1 ? a.kv_heads * D : 2 * a.kv_heads * D) + c;
            const float *w = (part == 0 ? a.conv_q : part == 1 ? a.conv_k : a.conv_v) + (size_t)c * taps;
            const float xi = x[at];
            float y = w[taps - 1] * xi;
#pragma unroll 4
            for (int back = 1; back < taps; ++back) {
                const int slot = now - back < 0 ? now - back + taps : now - back;
                const float p = pos >= back ? tail[(size_t)slot * channels + ch] : 0.f;
                y = fmaf(w[taps - 1 - back], p, y);
            }
            (part == 0 ? sq : part == 1 ? sk : sv)[e] = act_silu(y);
            if (own || part == 2) tail[(size_t)now * channels + ch] = xi;       // (not a slot that is read in this call: those are of taps - 1 other positions)
        }
        __syncthreads();
        if (wave < 2) {
            float *u = wave == 0 ? sq : sk, ss = 0.f;
            for (int d = lane; d < D; d += 64) ss = fmaf(u[d], u[d], ss);
            const float r = (wave == 0 ? 1.0f / sqrtf((float)D) : 1.0f) / sqrtf(gs_wave_sum(ss) + UNIT_EPS);
            for (int d = lane; d < D; d += 64) u[d] *= r;
        }
    } else {
        const float qs = 1.0f / sqrtf((float)D);
        for (int d = tid; d < D; d += THREADS) {
            sq[d] = x[a.at_q + h * D + d] * qs;
            sk[d] = x[a.at_k + h * D + d];
        }
        // four lanes per channel
        for (int d0 = 0; d0 < D; d0 += THREADS / 4) {
            const int d = d0 + (tid >> 2);
            float z = 0.f;
            if (d < D) {
                const float *w = a.a2 + (size_t)(h * D + d) * a.rank;
#pragma unroll 4
                for (int r = tid & 3; r < a.rank; r += 4) z = fmaf(w[r], x[a.at_a + r], z);
            }
            z += __shfl_xor(z, 1);
            z += __shfl_xor(z, 2);
            if (d < D && (tid & 3) == 0) sd[d] = expf(-gs_softplus(-(z + a.a2_bias[h * D + d])) * a.inv_tau);
        }
        for (int v = tid; v < V; v += THREADS) sv[v] = x[a.at_v + h * V + v];
    }
    __syncthreads();
    if (wave == 0) {
        float s = 0.f;
        for (int d = lane; d < D; d += 64) s = fmaf(sq[d], sk[d], s);
        s = gs_wave_sum(s);
        if (lane == 0) s_qk = s;
    }
    // S^T k and S^T q of the decayed state; with them o = S^T q + (k . q) u needs no second walk
    float dk = 0.f, dq = 0.f;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int d = grp + i * groups < D ? grp + i * groups : D - 1;          // (rows past the state are zeros)
        S[i] *= a.delta ? decay : sd[d];
        dk = fmaf(S[i], sk[d], dk);
        dq = fmaf(S[i], sq[d], dq);
    }
    red[0][tid] = dk; red[1][tid] = dq;
    __syncthreads();
    dk = dq = 0.f;
    for (int g = 0; g < groups; ++g) { dk += red[0][g * vt + col]; dq += red[1][g * vt + col]; }
    const float v = col < V ? sv[col] : 0.f;
    const float u = a.delta ? beta * (v - dk) : v;
#pragma unroll
    for (int i = 0; i < RPT; ++i) {
        const int d = grp + i * groups;
        if (d < D && col < V) st[(size_t)d * V + col] = fmaf(sk[d], u, S[i]);
    }
    if (grp == 0 && col < V) so[col] = fmaf(s_qk, u, dq);
    __syncthreads();
    if (wave == 0) {
        float ss = 0.f;
        for (int i = lane; i < V; i += 64) ss = fmaf(so[i], so[i], ss);
        ss = gs_wave_sum(ss);
        if (lane == 0) s_ss = ss;
    }
    __syncthreads();
    const float r = 1.0f / sqrtf(s_ss / (float)V + a.eps);
    const size_t to = (size_t)t * a.ld_out;
    auto put = [&](int i, float y) {
        if (a.act == ACT_BF16) static_cast<uint16_t *>(a.out)[to + i] = f32_to_bf16_bits(y);
        else static_cast<float *>(a.out)[to + i] = y;
    };
    if (tid < V) put(h * V + tid, so[tid] * r * out_norm * act_silu(out_gate));
    if (h == a.heads - 1)
        for (int i = a.heads * V + tid; i < a.ld_out; i += THREADS) put(i, 0.f);
}

// ---- chunks
__host__ __device__ constexpr int gs_pad64(int n) { return (n + 63) / 64 * 64; }
__host__ __device__ constexpr int gs_pad16(int n) { return (n + 15) / 16 * 16; }
// What the first launch leaves of a (chunk, head), in this order; Dp = dim padded to 64, Vp = vdim padded to 16, padding zero
struct GsMats {
    float *Q, *KT, *A, *G, *W, *U;          // [C][Dp], [Dp][C], [C][C], [Dp], [C][Dp], [C][Vp]
    __device__ __forceinline__ GsMats(float *ws, size_t index, int Dp, int Vp, bool delta) {
        const size_t n = (size_t)C * (2 * Dp + C) + Dp + (delta ? (size_t)C * (Dp + Vp) : 0);
        Q = ws + index * n;
        KT = Q + (size_t)C * Dp;
        A = KT + (size_t)C * Dp;
        G = A + C * C;
        W = G + Dp;
        U = W + (size_t)C * Dp;
    }
};
size_t gated_state_workspace(int n_chunks, int heads, int dim, int vdim) {
    const size_t Dp = (size_t)gs_pad64(dim), Vp = (size_t)gs_pad16(vdim);
    return (size_t)n_chunks * heads * (C * (3 * Dp + C + Vp) + Dp);
}

constexpr int PREP_THREADS = 256;

// grid (chunks, heads)
__global__ __launch_bounds__(PREP_THREADS) void delta_prepare_kernel(const GatedStateArgs a) {
    extern __shared__ __align__(16) float sm[];
    const int ci = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int D = a.dim, V = a.vdim, Dp = gs_pad64(D), Vp = gs_pad16(V), dp = Dp + 4, vp = Vp + 4;
    constexpr int LP = C + 4;
    float *sQ = sm, *sK = sQ + C * dp, *sV = sK + C * dp, *sL = sV + C * vp, *sA = sL + C * LP, *sT = sA + C * LP;
    float *s_cum = sT + C * LP, *s_beta = s_cum + C, *s_since = s_beta + C, *s_until = s_since + C;       // decays since the chunk's start, until its end
    const int t0 = a.chunks.chunk[ci], n = a.chunks.chunk[ci + 1] - t0, first = a.chunks.first[ci];
    const int kvh = h / (a.heads / a.kv_heads), channels = 2 * a.kv_heads * D + a.heads * V;
    // a channel's half chunk per thread: columns of q, of k, of v
    const int pos0 = a.pos[t0];
    const float *tail = a.tail + (size_t)a.seq[t0] * a.taps * channels;
    for (int i = tid; i < 2 * (2 * Dp + Vp); i += PREP_THREADS) {
        const int half = i >= 2 * Dp + Vp, e = half ? i - (2 * Dp + Vp) : i, part = e < Dp ? 0 : e < 2 * Dp ? 1 : 2, d = e - part * Dp;
        const int c0 = part == 2 ? h * V + d : kvh * D + d, r0 = half * CONV_RUN;
        const int at = (part == 0 ? a.at_q : part == 1 ? a.at_k : a.at_v) + c0, ch = part * a.kv_heads * D + c0;
        const float *w = (part == 0 ? a.conv_q : part == 1 ? a.conv_k : a.conv_v) + (size_t)c0 * a.taps;
        float y[CONV_RUN];
        const int live = d < (part == 2 ? V : D) ? n - r0 : 0;
        if (live <= 0) {
#pragma unroll
            for (int k = 0; k < CONV_RUN; ++k) y[k] = 0.f;
        } else if (a.taps <= CONV_WINDOW) {
            delta_conv_run(a, w, t0 + r0, live, first, pos0 + r0, tail + ch, at, channels, y);
        } else {
#pragma unroll
            for (int k = 0; k < CONV_RUN; ++k) y[k] = k < live ? delta_conv(a, w, t0 + r0 + k, first, at, ch, channels) : 0.f;
        }
        float *dst = (part == 0 ? sQ : part == 1 ? sK : sV) + d;
        const int pitch = part == 2 ? vp : dp;
#pragma unroll
        for (int k = 0; k < CONV_RUN; ++k) dst[(r0 + k) * pitch] = y[k];
    }
    if (wave == 0) {          // logarithms of the decays, summed from the chunk's start
        float s = lane < n ? delta_log_decay(a, t0 + lane, h) : 0.f;
#pragma unroll
        for (int o = 1; o < C; o <<= 1) { const float p = __shfl_up(s, o); if (lane >= o) s += p; }
        const float end = __shfl(s, C - 1);
        if (lane < C) { s_cum[lane] = s; s_beta[lane] = lane < n ? delta_beta(a, t0 + lane, h) : 0.f; s_since[lane] = expf(s); s_until[lane] = expf(end - s); }
    }
    __syncthreads();
    const float qs = 1.0f / sqrtf((float)D);
    // sixteen lanes per row (the columns past dim are zeros)
#pragma unroll
    for (int r0 = 0; r0 < 2 * C; r0 += PREP_THREADS / 16) {
        const int r = r0 + (tid >> 4);
        float *u = (r < C ? sQ : sK) + (r & (C - 1)) * dp, ss = 0.f;
        for (int d = 4 * c; d < Dp; d += 64) {
            const float4 v = *reinterpret_cast<const float4 *>(u + d);
            ss = fmaf(v.x, v.x, fmaf(v.y, v.y, fmaf(v.z, v.z, fmaf(v.w, v.w, ss))));
        }
#pragma unroll
        for (int o = 8; o > 0; o >>= 1) ss += __shfl_xor(ss, o);
        const float f = (r < C ? qs : 1.0f) / sqrtf(ss + UNIT_EPS);
        for (int d = 4 * c; d < Dp; d += 64) {
            float4 v = *reinterpret_cast<const float4 *>(u + d);
            v.x *= f; v.y *= f; v.z *= f; v.w *= f;
            *reinterpret_cast<float4 *>(u + d) = v;
        }
    }
    __syncthreads();
    // products of keys with keys and queries with keys, one 16 x 16 tile a wave
    {
        const int rt = wave >> 1, ct = wave & 1;
        gs_f4 kk = {0.f, 0.f, 0.f, 0.f}, qk = kk;
        for (int d = 0; d < Dp; d += 16) {
            const float4 b = *reinterpret_cast<const float4 *>(sK + (16 * ct + c) * dp + d + 4 * g);
            kk = gs_mma(*reinterpret_cast<const float4 *>(sK + (16 * rt + c) * dp + d + 4 * g), b, kk);
            qk = gs_mma(*reinterpret_cast<const float4 *>(sQ + (16 * rt + c) * dp + d + 4 * g), b, qk);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int r = 16 * rt + 4 * g + i, j = 16 * ct + c;
            const float f = j <= r ? expf(s_cum[r] - s_cum[j]) : 0.f;
            sL[r * LP + j] = j < r ? s_beta[r] * f * kk[i] : 0.f;
            sA[r * LP + j] = f * qk[i];
        }
    }
    __syncthreads();
    const GsMats m(a.ws, (size_t)ci * a.heads + h, Dp, Vp, true);
    if (wave == 0) {
        // T = (I + L)^-1, a column per lane by forward substitution (lanes past the chunk repeat a column)
        const int j = lane & (C - 1);
        float x[C];
#pragma unroll
        for (int r = 0; r < C; ++r) {
            float v[4] = {r == j ? 1.f : 0.f, 0.f, 0.f, 0.f};          // (four sums: the chain through x is long enough)
#pragma unroll
            for (int k = 0; k < r; ++k) v[k & 3] = fmaf(-sL[r * LP + k], x[k], v[k & 3]);
            x[r] = (v[0] + v[1]) + (v[2] + v[3]);
        }
        if (lane < C) {
#pragma unroll
            for (int r = 0; r < C; ++r) sT[r * LP + j] = x[r];
        }
    } else {
        const int id = tid - 64, step = PREP_THREADS - 64;
        for (int r = wave - 1; r < C; r += 3) {
            const float f = s_since[r];
            for (int d = lane * 4; d < Dp; d += 256) {
                float4 q = *reinterpret_cast<const float4 *>(sQ + r * dp + d);
                q.x *= f; q.y *= f; q.z *= f; q.w *= f;
                *reinterpret_cast<float4 *>(m.Q + (size_t)r * Dp + d) = q;
            }
        }
        for (int i = id; i < Dp * (C / 4); i += step) {
            const int d = i / (C / 4), r = i % (C / 4) * 4;
            *reinterpret_cast<float4 *>(m.KT + (size_t)d * C + r) =
                make_float4(sK[r * dp + d] * s_until[r], sK[(r + 1) * dp + d] * s_until[r + 1], sK[(r + 2) * dp + d] * s_until[r + 2], sK[(r + 3) * dp + d] * s_until[r + 3]);
        }
        for (int i = id; i < C * C / 4; i += step) *reinterpret_cast<float4 *>(m.A + 4 * i) = *reinterpret_cast<const float4 *>(sA + (i / (C / 4)) * LP + i % (C / 4) * 4);
        for (int i = id; i < Dp; i += step) m.G[i] = s_since[C - 1];
    }
    __syncthreads();
    // W = T (beta decay K), U = T (beta V): column tiles dealt to the waves, both row tiles of each
    const int nd = Dp / 16, nv = Vp / 16;
    for (int ct = wave; ct < nd + nv; ct += 4) {
        const bool w = ct < nd;
        const float *X = w ? sK + 16 * ct : sV + 16 * (ct - nd);
        const int xp = w ? dp : vp;
        gs_f4 acc[2] = {gs_f4{0.f, 0.f, 0.f, 0.f}, gs_f4{0.f, 0.f, 0.f, 0.f}};
#pragma unroll
        for (int s = 0; s < 2; ++s) {
            gs_f4 b;
#pragma unroll
            for (int j = 0; j < 4; ++j) {
                const int k = 16 * s + 4 * g + j;
                b[j] = X[k * xp + c] * s_beta[k] * (w ? s_since[k] : 1.f);
            }
#pragma unroll
            for (int rt = s; rt < 2; ++rt) acc[rt] = gs_mma(*reinterpret_cast<const float4 *>(sT + (16 * rt + c) * LP + 16 * s + 4 * g), b, acc[rt]);
        }
#pragma unroll
        for (int rt = 0; rt < 2; ++rt)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int r = 16 * rt + 4 * g + i;
                if (w) m.W[(size_t)r * Dp + 16 * ct + c] = acc[rt][i];
                else m.U[(size_t)r * Vp + 16 * (ct - nd) + c] = acc[rt][i];
            }
    }
}
static size_t delta_prepare_lds(int dim, int vdim) {
    return ((size_t)C * (2 * (gs_pad64(dim) + 4) + gs_pad16(vdim) + 4 + 3 * (C + 4)) + 4 * C) * sizeof(float);
}

// grid (chunks, heads)
__global__ __launch_bounds__(PREP_THREADS) void gla_prepare_kernel(const GatedStateArgs a) {
    extern __shared__ __align__(16) float sm[];
    const int ci = blockIdx.x, h = blockIdx.y, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int D = a.dim, Dp = gs_pad64(D), dp = Dp + 4;
    float *sQ = sm, *sK = sQ + C * dp, *sG = sK + C * dp;         // queries, keys, logarithms of the decays summed from the chunk's start
    const int t0 = a.chunks.chunk[ci], n = a.chunks.chunk[ci + 1] - t0;
    float *sX = sG + C * dp, *sS = sX + C * a.rank;               // a1 rows; sums over the first half chunk
    const float qs = 1.0f / sqrtf((float)D);
    // a wave's rows of 64 columns are all on their way before the first is kept
    constexpr int ROWS = C / 4;
    const float *xr[ROWS];
#pragma unroll
    for (int i = 0; i < ROWS; ++i) xr[i] = a.in + (size_t)(t0 + (wave + 4 * i < n ? wave + 4 * i : 0)) * a.ld;
    for (int k = lane; k < a.rank; k += 64) {
        float v[ROWS];
#pragma unroll
        for (int i = 0; i < ROWS; ++i) v[i] = xr[i][a.at_a + k];
#pragma unroll
        for (int i = 0; i < ROWS; ++i) sX[(wave + 4 * i) * a.rank + k] = wave + 4 * i < n ? v[i] : 0.f;
    }
    for (int d = lane; d < Dp; d += 64) {
        float q[ROWS], k[ROWS];
        const int from = h * D + (d < D ? d : 0);
#pragma unroll
        for (int i = 0; i < ROWS; ++i) { q[i] = xr[i][a.at_q + from]; k[i] = xr[i][a.at_k + from]; }
#pragma unroll
        for (int i = 0; i < ROWS; ++i) {
            const int r = wave + 4 * i;
            const bool live = r < n && d < D;
            sQ[r * dp + d] = live ? q[i] * qs : 0.f;
            sK[r * dp + d] = live ? k[i] : 0.f;
        }
    }
    __syncthreads();
    // a channel's half chunk per thread: its pre-activations, then the running sums of their logarithms
    constexpr int HALF = C / 2;
    for (int i0 = 0; i0 < 2 * Dp; i0 += PREP_THREADS) {
        const int i = i0 + tid, half = i >= Dp, d = half ? i - Dp : i, r0 = half * HALF;
        float z[HALF];
        if (i < 2 * Dp) {
            const float *w = a.a2 + (size_t)(h * D + (d < D ? d : 0)) * a.rank;
            const float bias = d < D ? a.a2_bias[h * D + d] : 0.f;
#pragma unroll
            for (int k = 0; k < HALF; ++k) z[k] = bias;
            constexpr int WB = 8;             // weights of a channel on their way at once
            for (int j0 = 0; j0 < a.rank; j0 += WB) {
                float wj[WB];
#pragma unroll
                for (int j = 0; j < WB; ++j) wj[j] = j0 + j < a.rank ? w[j0 + j] : 0.f;
#pragma unroll
                for (int j = 0; j < WB; ++j) {
                    const int at = j0 + j < a.rank ? j0 + j : 0;
#pragma unroll
                    for (int k = 0; k < HALF; ++k) z[k] = fmaf(wj[j], sX[(r0 + k) * a.rank + at], z[k]);
                }
            }
            float sum = 0.f;
#pragma unroll
            for (int k = 0; k < HALF; ++k) {
                sum += d < D && r0 + k < n ? -gs_softplus(-z[k]) * a.inv_tau : 0.f;
                z[k] = sum;
            }
            if (!half) sS[d] = sum;
        }
        __syncthreads();            // (first halves are behind when their second halves add them: Dp <= PREP_THREADS)
        if (i < 2 * Dp) {
            const float before = half ? sS[d] : 0.f;
#pragma unroll
            for (int k = 0; k < HALF; ++k) sG[(r0 + k) * dp + d] = z[k] + before;
        }
    }
    __syncthreads();
    const GsMats m(a.ws, (size_t)ci * a.heads + h, Dp, 0, false);
    for (int r = wave; r < C; r += 4)
        for (int d = lane; d < Dp; d += 64) m.Q[(size_t)r * Dp + d] = sQ[r * dp + d] * expf(sG[r * dp + d]);
    for (int i = tid; i < Dp * (C / 4); i += PREP_THREADS) {
        const int d = i / (C / 4), r = i % (C / 4) * 4;
        const float end = sG[(C - 1) * dp + d];
        float k[4];
#pragma unroll
        for (int j = 0; j < 4; ++j) k[j] = sK[(r + j) * dp + d] * expf(end - sG[(r + j) * dp + d]);
        *reinterpret_cast<float4 *>(m.KT + (size_t)d * C + r) = make_float4(k[0], k[1], k[2], k[3]);
    }
    for (int d = tid; d < Dp; d += PREP_THREADS) m.G[d] = expf(sG[(C - 1) * dp + d]);
    // A: a decay per channel does not leave the sum over channels.  Within a 16 x 16 diagonal block each pair takes its own
    // exponentials (a token with itself has none: eight lanes share its sum); the block below them is a product of queries decayed
    // since token 15 and keys decayed until it.  No exponent is ever positive.
    constexpr int PAIRS = 16 * 15 / 2;
    static_assert(2 * PAIRS <= PREP_THREADS && PREP_THREADS == 8 * C, "one turn per thread");
    {
        const int r = tid >> 3;
        float s = 0.f;
        for (int d = 4 * (tid & 7); d < Dp; d += 32) {
            const float4 q = *reinterpret_cast<const float4 *>(sQ + r * dp + d), k = *reinterpret_cast<const float4 *>(sK + r * dp + d);
            s = fmaf(q.x, k.x, fmaf(q.y, k.y, fmaf(q.z, k.z, fmaf(q.w, k.w, s))));
        }
        s += __shfl_xor(s, 1); s += __shfl_xor(s, 2); s += __shfl_xor(s, 4);
        if ((tid & 7) == 0) m.A[r * C + r] = s;
    }
    if (tid < 2 * PAIRS) {
        // pair p of a block: row r >= 1, column p - r (r - 1) / 2 < r
        const int b = tid / PAIRS, p = tid % PAIRS;
        int r = (int)((sqrtf(8.f * p + 1.f) - 1.f) * 0.5f) + 1;
        r += r * (r + 1) / 2 <= p ? 1 : 0;
        r -= r * (r - 1) / 2 > p ? 1 : 0;
        const int j = 16 * b + p - r * (r - 1) / 2;
        r += 16 * b;
        float s = 0.f;
        for (int d = 0; d < Dp; d += 4) {
            const float4 q = *reinterpret_cast<const float4 *>(sQ + r * dp + d), k = *reinterpret_cast<const float4 *>(sK + j * dp + d);
            const float4 gr = *reinterpret_cast<const float4 *>(sG + r * dp + d), gj = *reinterpret_cast<const float4 *>(sG + j * dp + d);
            s = fmaf(q.x * k.x, act_exp_neg(gj.x - gr.x), s);
            s = fmaf(q.y * k.y, act_exp_neg(gj.y - gr.y), s);
            s = fmaf(q.z * k.z, act_exp_neg(gj.z - gr.z), s);
            s = fmaf(q.w * k.w, act_exp_neg(gj.w - gr.w), s);
        }
        m.A[r * C + j] = s;
        m.A[j * C + r] = 0.f;
    }
    if (wave == 3) {
        gs_f4 acc = {0.f, 0.f, 0.f, 0.f};
        for (int d = 4 * g; d < Dp; d += 16) {
            const float4 ref = *reinterpret_cast<const float4 *>(sG + 15 * dp + d);
            const float4 q = *reinterpret_cast<const float4 *>(sQ + (16 + c) * dp + d), gq = *reinterpret_cast<const float4 *>(sG + (16 + c) * dp + d);
            const float4 k = *reinterpret_cast<const float4 *>(sK + c * dp + d), gk = *reinterpret_cast<const float4 *>(sG + c * dp + d);
            const float4 qa = make_float4(q.x * act_exp_neg(ref.x - gq.x), q.y * act_exp_neg(ref.y - gq.y), q.z * act_exp_neg(ref.z - gq.z), q.w * act_exp_neg(ref.w - gq.w));
            const float4 kb = make_float4(k.x * act_exp_neg(gk.x - ref.x), k.y * act_exp_neg(gk.y - ref.y), k.z * act_exp_neg(gk.z - ref.z), k.w * act_exp_neg(gk.w - ref.w));
            acc = gs_mma(qa, kb, acc);
        }
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            m.A[(16 + 4 * g + i) * C + c] = acc[i];
            m.A[(4 * g + i) * C + 16 + c] = 0.f;
        }
    }
}
static size_t gla_prepare_lds(int dim, int rank) { return ((size_t)C * (3 * (gs_pad64(dim) + 4) + rank) + gs_pad64(dim)) * sizeof(float); }

// grid (heads, 16-column slices of the values, sequences of the call).  Wave w owns rows [16 NT w, 16 NT (w + 1)) of the state.
template <bool DELTA, int NT>
__global__ __launch_bounds__(256) void state_scan_kernel(const GatedStateArgs a) {
    constexpr int Dp = 64 * NT;
    __shared__ __align__(16) float red[2][4][DELTA ? 4 : 2][64][4];        // by chunk parity, wave: partial W S and Q S of the two row tiles
    const int h = blockIdx.x, v0 = blockIdx.y * 16, run = blockIdx.z;
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int D = a.dim, V = a.vdim, Vp = gs_pad16(V), col = v0 + c, d0 = wave * 16 * NT;
    const int c0 = a.chunks.run[run], c1 = a.chunks.run[run + 1];
    const int t_first = a.chunks.chunk[c0];
    float *st = a.state + ((size_t)a.seq[t_first] * a.heads + h) * D * V;
    const bool zero = a.pos[t_first] == 0;
    gs_f4 S[NT];
#pragma unroll
    for (int k = 0; k < NT; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = d0 + 16 * k + 4 * g + i;
            S[k][i] = !zero && d < D && col < V ? st[(size_t)d * V + col] : 0.f;
        }
    // what a chunk brings: W (DELTA), Q by (row tile, own d tile), K^T by (own d tile, token tile), G, U
    struct Frag {
        float4 w[DELTA ? 2 : 1][NT], q[2][NT], k[NT][2];
        gs_f4 gd[NT], u[2];
        float4 a[2];                    // the rows of A of this wave's output tile (waves 0 and 1)
    };
    // (every chunk of a run but its last is whole)
    const int t_end = a.chunks.chunk[c1];
    auto load = [&](int ci, Frag &f) {
        const GsMats m(a.ws, (size_t)ci * a.heads + h, Dp, Vp, DELTA);
#pragma unroll
        for (int k = 0; k < NT; ++k) {
            const int d = d0 + 16 * k + 4 * g;
#pragma unroll
            for (int r = 0; r < 2; ++r) {
                if constexpr (DELTA) f.w[r][k] = *reinterpret_cast<const float4 *>(m.W + (size_t)(16 * r + c) * Dp + d);
                f.q[r][k] = *reinterpret_cast<const float4 *>(m.Q + (size_t)(16 * r + c) * Dp + d);
                f.k[k][r] = *reinterpret_cast<const float4 *>(m.KT + (size_t)(d0 + 16 * k + c) * C + 16 * r + 4 * g);
            }
            const float4 gv = *reinterpret_cast<const float4 *>(m.G + d);
            f.gd[k] = gs_f4{gv.x, gv.y, gv.z, gv.w};
        }
        const int t0 = t_first + (ci - c0) * C, n = t_end - t0;
#pragma unroll
        for (int r = 0; r < 2; ++r)
            if (r <= wave && wave < 2) f.a[r] = *reinterpret_cast<const float4 *>(m.A + (16 * wave + c) * C + 16 * r + 4 * g);
#pragma unroll
        for (int r = 0; r < 2; ++r)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int tk = 16 * r + 4 * g + i;
                if constexpr (DELTA) f.u[r][i] = m.U[(size_t)tk * Vp + col];
                else f.u[r][i] = tk < n && col < V ? a.in[(size_t)(t0 + tk) * a.ld + a.at_v + h * V + col] : 0.f;
            }
    };
    // the chunk in `cur`, while the one AHEAD behind it is fetched into `ahead` (as many as the registers hold)
    constexpr int AHEAD = NT < 4 ? 2 : 1;
    auto step = [&](int ci, const Frag &cur, Frag &ahead) {
        if (ci + AHEAD < c1) load(ci + AHEAD, ahead);
        float (*rd)[DELTA ? 4 : 2][64][4] = red[(ci - c0) & 1];
        gs_f4 ws[2], qs[2];
#pragma unroll
        for (int r = 0; r < 2; ++r) {
            ws[r] = qs[r] = gs_f4{0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int k = 0; k < NT; ++k) {
                if constexpr (DELTA) ws[r] = gs_mma(cur.w[r][k], S[k], ws[r]);
                qs[r] = gs_mma(cur.q[r][k], S[k], qs[r]);
            }
            *reinterpret_cast<gs_f4 *>(rd[wave][r][lane]) = qs[r];
            if constexpr (DELTA) *reinterpret_cast<gs_f4 *>(rd[wave][2 + r][lane]) = ws[r];
        }
        // one barrier a chunk: the buffer of this parity is written again two chunks on, behind the next chunk's barrier
        __syncthreads();
        gs_f4 u[2] = {cur.u[0], cur.u[1]};
        if constexpr (DELTA) {
#pragma unroll
            for (int r = 0; r < 2; ++r)
#pragma unroll
                for (int w = 0; w < 4; ++w) u[r] -= *reinterpret_cast<const gs_f4 *>(rd[w][2 + r][lane]);
        }
        if (wave < 2) {                 // the outputs of row tile `wave`
            gs_f4 o = {0.f, 0.f, 0.f, 0.f};
#pragma unroll
            for (int w = 0; w < 4; ++w) o += *reinterpret_cast<const gs_f4 *>(rd[w][wave][lane]);
#pragma unroll
            for (int s = 0; s < 2; ++s)
                if (s <= wave) o = gs_mma(cur.a[s], u[s], o);
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                const int tk = 16 * wave + 4 * g + i;
                const int t = t_first + (ci - c0) * C + tk;
                if (t < t_end && col < V) a.o[(size_t)t * a.heads * V + h * V + col] = o[i];
            }
        }
#pragma unroll
        for (int k = 0; k < NT; ++k) {
            gs_f4 s = S[k] * cur.gd[k];
            s = gs_mma(cur.k[k][0], u[0], s);
            S[k] = gs_mma(cur.k[k][1], u[1], s);
        }
    };
    Frag f0, f1;
    load(c0, f0);
    if constexpr (AHEAD == 2) {
        Frag f2;
        if (c0 + 1 < c1) load(c0 + 1, f1);
        for (int ci = c0; ci < c1; ci += 3) {
            step(ci, f0, f2);
            if (ci + 1 < c1) step(ci + 1, f1, f0);
            if (ci + 2 < c1) step(ci + 2, f2, f1);
        }
    } else {
        for (int ci = c0; ci < c1; ci += 2) {
            step(ci, f0, f1);
            if (ci + 1 < c1) step(ci + 1, f1, f0);
        }
    }
#pragma unroll
    for (int k = 0; k < NT; ++k)
#pragma unroll
        for (int i = 0; i < 4; ++i) {
            const int d = d0 + 16 * k + 4 * g + i;
            if (d < D && col < V) st[(size_t)d * V + col] = S[k][i];
        }
}

// grid (T, groups of heads): a wave per head; the convolutions' inputs of a sequence's last tokens go to the tail (read by the
// launches before)
template <ActType ACT>
__global__ __launch_bounds__(256) void gated_norm_kernel(const GatedStateArgs a, int T) {
    const int t = blockIdx.x, tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, V = a.vdim, n = a.heads * V;
    const float *o = a.o + (size_t)t * n, *x = a.in + (size_t)t * a.ld;
    const size_t to = (size_t)t * a.ld_out;
    auto put = [&](int i, float y) {
        if constexpr (ACT == ACT_BF16) static_cast<uint16_t *>(a.out)[to + i] = f32_to_bf16_bits(y);
        else static_cast<float *>(a.out)[to + i] = y;
    };
    for (int h = blockIdx.y * 4 + wave; h < a.heads; h += 4 * gridDim.y) {
        float ss = 0.f, v[STATE_DIM_MAX / 64], gate[STATE_DIM_MAX / 64];
#pragma unroll
        for (int k = 0; k < STATE_DIM_MAX / 64; ++k) {
            const int i = lane + 64 * k;
            v[k] = i < V ? o[h * V + i] : 0.f;
            gate[k] = i < V ? x[a.at_g + h * V + i] : 0.f;
            ss = fmaf(v[k], v[k], ss);
        }
        const float r = 1.0f / sqrtf(gs_wave_sum(ss) / (float)V + a.eps);
#pragma unroll
        for (int k = 0; k < STATE_DIM_MAX / 64; ++k) {
            const int i = lane + 64 * k;
            if (i < V) put(h * V + i, v[k] * r * a.norm[i] * act_silu(gate[k]));
        }
    }
    if (blockIdx.y == 0)
        for (int i = n + tid; i < a.ld_out; i += 256) put(i, 0.f);
    if (a.delta && a.taps > 1 && (t + a.taps - 1 >= T || a.seq[t + a.taps - 1] != a.seq[t])) {
        const int qk = a.kv_heads * a.dim, channels = 2 * qk + n;
        float *slot = a.tail + ((size_t)a.seq[t] * a.taps + a.pos[t] % a.taps) * channels;
        for (int i = blockIdx.y * 256 + tid; i < channels; i += 256 * gridDim.y) slot[i] = x[i < qk ? a.at_q + i : i < 2 * qk ? a.at_k + i - qk : a.at_v + i - 2 * qk];
    }
}

// ------------------------------------------------------------------------------------------------ host
static bool args_ok(const GatedStateArgs &a) {
    return a.heads >= 1 && a.kv_heads >= 1 && a.heads % a.kv_heads == 0 && a.dim >= 1 && a.vdim >= 1 && gated_state_supported(a.dim, a.vdim) && a.in && a.norm && a.state && a.pos &&
           a.seq && a.out && a.ld_out >= a.heads * a.vdim &&
           (a.delta ? a.taps >= 1 && a.tail && a.conv_q && a.conv_k && a.conv_v && a.A && a.dt_bias : a.kv_heads == a.heads && a.rank >= 1 && a.rank <= STATE_RANK_MAX && a.a2 && a.a2_bias);
}

int gated_state_step(const GatedStateArgs &a, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!args_ok(a) || T > 65535) return fail(MESH_ERR_INVALID, "gated_state_step: bad operands");
    int vt = 16;
    while (vt < a.vdim) vt *= 2;
    const dim3 grid((unsigned)a.heads, (unsigned)T);
    const int rows512 = (a.dim + 512 / vt - 1) / (512 / vt);
    if (rows512 <= 4) MESH_LAUNCH((gated_step_kernel<512, 4>), grid, dim3(512), 0, stream, a, vt);
    else if (rows512 <= 8) MESH_LAUNCH((gated_step_kernel<512, 8>), grid, dim3(512), 0, stream, a, vt);
    else if (rows512 <= 16) MESH_LAUNCH((gated_step_kernel<512, 16>), grid, dim3(512), 0, stream, a, vt);
    else if (rows512 <= 32) MESH_LAUNCH((gated_step_kernel<512, 32>), grid, dim3(512), 0, stream, a, vt);
    else MESH_LAUNCH((gated_step_kernel<1024, 64>), grid, dim3(1024), 0, stream, a, vt);         // (up to 256 x 256)
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

template <bool DELTA>
static int launch_scan(const GatedStateArgs &a, hipStream_t stream) {
    const dim3 grid((unsigned)a.heads, (unsigned)(gs_pad16(a.vdim) / 16), (unsigned)a.chunks.n_runs), block(256);
    switch (gs_pad64(a.dim) / 64) {
        case 1: MESH_LAUNCH((state_scan_kernel<DELTA, 1>), grid, block, 0, stream, a); break;
        case 2: MESH_LAUNCH((state_scan_kernel<DELTA, 2>), grid, block, 0, stream, a); break;
        case 3: MESH_LAUNCH((state_scan_kernel<DELTA, 3>), grid, block, 0, stream, a); break;
        default: MESH_LAUNCH((state_scan_kernel<DELTA, 4>), grid, block, 0, stream, a); break;
    }
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int gated_state_chunks(const GatedStateArgs &a, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    const StateChunks &ch = a.chunks;
    if (!args_ok(a) || !a.ws || !a.o || !ch.chunk || !ch.first || !ch.run || ch.n_chunks < 1 || ch.n_runs < 1 || ch.n_runs > 65535 || a.heads > 65535)
        return fail(MESH_ERR_INVALID, "gated_state_chunks: bad operands");
    const dim3 grid((unsigned)ch.n_chunks, (unsigned)a.heads), block(PREP_THREADS);
    const size_t lds = a.delta ? delta_prepare_lds(a.dim, a.vdim) : gla_prepare_lds(a.dim, a.rank);
    static bool ready = false;        // (hosts are single-threaded per session; a second thread sets the same attributes)
    if (!ready) {
        MESH_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(delta_prepare_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)delta_prepare_lds(STATE_DIM_MAX, STATE_DIM_MAX)));
        MESH_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(gla_prepare_kernel), hipFuncAttributeMaxDynamicSharedMemorySize, (int)gla_prepare_lds(STATE_DIM_MAX, STATE_RANK_MAX)));
        ready = true;
    }
    if (a.delta) MESH_LAUNCH(delta_prepare_kernel, grid, block, lds, stream, a);
    else MESH_LAUNCH(gla_prepare_kernel, grid, block, lds, stream, a);
    MESH_LAUNCH_CHECK();
    const int rc = a.delta ? launch_scan<true>(a, stream) : launch_scan<false>(a, stream);
    if (rc != MESH_OK) return rc;
    const dim3 norm_grid((unsigned)T, (unsigned)((a.heads + 7) / 8));          // two heads per wave
    if (a.act == ACT_BF16) MESH_LAUNCH((gated_norm_kernel<ACT_BF16>), norm_grid, dim3(256), 0, stream, a, T);
    else MESH_LAUNCH((gated_norm_kernel<ACT_F32>), norm_grid, dim3(256), 0, stream, a, T);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

}  // namespace mesh
