// The single-token product: y = W x for a bf16 matrix and one f32 vector, bound by the weight stream.
//
// A wave takes R rows at a time; its 64 lanes cover 512 consecutive k per 16-byte load and R * U loads are in flight while
// the R * U before them are multiplied.  The input vector sits in LDS as f32.  Every workgroup derives it itself from what
// the launch before left (residual update with its output norm, polynomial activation: linear.hpp), which saves a launch
// between two products; the first weight loads go out before that work and travel behind it.  Sums of squares a later norm
// needs are left per workgroup and added in workgroup order by the consumer, so the result does not depend on timing.
#include "act_math.hpp"
#include "linear.hpp"

#include <algorithm>

namespace mesh {

constexpr int STEP_THREADS = 512, STEP_WAVES = STEP_THREADS / 64;
constexpr size_t STEP_LDS_MAX = 160 * 1024 - 1024;

// over the wave, in every lane: data-parallel-primitive moves inside a row of 16 lanes (swap neighbours, swap pairs, mirror the
// 8, mirror the 16), permutes across rows
__device__ __forceinline__ float step_wave_sum(float v) {
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0xB1, 0xF, 0xF, false));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x4E, 0xF, 0xF, false));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x141, 0xF, 0xF, false));
    v += __int_as_float(__builtin_amdgcn_update_dpp(0, __float_as_int(v), 0x140, 0xF, 0xF, false));
    v += __shfl_xor(v, 16);
    v += __shfl_xor(v, 32);
    return v;
}
// sum over the workgroup in a fixed order, the same in every thread
__device__ __forceinline__ float step_block_sum(float v, float *scratch, int lane, int wave) {
    v = step_wave_sum(v);
    __syncthreads();
    if (lane == 0) scratch[wave] = v;
    __syncthreads();
    float s = 0.f;
#pragma unroll
    for (int w = 0; w < STEP_WAVES; ++w) s += scratch[w];
    return s;
}

// four elements of a vector of K, zeros behind its end
__device__ __forceinline__ float4 ln_load4(const float *p, int k, int K) {
    if (k + 4 <= K) return *reinterpret_cast<const float4 *>(p + k);
    return make_float4(k < K ? p[k] : 0.f, k + 1 < K ? p[k + 1] : 0.f, k + 2 < K ? p[k + 2] : 0.f, 0.f);
}
// xs[k .. k + 3] = map(k, load(k)) over [0, Kp), four loads of a thread in flight
template <typename Load, typename Map>
__device__ __forceinline__ void step_vec(int K, int Kp, int tid, Load load, Map map, float *xs) {
    constexpr int N = 4;
    for (int k0 = tid * 4; k0 < Kp; k0 += N * STEP_THREADS * 4) {
        float4 v[N];
#pragma unroll
        for (int i = 0; i < N; ++i) v[i] = load(k0 + i * STEP_THREADS * 4);
#pragma unroll
        for (int i = 0; i < N; ++i) {
            const int k = k0 + i * STEP_THREADS * 4;
            if (k < Kp) *reinterpret_cast<float4 *>(xs + k) = map(k, v[i]);
        }
    }
}

template <int R, int U, StepIn IN, StepOut OUT>
__global__ __launch_bounds__(STEP_THREADS) void linear_step_kernel(const uint16_t *p_w, int p_Kp, int p_groups, int p_width, int p_K, const StepArgs a) {
    extern __shared__ __align__(16) uint8_t smem[];
    __shared__ float scratch[STEP_WAVES][4];
    float *xs = reinterpret_cast<float *>(smem);
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6;
    const int K = p_K, Kp = p_Kp;
    const int batches = (Kp + 512 * U - 1) / (512 * U);
    const int g_step = gridDim.x * STEP_WAVES;
    int grp = blockIdx.x * STEP_WAVES + wave, batch = 0;
    auto row_of = [&](int gr, int r) { return OUT == STEP_OUT_MIN_GRU ? r * p_width + gr : gr * R + r; };
    auto fetch = [&](uint4 (&b)[R][U], int gr, int bt) {
#pragma unroll
        for (int r = 0; r < R; ++r) {
            const uint16_t *wr = p_w + (size_t)row_of(gr, r) * Kp;
#pragma unroll
            for (int u = 0; u < U; ++u) {
                const int k = (bt * U + u) * 512 + lane * 8;
                b[r][u] = make_uint4(0, 0, 0, 0);
                if (k < Kp) b[r][u] = *reinterpret_cast<const uint4 *>(wr + k);
            }
        }
    };
    uint4 b0[R][U], b1[R][U];
    if (grp < p_groups) fetch(b0, grp, 0);

    // ---- the input vector
    if constexpr (IN == STEP_IN_VEC) {
        step_vec(K, Kp, tid, [&](int k) { return ln_load4(a.in, k, K); }, [&](int k, const float4 &v) { return v; }, xs);
    } else if constexpr (IN == STEP_IN_POLY) {
        float p2 = 0.f, p4 = 0.f, p6 = 0.f;
        for (int i = tid; i < a.n_part; i += STEP_THREADS) { p2 += a.part[i]; p4 += a.part[a.n_part + i]; p6 += a.part[2 * a.n_part + i]; }
        p2 = step_block_sum(p2, &scratch[0][0], lane, wave);
        p4 = step_block_sum(p4, &scratch[0][0], lane, wave);
        p6 = step_block_sum(p6, &scratch[0][0], lane, wave);
        const float c1 = a.coef[0] / sqrtf(p2 / (float)K + a.eps), c2 = a.coef[1] / sqrtf(p4 / (float)K + a.eps), c3 = a.coef[2] / sqrtf(p6 / (float)K + a.eps);
        const float c0 = a.coef[3];
        auto poly = [&](float u) { return ((c3 * u + c2) * u + c1) * u + c0; };
        step_vec(K, Kp, tid, [&](int k) { return ln_load4(a.in, k, K); },
                 [&](int k, const float4 &u) {
                     return make_float4(k < K ? poly(u.x) : 0.f, k + 1 < K ? poly(u.y) : 0.f, k + 2 < K ? poly(u.z) : 0.f, k + 3 < K ? poly(u.w) : 0.f);
                 }, xs);
    } else if constexpr (IN == STEP_IN_RELU2) {
        auto sq = [](float v) { const float p = fmaxf(v, 0.f); return p * p; };
        step_vec(K, Kp, tid, [&](int k) { return ln_load4(a.in, k, K); }, [&](int k, const float4 &v) { return make_float4(sq(v.x), sq(v.y), sq(v.z), sq(v.w)); }, xs);
    } else if constexpr (IN == STEP_IN_UNIT_RMS) {
        float ss = 0.f;
        step_vec(K, Kp, tid, [&](int k) { return ln_load4(a.in, k, K); },
                 [&](int k, const float4 &v) { ss += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w; return v; }, xs);
        const float rinv = 1.0f / sqrtf(step_block_sum(ss, &scratch[0][0], lane, wave) / (float)K + a.eps);
        for (int k = tid; k < K; k += STEP_THREADS) xs[k] *= rinv * a.gain[k];
    } else if constexpr (IN == STEP_IN_LAYER) {
        // a thread's first AHEAD groups of four, of every vector, are requested before the first sum; means first, then squared
        // deviations
        constexpr int AHEAD = 2, STRIDE = STEP_THREADS * 4;
        const int k0 = tid * 4;
        const float inv_n = 1.0f / (float)K;
        float4 x4[AHEAD], y4[AHEAD], g4[AHEAD], b4[AHEAD], ng4[AHEAD], nb4[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            const int k = k0 + i * STRIDE;
            x4[i] = ln_load4(a.in, k, K);
            if (a.y) { y4[i] = ln_load4(a.y, k, K); g4[i] = ln_load4(a.gain, k, K); b4[i] = ln_load4(a.bias, k, K); }
            ng4[i] = ln_load4(a.norm_gain, k, K); nb4[i] = ln_load4(a.norm_bias, k, K);
        }
        auto sum4 = [](const float4 &v) { return (v.x + v.y) + (v.z + v.w); };
        auto dev4 = [&](int k, const float4 &v, float mean) {
            const float d[4] = {v.x - mean, v.y - mean, v.z - mean, v.w - mean};
            float s = 0.f;
#pragma unroll
            for (int j = 0; j < 4; ++j) s = fmaf(k + j < K ? d[j] : 0.f, d[j], s);
            return s;
        };
        if (a.y) {
            float s = 0.f;
#pragma unroll
            for (int i = 0; i < AHEAD; ++i) s += sum4(y4[i]);
            for (int k = k0 + AHEAD * STRIDE; k < K; k += STRIDE) s += sum4(ln_load4(a.y, k, K));
            const float mean = step_block_sum(s, &scratch[0][0], lane, wave) * inv_n;
            s = 0.f;
#pragma unroll
            for (int i = 0; i < AHEAD; ++i) s += dev4(k0 + i * STRIDE, y4[i], mean);
            for (int k = k0 + AHEAD * STRIDE; k < K; k += STRIDE) s += dev4(k, ln_load4(a.y, k, K), mean);
            const float rs = 1.0f / sqrtf(step_block_sum(s, &scratch[0][0], lane, wave) * inv_n + a.eps);
            auto update = [&](int k, const float4 &x, const float4 &y, const float4 &g, const float4 &b) {
                const float4 v = make_float4(x.x + ((y.x - mean) * rs * g.x + b.x), x.y + ((y.y - mean) * rs * g.y + b.y), x.z + ((y.z - mean) * rs * g.z + b.z),
                                             x.w + ((y.w - mean) * rs * g.w + b.w));
                if (blockIdx.x == 0) {
                    const float o[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
                    for (int j = 0; j < 4; ++j)
                        if (k + j < K) a.x_out[k + j] = o[j];
                }
                return v;
            };
#pragma unroll
            for (int i = 0; i < AHEAD; ++i) x4[i] = update(k0 + i * STRIDE, x4[i], y4[i], g4[i], b4[i]);
            for (int k = k0 + AHEAD * STRIDE; k < Kp; k += STRIDE)
                *reinterpret_cast<float4 *>(xs + k) = update(k, ln_load4(a.in, k, K), ln_load4(a.y, k, K), ln_load4(a.gain, k, K), ln_load4(a.bias, k, K));
        } else {
            for (int k = k0 + AHEAD * STRIDE; k < Kp; k += STRIDE) *reinterpret_cast<float4 *>(xs + k) = ln_load4(a.in, k, K);
        }
        // (groups behind the first AHEAD wait in LDS, every thread's its own)
        float s = 0.f;
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) s += sum4(x4[i]);
        for (int k = k0 + AHEAD * STRIDE; k < Kp; k += STRIDE) s += sum4(*reinterpret_cast<const float4 *>(xs + k));
        const float mean = step_block_sum(s, &scratch[0][0], lane, wave) * inv_n;
        s = 0.f;
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) s += dev4(k0 + i * STRIDE, x4[i], mean);
        for (int k = k0 + AHEAD * STRIDE; k < Kp; k += STRIDE) s += dev4(k, *reinterpret_cast<const float4 *>(xs + k), mean);
        const float rs = 1.0f / sqrtf(step_block_sum(s, &scratch[0][0], lane, wave) * inv_n + a.eps);
        auto put = [&](int k, const float4 &v, const float4 &g, const float4 &b) {
            if (k < Kp) *reinterpret_cast<float4 *>(xs + k) = make_float4((v.x - mean) * rs * g.x + b.x, (v.y - mean) * rs * g.y + b.y, (v.z - mean) * rs * g.z + b.z, (v.w - mean) * rs * g.w + b.w);
        };
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) put(k0 + i * STRIDE, x4[i], ng4[i], nb4[i]);
        for (int k = k0 + AHEAD * STRIDE; k < Kp; k += STRIDE) put(k, *reinterpret_cast<const float4 *>(xs + k), ln_load4(a.norm_gain, k, K), ln_load4(a.norm_bias, k, K));
    } else {
        float ss = 0.f;
        for (int i = tid; i < a.n_part; i += STEP_THREADS) ss += a.part[i];
        // the vectors' loads go out before the partial sums are added up
        constexpr int AHEAD = 2;
        float4 x4[AHEAD], y4[AHEAD], g4[AHEAD];
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) {
            const int k = (tid + i * STEP_THREADS) * 4;
            x4[i] = ln_load4(a.in, k, K); y4[i] = ln_load4(a.y, k, K); g4[i] = ln_load4(a.gain, k, K);
        }
        ss = step_block_sum(ss, &scratch[0][0], lane, wave);
        const float rinv = 1.0f / sqrtf(ss / (float)K + a.eps);
        float sx = 0.f;
        auto update = [&](int k, const float4 &x, const float4 &y, const float4 &g) {
            if (k >= Kp) return;
            const float4 v = make_float4(x.x + y.x * rinv * g.x, x.y + y.y * rinv * g.y, x.z + y.z * rinv * g.z, x.w + y.w * rinv * g.w);
            *reinterpret_cast<float4 *>(xs + k) = v;
            sx += v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
            if (blockIdx.x == 0) {
                const float o[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
                for (int j = 0; j < 4; ++j)
                    if (k + j < K) a.x_out[k + j] = o[j];
            }
        };
#pragma unroll
        for (int i = 0; i < AHEAD; ++i) update((tid + i * STEP_THREADS) * 4, x4[i], y4[i], g4[i]);
        for (int k = (tid + AHEAD * STEP_THREADS) * 4; k < Kp; k += STEP_THREADS * 4) update(k, ln_load4(a.in, k, K), ln_load4(a.y, k, K), ln_load4(a.gain, k, K));
        if constexpr (IN == STEP_IN_RESIDUAL_NORM) {
            sx = step_block_sum(sx, &scratch[0][0], lane, wave);
            const float z = a.norm_gain[0] / sqrtf(sx / (float)K + a.eps);
            for (int k = tid; k < Kp; k += STEP_THREADS) xs[k] *= z;
        }
    }
    __syncthreads();

    // ---- rows
    float acc[R], s2 = 0.f, s4 = 0.f, s6 = 0.f;
#pragma unroll
    for (int r = 0; r < R; ++r) acc[r] = 0.f;
    auto finish = [&](int gr) {
        float v[R];
#pragma unroll
        for (int r = 0; r < R; ++r) { v[r] = step_wave_sum(acc[r]); acc[r] = 0.f; }
        if constexpr (OUT == STEP_OUT_MIN_GRU) {
            if (lane == 0) {
                const MinGruGate g = min_gru_gate(v[0] + a.bias_z[gr], v[1] + a.bias_x[gr]);
                float *st = a.state + (size_t)a.seq[0] * p_width + gr;
                const float s = a.pos[0] == 0 ? g.in : fmaf(g.keep, *st, g.in);
                *st = s;
                a.out[gr] = s * act_silu(v[2]);
            }
        } else {
#pragma unroll
            for (int r = 0; r < R; ++r) {
                const int m = gr * R + r;
                if (m >= a.W.M) continue;
                float o = v[r];
                if constexpr (OUT == STEP_OUT_SIDE) {
                    const float e = bf16_bits_to_f32(a.side[(size_t)a.tok[0] * a.side_stride + a.side_offset + m]);
                    o = act_gelu_tanh(o) * e;
                }
                if (lane == 0) a.out[m] = o;
                const float q = o * o;
                if constexpr (OUT == STEP_OUT_SUMSQ || OUT == STEP_OUT_POWERS) s2 += q;
                if constexpr (OUT == STEP_OUT_POWERS) { s4 += q * q; s6 += q * q * q; }
            }
        }
    };
    auto use = [&](const uint4 (&b)[R][U], int bt) {
#pragma unroll
        for (int u = 0; u < U; ++u) {
            const int k = (bt * U + u) * 512 + lane * 8;
            if (k < Kp) {
                const float4 xa = *reinterpret_cast<const float4 *>(xs + k), xb = *reinterpret_cast<const float4 *>(xs + k + 4);
                const float xf[8] = {xa.x, xa.y, xa.z, xa.w, xb.x, xb.y, xb.z, xb.w};
#pragma unroll
                for (int r = 0; r < R; ++r) {
                    const uint32_t w[4] = {b[r][u].x, b[r][u].y, b[r][u].z, b[r][u].w};
#pragma unroll
                    for (int j = 0; j < 8; ++j) acc[r] = fmaf(__uint_as_float((j & 1) ? (w[j >> 1] & 0xFFFF0000u) : (w[j >> 1] << 16)), xf[j], acc[r]);
                }
            }
        }
    };
    // (group, batch) pairs in order; each is fetched while the one before it is used
    auto step = [&](uint4 (&cur)[R][U], uint4 (&next)[R][U]) {
        const int gr = grp, bt = batch;
        if (++batch == batches) { batch = 0; grp += g_step; }
        if (grp < p_groups) fetch(next, grp, batch);
        use(cur, bt);
        if (bt == batches - 1) finish(gr);
    };
    while (grp < p_groups) {
        step(b0, b1);
        if (grp >= p_groups) break;
        step(b1, b0);
    }
    if constexpr (OUT == STEP_OUT_SUMSQ || OUT == STEP_OUT_POWERS) {
        // (every lane of a wave holds the wave's sums)
        __syncthreads();
        if (lane == 0) { scratch[wave][0] = s2; scratch[wave][1] = s4; scratch[wave][2] = s6; }
        __syncthreads();
        if (tid < (OUT == STEP_OUT_POWERS ? 3 : 1)) {
            float s = 0.f;
            for (int w = 0; w < STEP_WAVES; ++w) s += scratch[w][tid];
            a.out_part[(size_t)tid * gridDim.x + blockIdx.x] = s;
        }
    }
}

bool linear_step_supported(const LinearWeight &W) { return (size_t)W.Kp * sizeof(float) <= STEP_LDS_MAX; }

static int rows_per_group(const StepArgs &a) { return a.out_kind == STEP_OUT_MIN_GRU ? 3 : a.W.M < 4096 ? 1 : 2; }
static int step_groups(const StepArgs &a) { return a.out_kind == STEP_OUT_MIN_GRU ? a.width : (a.W.M + rows_per_group(a) - 1) / rows_per_group(a); }

int linear_step_grid(const StepArgs &a) {
    // as many workgroups as the chip holds at once, two per CU; more rows mean more turns per wave, equally many for all
    const int wgs = (step_groups(a) + STEP_WAVES - 1) / STEP_WAVES;
    const int turns = (wgs + STEP_PARTS_MAX - 1) / STEP_PARTS_MAX;
    return (wgs + turns - 1) / turns;
}

template <int R, int U, StepIn IN, StepOut OUT>
static int launch_step(const StepArgs &a, hipStream_t stream) {
    const size_t lds = (size_t)a.W.Kp * sizeof(float);
    static bool ready = false;        // (hosts are single-threaded per session; a second thread sets the same attribute)
    if (!ready) {
        MESH_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(linear_step_kernel<R, U, IN, OUT>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)STEP_LDS_MAX));
        ready = true;
    }
    MESH_LAUNCH((linear_step_kernel<R, U, IN, OUT>), dim3((unsigned)linear_step_grid(a)), dim3(STEP_THREADS), lds, stream, a.W.w, a.W.Kp, step_groups(a), a.width, a.W.K, a);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}
template <StepIn IN, StepOut OUT>
static int launch_step_rows(const StepArgs &a, hipStream_t stream) {
    return rows_per_group(a) == 1 ? launch_step<1, 4, IN, OUT>(a, stream) : launch_step<2, 4, IN, OUT>(a, stream);
}

int linear_step(const StepArgs &a, hipStream_t stream) {
    const LinearWeight &W = a.W;
    if (!W.w || !a.in || !a.out || W.M < 1 || W.Kp % LINEAR_K_PAD || W.Kp < W.K || W.Mp < W.M || !linear_step_supported(W))
        return fail(MESH_ERR_INVALID, "linear_step: bad operands (%d x %d)", W.M, W.K);
    const bool resid = a.in_kind == STEP_IN_RESIDUAL || a.in_kind == STEP_IN_RESIDUAL_NORM;
    if ((resid && (!a.y || !a.gain || !a.part || !a.x_out || a.x_out == a.in || a.n_part < 1 || a.n_part > STEP_PARTS_MAX)) ||
        (a.in_kind == STEP_IN_RESIDUAL_NORM && !a.norm_gain) || (a.in_kind == STEP_IN_POLY && (!a.part || !a.coef || a.n_part < 1 || a.n_part > STEP_PARTS_MAX)))
        return fail(MESH_ERR_INVALID, "linear_step: input description incomplete");
    if ((a.in_kind == STEP_IN_LAYER && (!a.norm_gain || !a.norm_bias || (a.y && (!a.gain || !a.bias || !a.x_out || a.x_out == a.in)))) || (a.in_kind == STEP_IN_UNIT_RMS && !a.gain))
        return fail(MESH_ERR_INVALID, "linear_step: input description incomplete");
    if (((a.out_kind == STEP_OUT_SUMSQ || a.out_kind == STEP_OUT_POWERS) && !a.out_part) ||
        (a.out_kind == STEP_OUT_MIN_GRU && (!a.state || !a.pos || !a.seq || !a.bias_z || !a.bias_x || a.width < 1 || W.M != 3 * a.width)) ||
        (a.out_kind == STEP_OUT_SIDE && (!a.side || !a.tok)))
        return fail(MESH_ERR_INVALID, "linear_step: output description incomplete");
#define MESH_STEP_CASE(IN, OUT) \
    if (a.in_kind == IN && a.out_kind == OUT) return launch_step_rows<IN, OUT>(a, stream);
    MESH_STEP_CASE(STEP_IN_VEC, STEP_OUT_PLAIN)
    MESH_STEP_CASE(STEP_IN_RESIDUAL, STEP_OUT_PLAIN)
    MESH_STEP_CASE(STEP_IN_RESIDUAL_NORM, STEP_OUT_PLAIN)
    MESH_STEP_CASE(STEP_IN_LAYER, STEP_OUT_PLAIN)
    MESH_STEP_CASE(STEP_IN_UNIT_RMS, STEP_OUT_PLAIN)
    MESH_STEP_CASE(STEP_IN_RELU2, STEP_OUT_PLAIN)
    MESH_STEP_CASE(STEP_IN_VEC, STEP_OUT_SUMSQ)
    MESH_STEP_CASE(STEP_IN_POLY, STEP_OUT_SUMSQ)
    MESH_STEP_CASE(STEP_IN_RESIDUAL, STEP_OUT_POWERS)
    MESH_STEP_CASE(STEP_IN_RESIDUAL, STEP_OUT_SIDE)
#undef MESH_STEP_CASE
    if (a.in_kind == STEP_IN_VEC && a.out_kind == STEP_OUT_MIN_GRU) return launch_step<3, 2, STEP_IN_VEC, STEP_OUT_MIN_GRU>(a, stream);
    if (a.in_kind == STEP_IN_RESIDUAL && a.out_kind == STEP_OUT_MIN_GRU) return launch_step<3, 2, STEP_IN_RESIDUAL, STEP_OUT_MIN_GRU>(a, stream);
    return fail(MESH_ERR_UNSUPPORTED, "linear_step: no kernel for input %d with output %d", (int)a.in_kind, (int)a.out_kind);
}

}  // namespace mesh
