// See rowops.hpp.  One workgroup per token row; sums of squares in f32.
#include "rowops.hpp"

#include "kv_cache.hpp"

namespace mesh {

constexpr int ROW_THREADS = 256, ROW_WAVES = ROW_THREADS / 64;

template <ActType ACT> __device__ __forceinline__ void act_store(void *out, size_t i, float v) {
    if constexpr (ACT == ACT_BF16) static_cast<uint16_t *>(out)[i] = f32_to_bf16_bits(v);
    else static_cast<float *>(out)[i] = v;
}

__device__ __forceinline__ float row_sum(float v, float *scratch) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

__global__ __launch_bounds__(ROW_THREADS) void embed_rows_kernel(const uint16_t *table, const int32_t *tok, const int32_t *pos, const float *freq, float scale,
                                                                 int n, float *x) {
    const int t = blockIdx.x;
    const uint16_t *e = table + (size_t)tok[t] * n;
    const float p = (float)pos[t];
    for (int i = threadIdx.x; i < n; i += ROW_THREADS) {
        const float angle = p * freq[i >> 1];
        x[(size_t)t * n + i] = bf16_bits_to_f32(e[i]) * scale + ((i & 1) ? cosf(angle) : sinf(angle));
    }
}

template <ActType ACT>
__global__ __launch_bounds__(ROW_THREADS) void residual_norm_kernel(float *x, const float *y, const float *gain, float eps, int n, void *out, int ld) {
    __shared__ float scratch[ROW_WAVES];
    const size_t at = (size_t)blockIdx.x * n, to = (size_t)blockIdx.x * ld;
    float rinv = 0.f;
    if (y) {
        float ss = 0.f;
        for (int i = threadIdx.x; i < n; i += ROW_THREADS) ss = fmaf(y[at + i], y[at + i], ss);
        rinv = 1.0f / sqrtf(row_sum(ss, scratch) / (float)n + eps);
    }
    for (int i = threadIdx.x; i < ld; i += ROW_THREADS) {
        float v = 0.f;
        if (i < n) {
            v = x[at + i];
            if (y) {
                v = v + y[at + i] * rinv * gain[i];
                x[at + i] = v;
            }
        }
        act_store<ACT>(out, to + i, v);
    }
}

template <ActType ACT>
__global__ __launch_bounds__(ROW_THREADS) void scalar_norm_kernel(const float *x, const int32_t *row, const float *gain, float eps, int n, void *out, int ld) {
    __shared__ float scratch[ROW_WAVES];
    const size_t at = (size_t)(row ? row[blockIdx.x] : (int)blockIdx.x) * n, to = (size_t)blockIdx.x * ld;
    float ss = 0.f;
    for (int i = threadIdx.x; i < n; i += ROW_THREADS) ss = fmaf(x[at + i], x[at + i], ss);
    const float z = gain[0] / sqrtf(row_sum(ss, scratch) / (float)n + eps);
    for (int i = threadIdx.x; i < ld; i += ROW_THREADS) act_store<ACT>(out, to + i, i < n ? x[at + i] * z : 0.f);
}

template <ActType ACT>
__global__ __launch_bounds__(ROW_THREADS) void poly_norm_kernel(const float *u, const float *coef, float eps, int n, void *out, int ld) {
    __shared__ float scratch[ROW_WAVES];
    const size_t at = (size_t)blockIdx.x * n, to = (size_t)blockIdx.x * ld;
    float p2 = 0.f, p4 = 0.f, p6 = 0.f;
    for (int i = threadIdx.x; i < n; i += ROW_THREADS) {
        const float q = u[at + i] * u[at + i];
        p2 += q; p4 += q * q; p6 += q * q * q;
    }
    p2 = row_sum(p2, scratch); p4 = row_sum(p4, scratch); p6 = row_sum(p6, scratch);
    const float c1 = coef[0] / sqrtf(p2 / (float)n + eps), c2 = coef[1] / sqrtf(p4 / (float)n + eps), c3 = coef[2] / sqrtf(p6 / (float)n + eps), c0 = coef[3];
    for (int i = threadIdx.x; i < ld; i += ROW_THREADS) {
        const float v = i < n ? u[at + i] : 0.f;
        act_store<ACT>(out, to + i, i < n ? ((c3 * v + c2) * v + c1) * v + c0 : 0.f);
    }
}

template <ActType ACT>
__global__ __launch_bounds__(64) void side_gate_kernel(const float *g, const uint16_t *side, const int32_t *tok, int stride, int offset, int n, void *out, int ld) {
    const int t = blockIdx.x;
    const uint16_t *e = side + (size_t)tok[t] * stride + offset;
    for (int i = threadIdx.x; i < ld; i += 64) {
        float v = 0.f;
        if (i < n) {
            const float z = g[(size_t)t * n + i];
            v = 0.5f * z * (1.0f + tanhf(0.7978845608028654f * (z + 0.044715f * z * z * z))) * bf16_bits_to_f32(e[i]);
        }
        act_store<ACT>(out, (size_t)t * ld + i, v);
    }
}

__device__ __forceinline__ void append_value(uint8_t *cache, int type, size_t at, float v, unsigned *sat) {
    if (type == MESH_F32) { reinterpret_cast<float *>(cache)[at] = v; return; }
    note_f16_clamp(sat, v, 0.f);
    reinterpret_cast<uint16_t *>(cache)[at] = f32_to_f16_bits(fminf(fmaxf(v, -65504.f), 65504.f));
}

// grid (slices of the heads, T); every workgroup sums the whole row itself, so that slices need not meet
__global__ __launch_bounds__(ROW_THREADS) void qk_norm_append_kernel(const QkAppendArgs a) {
    __shared__ float scratch[ROW_WAVES];
    const int t = blockIdx.y, nq = a.n_head * a.hd, nk = a.n_kv * a.hd;
    const float *row = a.qk + (size_t)t * (nq + nk);
    float sq = 0.f, sk = 0.f;
    for (int i = threadIdx.x; i < nq; i += ROW_THREADS) sq = fmaf(row[i], row[i], sq);
    for (int i = threadIdx.x; i < nk; i += ROW_THREADS) sk = fmaf(row[nq + i], row[nq + i], sk);
    const float rq = 1.0f / sqrtf(row_sum(sq, scratch) / (float)(a.n_head * a.dim) + a.eps);
    const float rk = 1.0f / sqrtf(row_sum(sk, scratch) / (float)(a.n_kv * a.dim) + a.eps);
    const int pos = a.pos[t], seq = a.seq[t];
    const int stride = gridDim.x * ROW_THREADS, first = blockIdx.x * ROW_THREADS + threadIdx.x;
    for (int i = first; i < nq; i += stride) a.q[(size_t)t * nq + i] = row[i] * rq * a.q_norm[i];
    for (int i = first; i < nk; i += stride) {
        const int head = i / a.hd, d = i - head * a.hd;
        const size_t at = (((size_t)seq * a.n_kv + head) * a.n_ctx + pos) * a.hd + d;
        const float v = row[nq + i];
        append_value(a.kcache, a.kv_type, at, v * rk * a.k_norm[i], a.sat);
        append_value(a.vcache, a.kv_type, at, v, a.sat);
    }
}

#define MESH_ACT_LAUNCH(kernel, act, grid, block, ...)                                                     \
    do {                                                                                                   \
        if (act == ACT_BF16) MESH_LAUNCH((kernel<ACT_BF16>), grid, block, 0, stream, __VA_ARGS__);         \
        else MESH_LAUNCH((kernel<ACT_F32>), grid, block, 0, stream, __VA_ARGS__);                          \
        MESH_LAUNCH_CHECK();                                                                               \
    } while (0)

int embed_rows(const uint16_t *table, const int32_t *tok, const int32_t *pos, const float *freq, float scale, int T, int n, float *x, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    MESH_LAUNCH(embed_rows_kernel, dim3((unsigned)T), dim3(ROW_THREADS), 0, stream, table, tok, pos, freq, scale, n, x);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int residual_norm_rows(float *x, const float *y, const float *gain, float eps, int T, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (ld < n || (y && !gain)) return fail(MESH_ERR_INVALID, "residual_norm_rows: bad operands");
    MESH_ACT_LAUNCH(residual_norm_kernel, act, dim3((unsigned)T), dim3(ROW_THREADS), x, y, gain, eps, n, out, ld);
    return MESH_OK;
}

int scalar_norm_rows(const float *x, const int32_t *row, const float *gain, float eps, int n_rows, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (n_rows <= 0) return MESH_OK;
    if (ld < n) return fail(MESH_ERR_INVALID, "scalar_norm_rows: bad operands");
    MESH_ACT_LAUNCH(scalar_norm_kernel, act, dim3((unsigned)n_rows), dim3(ROW_THREADS), x, row, gain, eps, n, out, ld);
    return MESH_OK;
}

int poly_norm_rows(const float *u, const float *coef, float eps, int T, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (ld < n) return fail(MESH_ERR_INVALID, "poly_norm_rows: bad operands");
    MESH_ACT_LAUNCH(poly_norm_kernel, act, dim3((unsigned)T), dim3(ROW_THREADS), u, coef, eps, n, out, ld);
    return MESH_OK;
}

int side_gate_rows(const float *g, const uint16_t *side, const int32_t *tok, int stride, int offset, int T, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (ld < n || offset + n > stride) return fail(MESH_ERR_INVALID, "side_gate_rows: bad operands");
    MESH_ACT_LAUNCH(side_gate_kernel, act, dim3((unsigned)T), dim3(64), g, side, tok, stride, offset, n, out, ld);
    return MESH_OK;
}

int qk_norm_append(const QkAppendArgs &a, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if ((a.kv_type != MESH_F16 && a.kv_type != MESH_F32) || a.dim > a.hd || T > 65535 || a.n_head < 1 || a.n_kv < 1)
        return fail(MESH_ERR_INVALID, "qk_norm_append: bad operands");
    // a few tokens: spread a row over several workgroups
    const int cols = (a.n_head + a.n_kv) * a.hd;
    const int slices = T >= 64 ? 1 : (cols + 4 * ROW_THREADS - 1) / (4 * ROW_THREADS);
    MESH_LAUNCH(qk_norm_append_kernel, dim3((unsigned)slices, (unsigned)T), dim3(ROW_THREADS), 0, stream, a);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

}  // namespace mesh
