// See rowops.hpp.  One workgroup per token row; sums of squares in f32.
#include "rowops.hpp"

#include "act_math.hpp"

#include "kv_cache.hpp"

namespace mesh {

constexpr int ROW_THREADS = 256, ROW_WAVES = ROW_THREADS / 64;

template <ActType ACT> __device__ __forceinline__ void act_store(void *out, size_t i, float v) {
    if constexpr (ACT == ACT_BF16) static_cast<uint16_t *>(out)[i] = f32_to_bf16_bits(v);
    else static_cast<float *>(out)[i] = v;
}

// Rows are walked four elements at a time when their length is a multiple of four (every row then starts on 16 bytes), else
// one at a time: V elements from i on, and their counterpart on the way out.
template <int V> struct RowVec { float v[V]; };
template <int V> __device__ __forceinline__ RowVec<V> row_load(const float *p) {
    RowVec<V> r;
    if constexpr (V == 4) { const float4 q = *reinterpret_cast<const float4 *>(p); r.v[0] = q.x; r.v[1] = q.y; r.v[2] = q.z; r.v[3] = q.w; }
    else r.v[0] = p[0];
    return r;
}
template <int V> __device__ __forceinline__ void row_store(float *p, const RowVec<V> &r) {
    if constexpr (V == 4) *reinterpret_cast<float4 *>(p) = make_float4(r.v[0], r.v[1], r.v[2], r.v[3]);
    else p[0] = r.v[0];
}
template <ActType ACT, int V> __device__ __forceinline__ void act_store_row(void *out, size_t i, const RowVec<V> &r) {
    if constexpr (ACT == ACT_F32) row_store<V>(static_cast<float *>(out) + i, r);
    else if constexpr (V == 4)
        *reinterpret_cast<uint2 *>(static_cast<uint16_t *>(out) + i) = make_uint2((uint32_t)f32_to_bf16_bits(r.v[0]) | ((uint32_t)f32_to_bf16_bits(r.v[1]) << 16),
                                                                                  (uint32_t)f32_to_bf16_bits(r.v[2]) | ((uint32_t)f32_to_bf16_bits(r.v[3]) << 16));
    else act_store<ACT>(out, i, r.v[0]);
}

__device__ __forceinline__ float row_sum(float v, float *scratch) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}

__global__ __launch_bounds__(ROW_THREADS) void embed_rows_kernel(const uint16_t *table, int ldt, const int32_t *tok, const int32_t *pos, const float *freq, float scale,
                                                                 int n, float *x) {
    const int t = blockIdx.x;
    const uint16_t *e = table + (size_t)tok[t] * ldt;
    const float p = (float)pos[t];
    for (int i = threadIdx.x; i < n; i += ROW_THREADS) {
        float v = bf16_bits_to_f32(e[i]) * scale;
        if (freq) {
            const float angle = p * freq[i >> 1];
            v += (i & 1) ? cosf(angle) : sinf(angle);
        }
        x[(size_t)t * n + i] = v;
    }
}

template <ActType ACT, int V>
__global__ __launch_bounds__(ROW_THREADS) void residual_norm_kernel(float *x, const float *y, const float *gain, float eps, int n, void *out, int ld) {
    __shared__ float scratch[ROW_WAVES];
    const size_t at = (size_t)blockIdx.x * n, to = (size_t)blockIdx.x * ld;
    float rinv = 0.f;
    if (y) {
        float ss = 0.f;
#pragma unroll 4
        for (int i = threadIdx.x * V; i < n; i += ROW_THREADS * V) {
            const RowVec<V> r = row_load<V>(y + at + i);
#pragma unroll
            for (int j = 0; j < V; ++j) ss = fmaf(r.v[j], r.v[j], ss);
        }
        rinv = 1.0f / sqrtf(row_sum(ss, scratch) / (float)n + eps);
    }
#pragma unroll 4
    for (int i = threadIdx.x * V; i < ld; i += ROW_THREADS * V) {
        RowVec<V> v = {};
        if (i < n) {
            v = row_load<V>(x + at + i);
            if (y) {
                const RowVec<V> r = row_load<V>(y + at + i), g = row_load<V>(gain + i);
#pragma unroll
                for (int j = 0; j < V; ++j) v.v[j] = v.v[j] + r.v[j] * rinv * g.v[j];
                row_store<V>(x + at + i, v);
            }
        }
        act_store_row<ACT, V>(out, to + i, v);
    }
}

// The same with layer norms on both sides: x += post(y), act = pre(x).  A thread keeps its NV groups of V elements of the row
// in registers (NV 0: rows of any length, read again for every pass).  Means first, then squared deviations.
template <ActType ACT, int V, int NV>
__global__ __launch_bounds__(ROW_THREADS) void layer_norm_kernel(const float *src, const int32_t *row, float *x, const float *y, const RowNorm post, const RowNorm pre,
                                                                 float eps, int n, void *out, int ld) {
    __shared__ float scratch[ROW_WAVES];
    constexpr int NR = NV ? NV : 1;
    const size_t at = (size_t)(row ? row[blockIdx.x] : (int)blockIdx.x) * n, to = (size_t)blockIdx.x * ld;
    const float inv_n = 1.0f / (float)n;
    RowVec<V> r[NR];
    auto each = [&](auto fn) {         // fn(first element, register group)
        if constexpr (NV > 0) {
#pragma unroll
            for (int k = 0; k < NV; ++k) {
                const int i = (k * ROW_THREADS + (int)threadIdx.x) * V;
                if (i < n) fn(i, r[k]);
            }
        } else {
            for (int i = threadIdx.x * V; i < n; i += ROW_THREADS * V) fn(i, r[0]);
        }
    };
    auto moments = [&](const float *p, float &mean, float &rstd) {
        float s = 0.f;
        each([&](int i, RowVec<V> &v) {
            if (NV == 0) v = row_load<V>(p + i);
#pragma unroll
            for (int j = 0; j < V; ++j) s += v.v[j];
        });
        mean = row_sum(s, scratch) * inv_n;
        float d2 = 0.f;
        each([&](int i, RowVec<V> &v) {
            if (NV == 0) v = row_load<V>(p + i);
#pragma unroll
            for (int j = 0; j < V; ++j) { const float d = v.v[j] - mean; d2 = fmaf(d, d, d2); }
        });
        rstd = 1.0f / sqrtf(row_sum(d2, scratch) * inv_n + eps);
    };
    float mean, rstd;
    if (y) {
        if (NV > 0) each([&](int i, RowVec<V> &v) { v = row_load<V>(y + at + i); });
        moments(y + at, mean, rstd);
        each([&](int i, RowVec<V> &v) {
            if (NV == 0) v = row_load<V>(y + at + i);
            const RowVec<V> g = row_load<V>(post.gain + i), b = row_load<V>(post.bias + i), xv = row_load<V>(src + at + i);
#pragma unroll
            for (int j = 0; j < V; ++j) v.v[j] = xv.v[j] + ((v.v[j] - mean) * rstd * g.v[j] + b.v[j]);
            row_store<V>(x + at + i, v);
        });
        src = x;
    } else if (NV > 0) {
        each([&](int i, RowVec<V> &v) { v = row_load<V>(src + at + i); });
    }
    if (!out) return;
    mean = 0.f; rstd = 1.f;
    if (pre.kind == NORM_LAYER) moments(src + at, mean, rstd);
    each([&](int i, RowVec<V> &v) {
        if (NV == 0) v = row_load<V>(src + at + i);
        RowVec<V> o = v;
        if (pre.kind == NORM_LAYER) {
            const RowVec<V> g = row_load<V>(pre.gain + i), b = row_load<V>(pre.bias + i);
#pragma unroll
            for (int j = 0; j < V; ++j) o.v[j] = (v.v[j] - mean) * rstd * g.v[j] + b.v[j];
        }
        act_store_row<ACT, V>(out, to + i, o);
    });
    for (int i = n + threadIdx.x; i < ld; i += ROW_THREADS) act_store<ACT>(out, to + i, 0.f);
}

template <ActType ACT>
static int launch_layer_norm(const float *src, const int32_t *row, float *x, const float *y, const RowNorm &post, const RowNorm &pre, float eps, int rows, int n, void *out, int ld,
                             hipStream_t stream) {
    const dim3 grid((unsigned)rows), block(ROW_THREADS);
    const int groups = n % 4 == 0 ? (n + 4 * ROW_THREADS - 1) / (4 * ROW_THREADS) : 0;
    if (groups == 1) MESH_LAUNCH((layer_norm_kernel<ACT, 4, 1>), grid, block, 0, stream, src, row, x, y, post, pre, eps, n, out, ld);
    else if (groups == 2) MESH_LAUNCH((layer_norm_kernel<ACT, 4, 2>), grid, block, 0, stream, src, row, x, y, post, pre, eps, n, out, ld);
    else if (groups >= 3 && groups <= 4) MESH_LAUNCH((layer_norm_kernel<ACT, 4, 4>), grid, block, 0, stream, src, row, x, y, post, pre, eps, n, out, ld);
    else if (groups >= 5 && groups <= 8) MESH_LAUNCH((layer_norm_kernel<ACT, 4, 8>), grid, block, 0, stream, src, row, x, y, post, pre, eps, n, out, ld);
    else if (groups) MESH_LAUNCH((layer_norm_kernel<ACT, 4, 0>), grid, block, 0, stream, src, row, x, y, post, pre, eps, n, out, ld);
    else MESH_LAUNCH((layer_norm_kernel<ACT, 1, 0>), grid, block, 0, stream, src, row, x, y, post, pre, eps, n, out, ld);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
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

template <ActType ACT, int V>
__global__ __launch_bounds__(ROW_THREADS) void poly_norm_kernel(const float *u, const float *coef, float eps, int n, void *out, int ld) {
    __shared__ float scratch[ROW_WAVES];
    const size_t at = (size_t)blockIdx.x * n, to = (size_t)blockIdx.x * ld;
    float p2 = 0.f, p4 = 0.f, p6 = 0.f;
#pragma unroll 4
    for (int i = threadIdx.x * V; i < n; i += ROW_THREADS * V) {
        const RowVec<V> r = row_load<V>(u + at + i);
#pragma unroll
        for (int j = 0; j < V; ++j) {
            const float q = r.v[j] * r.v[j];
            p2 += q; p4 += q * q; p6 += q * q * q;
        }
    }
    p2 = row_sum(p2, scratch); p4 = row_sum(p4, scratch); p6 = row_sum(p6, scratch);
    const float c1 = coef[0] / sqrtf(p2 / (float)n + eps), c2 = coef[1] / sqrtf(p4 / (float)n + eps), c3 = coef[2] / sqrtf(p6 / (float)n + eps), c0 = coef[3];
#pragma unroll 4
    for (int i = threadIdx.x * V; i < ld; i += ROW_THREADS * V) {
        RowVec<V> v = {};
        if (i < n) {
            v = row_load<V>(u + at + i);
#pragma unroll
            for (int j = 0; j < V; ++j) v.v[j] = ((c3 * v.v[j] + c2) * v.v[j] + c1) * v.v[j] + c0;
        }
        act_store_row<ACT, V>(out, to + i, v);
    }
}

template <ActType ACT>
__global__ __launch_bounds__(64) void side_gate_kernel(const float *g, int slices, size_t slice_stride, const uint16_t *side, const int32_t *tok, int stride, int offset, int n, void *out, int ld) {
    const int t = blockIdx.x;
    const uint16_t *e = side + (size_t)tok[t] * stride + offset;
    for (int i = threadIdx.x; i < ld; i += 64) {
        float v = 0.f;
        if (i < n) {
            float z = 0.f;
            for (int s = 0; s < slices; ++s) z += g[s * slice_stride + (size_t)t * n + i];
            v = act_gelu_tanh(z) * bf16_bits_to_f32(e[i]);
        }
        act_store<ACT>(out, (size_t)t * ld + i, v);
    }
}

__device__ __forceinline__ void append4(uint8_t *cache, int type, size_t at, const float4 &v, unsigned *sat) {
    if (type == MESH_F32) { *reinterpret_cast<float4 *>(reinterpret_cast<float *>(cache) + at) = v; return; }
    note_f16_clamp(sat, v.x, v.y, v.z, v.w);
    auto h = [](float f) { return (uint32_t)f32_to_f16_bits(fminf(fmaxf(f, -65504.f), 65504.f)); };
    *reinterpret_cast<uint2 *>(reinterpret_cast<uint16_t *>(cache) + at) = make_uint2(h(v.x) | (h(v.y) << 16), h(v.z) | (h(v.w) << 16));
}

// grid (slices of the heads, T); every workgroup sums the whole row itself, so that slices need not meet
__global__ __launch_bounds__(ROW_THREADS) void qk_norm_append_kernel(const QkAppendArgs a) {
    __shared__ float scratch[ROW_WAVES];
    const int t = blockIdx.y, nq = a.n_head * a.hd, nk = a.n_kv * a.hd;
    const float *row = a.qk + (size_t)t * (nq + nk);
    float sq = 0.f, sk = 0.f;           // (head rows are a multiple of 64 long: four at a time)
#pragma unroll 4
    for (int i = threadIdx.x * 4; i < nq + nk; i += ROW_THREADS * 4) {
        const float4 v = *reinterpret_cast<const float4 *>(row + i);
        const float s = v.x * v.x + v.y * v.y + v.z * v.z + v.w * v.w;
        if (i < nq) sq += s; else sk += s;
    }
    const float rq = 1.0f / sqrtf(row_sum(sq, scratch) / (float)(a.n_head * a.dim) + a.eps);
    const float rk = 1.0f / sqrtf(row_sum(sk, scratch) / (float)(a.n_kv * a.dim) + a.eps);
    const int pos = a.pos[t], seq = a.seq[t];
    const int stride = gridDim.x * ROW_THREADS * 4;
    for (int i = (blockIdx.x * ROW_THREADS + threadIdx.x) * 4; i < nq + nk; i += stride) {
        const float4 v = *reinterpret_cast<const float4 *>(row + i);
        if (i < nq) {
            const float4 g = *reinterpret_cast<const float4 *>(a.q_norm + i);
            *reinterpret_cast<float4 *>(a.q + (size_t)t * nq + i) = make_float4(v.x * rq * g.x, v.y * rq * g.y, v.z * rq * g.z, v.w * rq * g.w);
            continue;
        }
        const int kk = i - nq, head = kk / a.hd;
        const float4 g = *reinterpret_cast<const float4 *>(a.k_norm + kk);
        const size_t at = (((size_t)seq * a.n_kv + head) * a.n_ctx + pos) * a.hd + (kk - head * a.hd);
        append4(a.kcache, a.kv_type, at, make_float4(v.x * rk * g.x, v.y * rk * g.y, v.z * rk * g.z, v.w * rk * g.w), a.sat);
        append4(a.vcache, a.kv_type, at, v, a.sat);
    }
}

#define MESH_ACT_LAUNCH(kernel, act, grid, block, ...)                                                     \
    do {                                                                                                   \
        if (act == ACT_BF16) MESH_LAUNCH((kernel<ACT_BF16>), grid, block, 0, stream, __VA_ARGS__);         \
        else MESH_LAUNCH((kernel<ACT_F32>), grid, block, 0, stream, __VA_ARGS__);                          \
        MESH_LAUNCH_CHECK();                                                                               \
    } while (0)

#define MESH_ROW_LAUNCH(kernel, act, vec, grid, block, ...)                                                \
    do {                                                                                                   \
        if (act == ACT_BF16 && (vec)) MESH_LAUNCH((kernel<ACT_BF16, 4>), grid, block, 0, stream, __VA_ARGS__); \
        else if (act == ACT_BF16) MESH_LAUNCH((kernel<ACT_BF16, 1>), grid, block, 0, stream, __VA_ARGS__);  \
        else if (vec) MESH_LAUNCH((kernel<ACT_F32, 4>), grid, block, 0, stream, __VA_ARGS__);               \
        else MESH_LAUNCH((kernel<ACT_F32, 1>), grid, block, 0, stream, __VA_ARGS__);                        \
        MESH_LAUNCH_CHECK();                                                                               \
    } while (0)

int embed_rows(const uint16_t *table, int ldt, const int32_t *tok, const int32_t *pos, const float *freq, float scale, int T, int n, float *x, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    MESH_LAUNCH(embed_rows_kernel, dim3((unsigned)T), dim3(ROW_THREADS), 0, stream, table, ldt, tok, pos, freq, scale, n, x);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

static bool norm_ok(const RowNorm &nm) { return nm.kind == NORM_NONE || (nm.gain && (nm.kind == NORM_RMS || nm.bias)); }

int residual_norm_rows(float *x, const float *y, const RowNorm &post, const RowNorm &pre, float eps, int T, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (ld < n || !norm_ok(post) || !norm_ok(pre) || (y && post.kind == NORM_NONE) || pre.kind == NORM_RMS) return fail(MESH_ERR_INVALID, "residual_norm_rows: bad operands");
    if (post.kind == NORM_LAYER || pre.kind == NORM_LAYER) {
        if (y && post.kind != NORM_LAYER) return fail(MESH_ERR_UNSUPPORTED, "residual_norm_rows: no kernel for norm %d before norm %d", (int)post.kind, (int)pre.kind);
        return act == ACT_BF16 ? launch_layer_norm<ACT_BF16>(x, nullptr, x, y, post, pre, eps, T, n, out, ld, stream)
                               : launch_layer_norm<ACT_F32>(x, nullptr, x, y, post, pre, eps, T, n, out, ld, stream);
    }
    MESH_ROW_LAUNCH(residual_norm_kernel, act, n % 4 == 0, dim3((unsigned)T), dim3(ROW_THREADS), x, y, post.gain, eps, n, out, ld);
    return MESH_OK;
}

int layer_norm_rows(const float *x, const int32_t *row, const RowNorm &norm, float eps, int n_rows, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (n_rows <= 0) return MESH_OK;
    if (ld < n || norm.kind != NORM_LAYER || !norm_ok(norm)) return fail(MESH_ERR_INVALID, "layer_norm_rows: bad operands");
    return act == ACT_BF16 ? launch_layer_norm<ACT_BF16>(x, row, nullptr, nullptr, RowNorm{}, norm, eps, n_rows, n, out, ld, stream)
                           : launch_layer_norm<ACT_F32>(x, row, nullptr, nullptr, RowNorm{}, norm, eps, n_rows, n, out, ld, stream);
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
    MESH_ROW_LAUNCH(poly_norm_kernel, act, n % 4 == 0, dim3((unsigned)T), dim3(ROW_THREADS), u, coef, eps, n, out, ld);
    return MESH_OK;
}

int side_gate_rows(const float *g, int slices, size_t slice_stride, const uint16_t *side, const int32_t *tok, int stride, int offset, int T, int n, void *out, ActType act, int ld, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (ld < n || offset + n > stride) return fail(MESH_ERR_INVALID, "side_gate_rows: bad operands");
    MESH_ACT_LAUNCH(side_gate_kernel, act, dim3((unsigned)T), dim3(64), g, slices, slice_stride, side, tok, stride, offset, n, out, ld);
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
