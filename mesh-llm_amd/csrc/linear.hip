// Products of bf16 weight matrices with many token rows, on the matrix cores.
//
// linear_rows_kernel streams the weights: a workgroup owns 16 weight rows and 16 * NT tokens, its four waves split K and
// meet in LDS.  The A operand is the weight row as it lies in memory (lane = row, 8 consecutive k), the B operand the
// activation row (lane = token).  With f32 activations the same fragments feed eight v_mfma_f32_16x16x4_f32 instead of one
// v_mfma_f32_16x16x32_bf16: step j multiplies element j of every lane's 8, and the sum over lanes groups and steps covers
// the same 32 products.
//
// linear_tile_kernel is the large-tile product (128 weight rows x 128 tokens x 64 k): both operands go from memory to
// LDS without passing through registers, two stages, one barrier per stage.  Rows of 64 elements are 128 bytes, eight
// 16-byte pieces; piece p of row r is kept at position p ^ ((r >> 1) & 7), so that the 16 rows a fragment read touches at
// a time fall on all 64 banks.  The destination of such a load is linear in the lane, so the swizzle is applied to the
// source address.
#include "linear.hpp"

namespace mesh {

typedef __bf16 ln_b8 __attribute__((ext_vector_type(8)));
typedef float ln_f4 __attribute__((ext_vector_type(4)));
typedef float ln_f16 __attribute__((ext_vector_type(16)));
typedef uint32_t ln_u4 __attribute__((ext_vector_type(4)));

constexpr int ROWS_WAVES = 4;

template <ActType ACT> struct RowsFrag;
template <> struct RowsFrag<ACT_BF16> {
    uint4 v;
    __device__ __forceinline__ void load(const void *x, size_t at) { v = *reinterpret_cast<const uint4 *>(static_cast<const uint16_t *>(x) + at); }
};
template <> struct RowsFrag<ACT_F32> {
    float4 a, b;
    __device__ __forceinline__ void load(const void *x, size_t at) {
        const float *p = static_cast<const float *>(x) + at;
        a = *reinterpret_cast<const float4 *>(p);
        b = *reinterpret_cast<const float4 *>(p + 4);
    }
};

__device__ __forceinline__ ln_f4 rows_mma(const uint4 &w, const RowsFrag<ACT_BF16> &x, ln_f4 acc) {
    return __builtin_amdgcn_mfma_f32_16x16x32_bf16(__builtin_bit_cast(ln_b8, w), __builtin_bit_cast(ln_b8, x.v), acc, 0, 0, 0);
}
__device__ __forceinline__ ln_f4 rows_mma(const uint4 &w, const RowsFrag<ACT_F32> &x, ln_f4 acc) {
    const uint32_t u[4] = {w.x, w.y, w.z, w.w};
    const float xf[8] = {x.a.x, x.a.y, x.a.z, x.a.w, x.b.x, x.b.y, x.b.z, x.b.w};
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const float wf = __uint_as_float((j & 1) ? (u[j >> 1] & 0xFFFF0000u) : (u[j >> 1] << 16));
        acc = __builtin_amdgcn_mfma_f32_16x16x4f32(wf, xf[j], acc, 0, 0, 0);
    }
    return acc;
}

// what becomes of a result: stored as it is, or as an activation of the product that follows
enum LinearOut { LINEAR_OUT_F32 = 0, LINEAR_OUT_RELU2 = 1 };
template <ActType ACT, LinearOut OUT> __device__ __forceinline__ void linear_store(void *y, size_t at, float v) {
    if constexpr (OUT == LINEAR_OUT_RELU2) {
        v = fmaxf(v, 0.f);
        v *= v;
    }
    if constexpr (OUT == LINEAR_OUT_F32 || ACT == ACT_F32) static_cast<float *>(y)[at] = v;
    else static_cast<uint16_t *>(y)[at] = f32_to_bf16_bits(v);
}

// grid (row blocks of 16, token blocks of 16 * NT)
template <ActType ACT, int NT, LinearOut OUT>
__global__ __launch_bounds__(64 * ROWS_WAVES) void linear_rows_kernel(const uint16_t *w, const void *x, void *y, int K, int M, int T, int ldy) {
    __shared__ float red[ROWS_WAVES][NT][16][17];
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int m0 = blockIdx.x * 16, t0 = blockIdx.y * 16 * NT;
    const uint16_t *wp = w + (size_t)(m0 + c) * K + 8 * g;
    size_t xo[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) {
        const int t = t0 + 16 * n + c;
        xo[n] = (size_t)(t < T ? t : T - 1) * K + 8 * g;       // columns past the call repeat its last token and are not stored
    }
    ln_f4 acc[NT];
#pragma unroll
    for (int n = 0; n < NT; ++n) acc[n] = ln_f4{0.f, 0.f, 0.f, 0.f};
    // several steps' loads go out together; a step past the end multiplies zero weights
    constexpr int UN = NT == 4 ? 2 : 4;
    for (int kb = wave * 32; kb < K; kb += UN * 32 * ROWS_WAVES) {
        uint4 wf[UN];
        RowsFrag<ACT> xf[UN][NT];
#pragma unroll
        for (int u = 0; u < UN; ++u) {
            const int k = kb + u * 32 * ROWS_WAVES;
            const int at = k < K ? k : 0;
            wf[u] = *reinterpret_cast<const uint4 *>(wp + at);
            if (k >= K) wf[u] = make_uint4(0, 0, 0, 0);
#pragma unroll
            for (int n = 0; n < NT; ++n) xf[u][n].load(x, xo[n] + at);
        }
#pragma unroll
        for (int u = 0; u < UN; ++u)
#pragma unroll
            for (int n = 0; n < NT; ++n) acc[n] = rows_mma(wf[u], xf[u][n], acc[n]);
    }
    // register i of a lane: weight row 4 * g + i, token c
#pragma unroll
    for (int n = 0; n < NT; ++n)
#pragma unroll
        for (int i = 0; i < 4; ++i) red[wave][n][c][4 * g + i] = acc[n][i];
    __syncthreads();
    for (int idx = tid; idx < NT * 256; idx += 64 * ROWS_WAVES) {
        const int r = idx & 15, tk = (idx >> 4) & 15, n = idx >> 8;
        float s = red[0][n][tk][r];
#pragma unroll
        for (int v = 1; v < ROWS_WAVES; ++v) s += red[v][n][tk][r];
        const int m = m0 + r, t = t0 + 16 * n + tk;
        if (m < M && t < T) linear_store<ACT, OUT>(y, (size_t)t * ldy + m, s);
    }
}

// ---- large tile -----------------------------------------------------------------------------------------------
constexpr int TILE_M = 128, TILE_T = 128, TILE_K = 64, TILE_THREADS = 256;

typedef const __attribute__((address_space(1))) uint32_t *ln_gptr;
typedef __attribute__((address_space(3))) uint32_t *ln_lptr;

__device__ __forceinline__ void tile_copy16(const uint16_t *src, uint16_t *lds_base) {
    __builtin_amdgcn_global_load_lds((ln_gptr)(src), (ln_lptr)(lds_base), 16, 0, 0);
}

// 1-D grid of (row blocks x token blocks); the workgroups a die is dealt (every eighth) take a contiguous run of tiles with
// the token block running fastest, so that the weight rows of a run stay in that die's cache
template <LinearOut OUT>
__global__ __launch_bounds__(TILE_THREADS) void linear_tile_kernel(const uint16_t *w, const uint16_t *x, void *y, int K, int M, int T, int ldy,
                                                                   int n_tblocks, int n_tiles, int k_slice, size_t y_slice) {
    // blockIdx.y: slice of K and the partial result it writes
    const int k_begin = blockIdx.y * k_slice, k_end = k_begin + k_slice < K ? k_begin + k_slice : K;
    y = static_cast<float *>(y) + blockIdx.y * y_slice;          // (slices are f32 results)
    __shared__ __align__(16) uint16_t sW0[TILE_M * TILE_K], sW1[TILE_M * TILE_K], sX0[TILE_T * TILE_K], sX1[TILE_T * TILE_K];
    const int tid = threadIdx.x, lane = tid & 63, wave = __builtin_amdgcn_readfirstlane(tid >> 6);
    int tile = blockIdx.x;
    {
        const int per = n_tiles >> 3, whole = per << 3;
        if (tile < whole) tile = (tile & 7) * per + (tile >> 3);
    }
    const int mb = tile / n_tblocks, tb = tile % n_tblocks;
    const int wm = (wave & 1) * 64, wt = (wave >> 1) * 64;      // this wave's 64 x 64 corner of the tile
    // staging: instruction j of a wave brings rows 32 * wave + 8 * j .. + 8, lane -> (row lane / 8, position lane % 8)
    const uint16_t *gw[4], *gx[4];
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int r = wave * 32 + j * 8 + (lane >> 3);
        const int piece = (lane & 7) ^ ((r >> 1) & 7);
        gw[j] = w + (size_t)(mb * TILE_M + r) * K + piece * 8;
        const int t = tb * TILE_T + r;
        gx[j] = x + (size_t)(t < T ? t : T - 1) * K + piece * 8;
    }
    auto stage = [&](uint16_t *dw, uint16_t *dx, int k) {
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            tile_copy16(gw[j] + k, dw + (wave * 32 + j * 8) * TILE_K);
            tile_copy16(gx[j] + k, dx + (wave * 32 + j * 8) * TILE_K);
        }
    };
    ln_f16 acc[2][2];
#pragma unroll
    for (int a = 0; a < 2; ++a)
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int i = 0; i < 16; ++i) acc[a][b][i] = 0.f;
    const int r32 = lane & 31, half = lane >> 5;
    const int sw = (r32 >> 1) & 7;                // (row >> 1) & 7 is the same for the rows 32 and 64 further down
    auto multiply = [&](const uint16_t *dw, const uint16_t *dx) {
#pragma unroll
        for (int ks = 0; ks < TILE_K / 16; ++ks) {
            const int at = ((2 * ks + half) ^ sw) * 8;
            ln_b8 xf[2], wf[2];
#pragma unroll
            for (int a = 0; a < 2; ++a) {
                xf[a] = *reinterpret_cast<const ln_b8 *>(dx + (wt + 32 * a + r32) * TILE_K + at);
                wf[a] = *reinterpret_cast<const ln_b8 *>(dw + (wm + 32 * a + r32) * TILE_K + at);
            }
            // result: rows = tokens, columns (lanes) = weight rows, so that a store covers whole lines of y
#pragma unroll
            for (int a = 0; a < 2; ++a)
#pragma unroll
                for (int b = 0; b < 2; ++b) acc[a][b] = __builtin_amdgcn_mfma_f32_32x32x16_bf16(xf[a], wf[b], acc[a][b], 0, 0, 0);
        }
    };
    // One barrier per stage: behind it every wave's loads of this stage have landed, and every wave is done reading the
    // other stage, which the next loads overwrite.
    auto arrive = [&]() {
        asm volatile("s_waitcnt vmcnt(0)" ::: "memory");
        __syncthreads();
    };
    stage(sW0, sX0, k_begin);
    for (int k = k_begin; k < k_end; k += 2 * TILE_K) {
        arrive();
        if (k + TILE_K < k_end) stage(sW1, sX1, k + TILE_K);
        multiply(sW0, sX0);
        if (k + TILE_K >= k_end) break;
        arrive();
        if (k + 2 * TILE_K < k_end) stage(sW0, sX0, k + 2 * TILE_K);
        multiply(sW1, sX1);
    }
#pragma unroll
    for (int b = 0; b < 2; ++b) {
        const int m = mb * TILE_M + wm + 32 * b + r32;
        if (m >= M) continue;
#pragma unroll
        for (int a = 0; a < 2; ++a)
#pragma unroll
            for (int i = 0; i < 16; ++i) {
                const int t = tb * TILE_T + wt + 32 * a + 8 * (i >> 2) + 4 * half + (i & 3);
                if (t < T) linear_store<ACT_BF16, OUT>(y, (size_t)t * ldy + m, acc[a][b][i]);
            }
    }
}

// M: columns of y to write, at least W.M (the rows of W behind it are zeros)
template <ActType ACT, LinearOut OUT>
static int launch_rows(const LinearWeight &W, const void *x, int T, void *y, int ldy, int M, hipStream_t stream) {
    const unsigned mb = (unsigned)((M + 15) / 16);
    const dim3 block(64 * ROWS_WAVES);
    if (T <= 16) MESH_LAUNCH((linear_rows_kernel<ACT, 1, OUT>), dim3(mb, 1), block, 0, stream, W.w, x, y, W.Kp, M, T, ldy);
    else if (T <= 32) MESH_LAUNCH((linear_rows_kernel<ACT, 2, OUT>), dim3(mb, 1), block, 0, stream, W.w, x, y, W.Kp, M, T, ldy);
    else MESH_LAUNCH((linear_rows_kernel<ACT, 4, OUT>), dim3(mb, (unsigned)((T + 63) / 64)), block, 0, stream, W.w, x, y, W.Kp, M, T, ldy);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

template <LinearOut OUT>
static int launch_tile(const LinearWeight &W, const void *x, int T, void *y, int ldy, int M, int slices, size_t stride, hipStream_t stream) {
    const int mblocks = (M + TILE_M - 1) / TILE_M, tblocks = (T + TILE_T - 1) / TILE_T;
    const int steps = W.Kp / TILE_K, k_slice = (steps + slices - 1) / slices * TILE_K;
    MESH_LAUNCH((linear_tile_kernel<OUT>), dim3((unsigned)(mblocks * tblocks), (unsigned)slices), dim3(TILE_THREADS), 0, stream, W.w, static_cast<const uint16_t *>(x), y, W.Kp, M,
                T, ldy, tblocks, mblocks * tblocks, k_slice, stride);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

static bool linear_ok(const LinearWeight &W, const void *x, int T, const void *y, int ldy) {
    return W.w && x && y && W.M >= 1 && W.Kp % LINEAR_K_PAD == 0 && W.Mp % LINEAR_ROW_PAD == 0 && W.Mp >= W.M && W.Kp >= W.K && ldy >= W.M && (T + 63) / 64 <= 65535;
}

int linear_sliced(const LinearWeight &W, const void *x, ActType act, int T, float *y, size_t stride, int big_from, hipStream_t stream) {
    const int tiles = (W.M + TILE_M - 1) / TILE_M * ((T + TILE_T - 1) / TILE_T), steps = W.Kp / TILE_K;
    int slices = 128 / (tiles > 0 ? tiles : 1);
    if (slices > LINEAR_SLICES_MAX) slices = LINEAR_SLICES_MAX;
    if (slices > steps / 4) slices = steps / 4;                  // (a slice of at least four steps)
    if (slices > 1) slices = (steps + (steps + slices - 1) / slices - 1) / ((steps + slices - 1) / slices);        // every slice has some
    if (act == ACT_F32 || T < big_from || slices <= 1 || stride < (size_t)T * W.M) {
        const int rc = linear(W, x, act, T, y, W.M, big_from, stream);
        return rc == MESH_OK ? 1 : rc;
    }
    if (!linear_ok(W, x, T, y, W.M)) return fail(MESH_ERR_INVALID, "linear_sliced: bad operands (%d x %d, %d tokens)", W.M, W.K, T);
    const int rc = launch_tile<LINEAR_OUT_F32>(W, x, T, y, W.M, W.M, slices, stride, stream);
    return rc == MESH_OK ? slices : rc;
}

int linear(const LinearWeight &W, const void *x, ActType act, int T, float *y, int ldy, int big_from, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!linear_ok(W, x, T, y, ldy)) return fail(MESH_ERR_INVALID, "linear: bad operands (%d x %d, %d tokens)", W.M, W.K, T);
    if (act == ACT_F32) return launch_rows<ACT_F32, LINEAR_OUT_F32>(W, x, T, y, ldy, W.M, stream);
    if (T < big_from || W.M < TILE_M) return launch_rows<ACT_BF16, LINEAR_OUT_F32>(W, x, T, y, ldy, W.M, stream);
    return launch_tile<LINEAR_OUT_F32>(W, x, T, y, ldy, W.M, 1, 0, stream);
}

int linear_relu2(const LinearWeight &W, const void *x, ActType act, int T, void *out, int ld, int big_from, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!linear_ok(W, x, T, out, ld) || ld > W.Mp) return fail(MESH_ERR_INVALID, "linear_relu2: bad operands (%d x %d, %d tokens)", W.M, W.K, T);
    if (act == ACT_F32) return launch_rows<ACT_F32, LINEAR_OUT_RELU2>(W, x, T, out, ld, ld, stream);
    if (T < big_from || W.M < TILE_M) return launch_rows<ACT_BF16, LINEAR_OUT_RELU2>(W, x, T, out, ld, ld, stream);
    return launch_tile<LINEAR_OUT_RELU2>(W, x, T, out, ld, ld, 1, 0, stream);
}

}  // namespace mesh
