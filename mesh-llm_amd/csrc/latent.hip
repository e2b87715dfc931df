// See latent.hpp.
//
// latent_attn_kernel: a workgroup takes one (key split, 16 heads, token or four consecutive tokens of a sequence).  A step stages 32 cache rows in LDS, once as they
// are and (f16) once with the latents transposed, pairs of keys as dwords, since the second product contracts over keys:
//   S^T (32 keys x 16 heads)   = rows . Q^T        v_mfma_f32_16x16x32_f16 per 32 elements of a row
//   O^T (rank x 16 heads)     += latents^T . P^T   the result registers of S^T are the P^T operand as they are
// With one token every wave computes the scores (they are few), so that no softmax state crosses waves, and owns a quarter of
// the rank's rows of O^T; with four each wave has a token.  With f32 rows the same fragments feed v_mfma_f32_16x16x4_f32, eight per 32 elements.
#include "latent.hpp"

#include <algorithm>

#include "act_math.hpp"
#include "attn.hpp"

namespace mesh {

typedef _Float16 lt_h8 __attribute__((ext_vector_type(8)));
typedef _Float16 lt_h2 __attribute__((ext_vector_type(2)));
typedef float lt_f4 __attribute__((ext_vector_type(4)));
typedef uint32_t lt_u4 __attribute__((ext_vector_type(4)));

constexpr int LT_THREADS = 256, LT_WAVES = LT_THREADS / 64;
constexpr int LT_KEYS = 32, LT_VPITCH = LT_KEYS / 2 + 2;      // keys per step; dwords per latent row of the transposed tile
constexpr int LT_QUERY_TOKENS = 4;                            // tokens that share a workgroup's weight rows in latent_query
constexpr size_t LT_LDS_MAX = 160 * 1024 - 1024;

__device__ __forceinline__ float lt_exp2(float x) { return __builtin_amdgcn_exp2f(x); }
__device__ __forceinline__ uint32_t lt_pack(float a, float b) {
    const lt_h2 h = {(_Float16)a, (_Float16)b};
    return __builtin_bit_cast(uint32_t, h);
}
__device__ __forceinline__ float lt_block_sum(float v, float *scratch) {
#pragma unroll
    for (int o = 32; o > 0; o >>= 1) v += __shfl_xor(v, o);
    __syncthreads();
    if ((threadIdx.x & 63) == 0) scratch[threadIdx.x >> 6] = v;
    __syncthreads();
    return scratch[0] + scratch[1] + scratch[2] + scratch[3];
}
// cosine and sine of position times frequency: the product and its whole turns in 64 bits, so that the angle is as exact at
// the end of a long context as at its start
__device__ __forceinline__ float2 lt_turn(int pos, double freq, float gain) {
    const double turns = (double)pos * freq * 0.15915494309189535;
    const float a = (float)((turns - rint(turns)) * 6.283185307179586);
    return make_float2(cosf(a) * gain, sinf(a) * gain);
}

template <ActType ACT> struct LtElem;
template <> struct LtElem<ACT_BF16> { typedef uint16_t type; };       // f16 bits
template <> struct LtElem<ACT_F32> { typedef float type; };
template <ActType ACT> __device__ __forceinline__ void lt_put(void *p, size_t at, float v, unsigned *sat) {
    if constexpr (ACT == ACT_F32) static_cast<float *>(p)[at] = v;
    else {
        note_f16_clamp(sat, v, 0.f);
        static_cast<uint16_t *>(p)[at] = f32_to_f16_bits(fminf(fmaxf(v, -65504.f), 65504.f));
    }
}

// one workgroup: the cache row of token t
template <ActType ACT>
__device__ __forceinline__ void lt_append(const LatentShape &s, const LatentCache &c, int t, float *scratch) {
    const float *p = c.in + (size_t)t * c.ld;
    const int pos = c.pos[t];
    const size_t at = ((size_t)c.seq[t] * c.n_ctx + pos) * s.row();
    float ss = 0.f;
    for (int i = threadIdx.x; i < s.rank; i += LT_THREADS) ss = fmaf(p[i], p[i], ss);
    const float r = 1.0f / sqrtf(lt_block_sum(ss, scratch) / (float)s.rank + c.eps);
    for (int i = threadIdx.x; i < s.rank_pad; i += LT_THREADS) lt_put<ACT>(c.rows, at + i, i < s.rank ? p[i] * r * c.gain[i] : 0.f, c.sat);
    for (int i = threadIdx.x; i < s.rot_pad / 2; i += LT_THREADS) {
        float u = 0.f, v = 0.f;
        if (2 * i < s.rot_dim) {
            const float2 w = lt_turn(pos, c.rot.freq[i], c.rot.gain);
            const float x = p[s.rank + 2 * i], y = p[s.rank + 2 * i + 1];
            u = x * w.x - y * w.y;
            v = y * w.x + x * w.y;
        }
        lt_put<ACT>(c.rows, at + s.rank_pad + 2 * i, u, c.sat);
        lt_put<ACT>(c.rows, at + s.rank_pad + 2 * i + 1, v, c.sat);
    }
}

template <ActType ACT>
__global__ __launch_bounds__(LT_THREADS) void latent_rows_kernel(const LatentShape s, const LatentCache c, const float *in, int ld, const float *gain, int n, void *out, int ld_out) {
    __shared__ float scratch[LT_WAVES];
    const int t = blockIdx.x;
    const float *p = in + (size_t)t * ld;
    float ss = 0.f;
    for (int i = threadIdx.x; i < n; i += LT_THREADS) ss = fmaf(p[i], p[i], ss);
    const float r = 1.0f / sqrtf(lt_block_sum(ss, scratch) / (float)n + c.eps);
    for (int i = threadIdx.x; i < ld_out; i += LT_THREADS) {
        const float v = i < n ? p[i] * r * gain[i] : 0.f;
        if constexpr (ACT == ACT_BF16) static_cast<uint16_t *>(out)[(size_t)t * ld_out + i] = f32_to_bf16_bits(v);
        else static_cast<float *>(out)[(size_t)t * ld_out + i] = v;
    }
    if (c.in) lt_append<ACT>(s, c, t, scratch);
}

// eight bf16 weights times eight floats of LDS
__device__ __forceinline__ float lt_dot8(const uint4 &w, const float *x, float acc) {
    const uint32_t u[4] = {w.x, w.y, w.z, w.w};
    const float4 xa = *reinterpret_cast<const float4 *>(x), xb = *reinterpret_cast<const float4 *>(x + 4);
    const float xf[8] = {xa.x, xa.y, xa.z, xa.w, xb.x, xb.y, xb.z, xb.w};
#pragma unroll
    for (int j = 0; j < 8; ++j) acc = fmaf(__uint_as_float((j & 1) ? (u[j >> 1] & 0xFFFF0000u) : (u[j >> 1] << 16)), xf[j], acc);
    return acc;
}

// grid (heads, or one more that appends; slices of the rank; groups of TB tokens).  Eight lanes per weight row.
template <ActType ACT, int TB>
__global__ __launch_bounds__(LT_THREADS) void latent_query_kernel(const LatentShape s, const LatentCache c, const float *q, const uint16_t *w, float scale, void *qa, int T) {
    extern __shared__ __align__(16) uint8_t smem[];
    __shared__ float scratch[LT_WAVES];
    const int h = blockIdx.x, t0 = blockIdx.z * TB, tid = threadIdx.x;
    if (h == s.heads) {
        if (blockIdx.y == 0)
            for (int t = t0; t < t0 + TB && t < T; ++t) lt_append<ACT>(s, c, t, scratch);
        return;
    }
    float *xs = reinterpret_cast<float *>(smem);          // [TB][dim_pad]
    const int D = s.dim, P = s.rot_dim, row_q = s.heads * (D + P);
    const float qs = scale * 1.44269504088896341f;
    for (int i = tid; i < TB * s.dim_pad; i += LT_THREADS) {
        const int b = i / s.dim_pad, d = i % s.dim_pad;
        xs[i] = d < D && t0 + b < T ? q[(size_t)(t0 + b) * row_q + h * (D + P) + d] * qs : 0.f;
    }
    if (blockIdx.y == 0) {
        for (int i = tid; i < TB * (s.rot_pad / 2); i += LT_THREADS) {
            const int b = i / (s.rot_pad / 2), pr = i % (s.rot_pad / 2), t = t0 + b;
            if (t >= T) break;
            float u = 0.f, v = 0.f;
            if (2 * pr < P) {
                const float2 cs = lt_turn(c.pos[t], c.rot.freq[pr], c.rot.gain);
                const float *p = q + (size_t)t * row_q + h * (D + P) + D + 2 * pr;
                u = (p[0] * cs.x - p[1] * cs.y) * qs;
                v = (p[1] * cs.x + p[0] * cs.y) * qs;
            }
            const size_t at = ((size_t)t * s.heads + h) * s.row() + s.rank_pad + 2 * pr;
            lt_put<ACT>(qa, at, u, c.sat);
            lt_put<ACT>(qa, at + 1, v, c.sat);
        }
    }
    __syncthreads();
    const int per = (s.rank_pad + gridDim.y - 1) / gridDim.y, r1 = min((int)(blockIdx.y + 1) * per, s.rank_pad);
    const int piece = tid & 7, pieces = s.dim_pad / 8;
    constexpr int ROWS = LT_THREADS / 8, UR = TB == 1 ? 1 : 4;            // rows of a thread on their way at once
    for (int r0 = blockIdx.y * per; r0 < r1; r0 += UR * ROWS) {
        float acc[UR][TB];
        const uint16_t *wr[UR];
#pragma unroll
        for (int u = 0; u < UR; ++u) {
            wr[u] = w + ((size_t)h * s.rank_pad + min(r0 + u * ROWS + (tid >> 3), r1 - 1)) * s.dim_pad;
#pragma unroll
            for (int b = 0; b < TB; ++b) acc[u][b] = 0.f;
        }
#pragma unroll 2
        for (int p = piece; p < pieces; p += 8) {
            uint4 wv[UR];
#pragma unroll
            for (int u = 0; u < UR; ++u) wv[u] = *reinterpret_cast<const uint4 *>(wr[u] + p * 8);
#pragma unroll
            for (int u = 0; u < UR; ++u)
#pragma unroll
                for (int b = 0; b < TB; ++b) acc[u][b] = lt_dot8(wv[u], xs + b * s.dim_pad + p * 8, acc[u][b]);
        }
#pragma unroll
        for (int u = 0; u < UR; ++u) {
            const int r = r0 + u * ROWS + (tid >> 3);
#pragma unroll
            for (int b = 0; b < TB; ++b) {
                float v = acc[u][b];
                v += __shfl_xor(v, 1); v += __shfl_xor(v, 2); v += __shfl_xor(v, 4);
                if (piece == 0 && r < r1 && t0 + b < T) lt_put<ACT>(qa, ((size_t)(t0 + b) * s.heads + h) * s.row() + r, v, c.sat);
            }
        }
    }
}

// ---- attention over cache rows
template <ActType ACT> struct LtFrag;
template <> struct LtFrag<ACT_BF16> {
    lt_h8 v;
    __device__ __forceinline__ void load(const uint16_t *p) { v = __builtin_bit_cast(lt_h8, *reinterpret_cast<const uint4 *>(p)); }
};
template <> struct LtFrag<ACT_F32> {
    float4 a, b;
    __device__ __forceinline__ void load(const float *p) { a = *reinterpret_cast<const float4 *>(p); b = *reinterpret_cast<const float4 *>(p + 4); }
};
__device__ __forceinline__ lt_f4 lt_mma(const LtFrag<ACT_BF16> &a, const LtFrag<ACT_BF16> &b, lt_f4 acc) { return __builtin_amdgcn_mfma_f32_16x16x32_f16(a.v, b.v, acc, 0, 0, 0); }
__device__ __forceinline__ lt_f4 lt_mma(const LtFrag<ACT_F32> &x, const LtFrag<ACT_F32> &y, lt_f4 acc) {
    const float xf[8] = {x.a.x, x.a.y, x.a.z, x.a.w, x.b.x, x.b.y, x.b.z, x.b.w}, yf[8] = {y.a.x, y.a.y, y.a.z, y.a.w, y.b.x, y.b.y, y.b.z, y.b.w};
#pragma unroll
    for (int j = 0; j < 8; ++j) acc = __builtin_amdgcn_mfma_f32_16x16x4f32(xf[j], yf[j], acc, 0, 0, 0);
    return acc;
}

__host__ __device__ constexpr int lt_pitch(ActType act, int row) { return row + (act == ACT_F32 ? 4 : 8); }
// keys per split: whole steps
__host__ __device__ constexpr int lt_split_keys(int n_keys, int n_splits) { return ((n_keys + n_splits - 1) / n_splits + LT_KEYS - 1) / LT_KEYS * LT_KEYS; }

// key range of a group of tokens: positions ascend by one within it
__device__ __forceinline__ int lt_group_keys(const int32_t *pos, int t0, int tokens, int T) { return pos[min(t0 + tokens, T) - 1] + 1; }

// NR: rank_pad / 64.  TOK 1: a workgroup has one token, and each wave owns NR 16-row blocks of O^T.  TOK 4: it has four
// consecutive tokens of one sequence, a wave each, which share the staged rows.
template <ActType ACT, int NR, int TOK>
__global__ __launch_bounds__(LT_THREADS) void latent_attn_kernel(const LatentAttnArgs a, int heads, int rot_pad, int T) {
    typedef typename LtElem<ACT>::type E;
    constexpr int RANK = 64 * NR, NO = TOK == 1 ? NR : 4 * NR;
    extern __shared__ __align__(16) uint8_t smem[];
    const int row = RANK + rot_pad, pitch = lt_pitch(ACT, row);
    E *sK = reinterpret_cast<E *>(smem);                                                  // [LT_KEYS][pitch]
    uint32_t *sV = reinterpret_cast<uint32_t *>(smem + (size_t)LT_KEYS * pitch * sizeof(E));  // f16: [RANK][LT_VPITCH]
    const int tid = threadIdx.x, lane = tid & 63, wave = tid >> 6, c = lane & 15, g = lane >> 4;
    const int split = blockIdx.x, t0 = blockIdx.z * TOK, h = blockIdx.y * LATENT_HEADS_TILE + c;
    const bool live = TOK == 1 || t0 + wave < T;
    const int t = TOK == 1 ? t0 : live ? t0 + wave : T - 1;
    const int ob = TOK == 1 ? wave * NR : 0;                  // first 16-row block of this wave
    const int n_keys = lt_group_keys(a.pos, t0, TOK, T), mine = a.pos[t] + 1, per = lt_split_keys(n_keys, a.n_splits);
    const int j0 = split * per, j1 = min(j0 + per, n_keys), jm = min(j1, mine);
    const size_t prow = ((size_t)t * heads + h) * a.n_splits + split;
    if (j0 >= j1) {
        if ((TOK > 1 ? live && lane < 16 : tid < 16) && h < heads) { a.ml[prow * 2] = -INFINITY; a.ml[prow * 2 + 1] = 0.f; }
        return;
    }
    const E *rows = static_cast<const E *>(a.rows) + (size_t)a.seq[t] * a.n_ctx * row;
    // rows on their way to LDS (f16): 8 elements of two neighbouring keys per item; a thread fetches its items of a step while
    // the step before it is multiplied.  Rows past the split are zeros (their scores are masked below).
    constexpr int ITEMS = ACT == ACT_BF16 ? (2 * (RANK + 64) + LT_THREADS - 1) / LT_THREADS : 1;
    uint4 r0[ITEMS], r1[ITEMS];
    auto fetch_item = [&](int k0, int i, uint4 &x, uint4 &y) {
        const int key = k0 + 2 * (i & 15), d = (i >> 4) * 8;
        x = y = make_uint4(0, 0, 0, 0);
        if (key < j1) x = *reinterpret_cast<const uint4 *>(rows + (size_t)key * row + d);
        if (key + 1 < j1) y = *reinterpret_cast<const uint4 *>(rows + (size_t)(key + 1) * row + d);
    };
    auto put_item = [&](int i, const uint4 &x, const uint4 &y) {
        const int kp = i & 15, d = (i >> 4) * 8;
        *reinterpret_cast<uint4 *>(sK + (2 * kp) * pitch + d) = x;
        *reinterpret_cast<uint4 *>(sK + (2 * kp + 1) * pitch + d) = y;
        if (d >= RANK) return;
        const uint32_t w0[4] = {x.x, x.y, x.z, x.w}, w1[4] = {y.x, y.y, y.z, y.w};
        uint32_t *dst = sV + d * LT_VPITCH + kp;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            dst[(2 * e) * LT_VPITCH] = (w0[e] & 0xffffu) | (w1[e] << 16);
            dst[(2 * e + 1) * LT_VPITCH] = (w0[e] >> 16) | (w1[e] & 0xffff0000u);
        }
    };
    const int items = 2 * row;
    auto fetch = [&](int k0) {
#pragma unroll
        for (int n = 0; n < ITEMS; ++n)
            if (tid + n * LT_THREADS < items) fetch_item(k0, tid + n * LT_THREADS, r0[n], r1[n]);
    };
    if constexpr (ACT == ACT_BF16) fetch(j0);
    const E *qp = static_cast<const E *>(a.qa) + ((size_t)t * heads + (h < heads ? h : heads - 1)) * row + 8 * g;
    constexpr int NQ = ACT == ACT_BF16 ? 2 * NR : 1;
    LtFrag<ACT> qf[NQ];
    if constexpr (ACT == ACT_BF16) {
#pragma unroll
        for (int n = 0; n < NQ; ++n) qf[n].load(qp + 32 * n);
    }
    lt_f4 o[NO];
#pragma unroll
    for (int n = 0; n < NO; ++n) o[n] = lt_f4{0.f, 0.f, 0.f, 0.f};
    float m = -INFINITY, l = 0.f;
    for (int k0 = j0; k0 < j1; k0 += LT_KEYS) {
        if constexpr (ACT == ACT_BF16) {
#pragma unroll
            for (int n = 0; n < ITEMS; ++n)
                if (tid + n * LT_THREADS < items) put_item(tid + n * LT_THREADS, r0[n], r1[n]);
            for (int i = tid + ITEMS * LT_THREADS; i < items; i += LT_THREADS) {           // (rotated parts of more than 64)
                uint4 x, y;
                fetch_item(k0, i, x, y);
                put_item(i, x, y);
            }
        } else {
            const int pieces = row / 4;
            for (int i = tid; i < LT_KEYS * pieces; i += LT_THREADS) {
                const int kk = i / pieces, d = (i % pieces) * 4;
                float4 v = make_float4(0.f, 0.f, 0.f, 0.f);
                if (k0 + kk < j1) v = *reinterpret_cast<const float4 *>(rows + (size_t)(k0 + kk) * row + d);
                *reinterpret_cast<float4 *>(sK + kk * pitch + d) = v;
            }
        }
        __syncthreads();
        if constexpr (ACT == ACT_BF16) {
            if (k0 + LT_KEYS < j1) fetch(k0 + LT_KEYS);
        }
        lt_f4 s[2] = {lt_f4{0.f, 0.f, 0.f, 0.f}, lt_f4{0.f, 0.f, 0.f, 0.f}};
        auto score = [&](int kc, const LtFrag<ACT> &q) {
            LtFrag<ACT> kf;
#pragma unroll
            for (int b = 0; b < 2; ++b) {
                kf.load(sK + (16 * b + c) * pitch + kc + 8 * g);
                s[b] = lt_mma(kf, q, s[b]);
            }
        };
        auto score_at = [&](int kc) {
            LtFrag<ACT> q;
            q.load(qp + kc);
            score(kc, q);
        };
        if constexpr (ACT == ACT_BF16) {
#pragma unroll
            for (int n = 0; n < NQ; ++n) score(32 * n, qf[n]);
        } else {
            for (int kc = 0; kc < RANK; kc += 32) score_at(kc);
        }
        for (int kc = RANK; kc < row; kc += 32) score_at(kc);
        // register i of tile b: key k0 + 16 b + 4 g + i for head column c
        float mx = m;
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int i = 0; i < 4; ++i) {
                if (k0 + 16 * b + 4 * g + i >= jm) s[b][i] = -INFINITY;
                mx = fmaxf(mx, s[b][i]);
            }
        mx = fmaxf(mx, __shfl_xor(mx, 16));
        mx = fmaxf(mx, __shfl_xor(mx, 32));
        // (a token before the group's last may see no key of the split: all is -inf then, and the reference 0 gives zeros)
        const float ref = mx == -INFINITY ? 0.f : mx;
        const float corr = lt_exp2(m - ref);          // exp2(-inf) = 0 the first time
        m = mx;
        float p[2][4], ps = 0.f;
#pragma unroll
        for (int b = 0; b < 2; ++b)
#pragma unroll
            for (int i = 0; i < 4; ++i) { p[b][i] = lt_exp2(s[b][i] - ref); ps += p[b][i]; }
        l = l * corr + ps;                            // (this lane's keys only)
        if (__builtin_amdgcn_ballot_w64(corr != 1.0f) != 0ull) {
#pragma unroll
            for (int n = 0; n < NO; ++n) o[n] *= corr;
        }
        if constexpr (ACT == ACT_BF16) {
            // key slots of lane group g: keys 4g .. 4g + 3 of either tile, which is how P^T lies in the registers
            const lt_u4 pu = {lt_pack(p[0][0], p[0][1]), lt_pack(p[0][2], p[0][3]), lt_pack(p[1][0], p[1][1]), lt_pack(p[1][2], p[1][3])};
            const lt_h8 pf = __builtin_bit_cast(lt_h8, pu);
#pragma unroll
            for (int n = 0; n < NO; ++n) {
                const uint32_t *v = sV + (16 * (ob + n) + c) * LT_VPITCH + 2 * g;
                const uint2 a0 = *reinterpret_cast<const uint2 *>(v), a1 = *reinterpret_cast<const uint2 *>(v + 8);
                const lt_u4 vu = {a0.x, a0.y, a1.x, a1.y};
                o[n] = __builtin_amdgcn_mfma_f32_16x16x32_f16(__builtin_bit_cast(lt_h8, vu), pf, o[n], 0, 0, 0);
            }
        } else {
#pragma unroll
            for (int n = 0; n < NO; ++n)
#pragma unroll
                for (int b = 0; b < 2; ++b)
#pragma unroll
                    for (int i = 0; i < 4; ++i)
                        o[n] = __builtin_amdgcn_mfma_f32_16x16x4f32(sK[(16 * b + 4 * g + i) * pitch + 16 * (ob + n) + c], p[b][i], o[n], 0, 0, 0);
        }
        __syncthreads();
    }
    l += __shfl_xor(l, 16);
    l += __shfl_xor(l, 32);
    if (h >= heads || !live) return;
    if ((TOK > 1 || wave == 0) && g == 0) { a.ml[prow * 2] = m; a.ml[prow * 2 + 1] = l; }
#pragma unroll
    for (int n = 0; n < NO; ++n) *reinterpret_cast<float4 *>(a.part + prow * RANK + 16 * (ob + n) + 4 * g) = make_float4(o[n][0], o[n][1], o[n][2], o[n][3]);
}

// grid (heads, slices of the value rows, groups of TB tokens).  Sixteen lanes per weight row.
template <int TB>
__global__ __launch_bounds__(LT_THREADS) void latent_out_kernel(const LatentShape s, const LatentAttnArgs a, int T) {
    extern __shared__ __align__(16) uint8_t smem[];
    __shared__ float s_w[TB][ATTN_SPLITS_CAP];
    static_assert(ATTN_SPLITS_CAP == 64, "a lane per split");
    float *xs = reinterpret_cast<float *>(smem);              // [TB][rank_pad]
    const int h = blockIdx.x, t0 = blockIdx.z * TB, tid = threadIdx.x, lane = tid & 63, S = a.n_splits;
    for (int b = tid >> 6; b < TB; b += LT_WAVES) {
        const int t = min(t0 + b, T - 1), tg = t / a.group * a.group;          // the attention launch's group of this token
        const int n_keys = lt_group_keys(a.pos, tg, a.group, T), per = lt_split_keys(n_keys, S), live = (n_keys + per - 1) / per;      // splits that had keys
        const size_t row = (size_t)t * s.heads + h;
        const float m = lane < live ? a.ml[(row * S + lane) * 2] : -INFINITY, l = lane < live ? a.ml[(row * S + lane) * 2 + 1] : 0.f;
        float mh = m;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) mh = fmaxf(mh, __shfl_xor(mh, o));
        const float w = lane < live ? lt_exp2(m - mh) : 0.f;
        float den = l * w;
#pragma unroll
        for (int o = 32; o > 0; o >>= 1) den += __shfl_xor(den, o);
        s_w[b][lane] = w / den;
    }
    __syncthreads();
    int live = 0, last[TB];       // splits of the group's longest token (the others' weights end in zeros); every token's last one
#pragma unroll
    for (int b = 0; b < TB; ++b) {
        const int tg = min(t0 + b, T - 1) / a.group * a.group, n_keys = lt_group_keys(a.pos, tg, a.group, T), per = lt_split_keys(n_keys, S);
        last[b] = (n_keys + per - 1) / per - 1;
        live = max(live, last[b] + 1);
    }
    const float *part[TB];
#pragma unroll
    for (int b = 0; b < TB; ++b) part[b] = a.part + ((size_t)min(t0 + b, T - 1) * s.heads + h) * S * s.rank_pad;
    for (int r = tid * 2; r < s.rank_pad; r += LT_THREADS * 2) {
        float2 v[TB];
#pragma unroll
        for (int b = 0; b < TB; ++b) v[b] = make_float2(0.f, 0.f);
        constexpr int KB = TB == 1 ? 16 : 8;            // splits on their way at once
        for (int k0 = 0; k0 < live; k0 += KB) {
            float2 x[KB][TB];
#pragma unroll
            for (int k = 0; k < KB; ++k)
#pragma unroll
                for (int b = 0; b < TB; ++b) x[k][b] = *reinterpret_cast<const float2 *>(part[b] + (size_t)min(k0 + k, last[b]) * s.rank_pad + r);
#pragma unroll
            for (int k = 0; k < KB; ++k)
#pragma unroll
                for (int b = 0; b < TB; ++b) {
                    const float f = k0 + k < live ? s_w[b][k0 + k] : 0.f;
                    v[b].x = fmaf(x[k][b].x, f, v[b].x);
                    v[b].y = fmaf(x[k][b].y, f, v[b].y);
                }
        }
#pragma unroll
        for (int b = 0; b < TB; ++b) *reinterpret_cast<float2 *>(xs + b * s.rank_pad + r) = v[b];
    }
    __syncthreads();
    const int slice = (s.v_pad + gridDim.y - 1) / gridDim.y, v1 = min((int)(blockIdx.y + 1) * slice, s.v_pad);
    const int piece = tid & 15, pieces = s.rank_pad / 8;
    float gate[TB];
#pragma unroll
    for (int b = 0; b < TB; ++b) gate[b] = act_sigmoid(a.gate[(size_t)min(t0 + b, T - 1) * a.gate_ld + h]);
    constexpr int ROWS = LT_THREADS / 16, UR = TB == 1 ? 1 : 4;           // rows of a thread on their way at once
    for (int v0 = blockIdx.y * slice; v0 < v1; v0 += UR * ROWS) {
        const int v = v0 + (tid >> 4);
        float acc[UR][TB];
#pragma unroll
        for (int u = 0; u < UR; ++u)
#pragma unroll
            for (int b = 0; b < TB; ++b) acc[u][b] = 0.f;
        const int end = min(v1, s.vdim);          // (rows past the values are zeros)
#pragma unroll 4
        for (int p = piece; p < pieces; p += 16) {
            uint4 wv[UR];
#pragma unroll
            for (int u = 0; u < UR; ++u) {
                wv[u] = make_uint4(0, 0, 0, 0);
                if (v + u * ROWS < end) wv[u] = *reinterpret_cast<const uint4 *>(a.w_uv + ((size_t)h * s.vdim + v + u * ROWS) * s.rank_pad + p * 8);
            }
#pragma unroll
            for (int u = 0; u < UR; ++u)
#pragma unroll
                for (int b = 0; b < TB; ++b) acc[u][b] = lt_dot8(wv[u], xs + b * s.rank_pad + p * 8, acc[u][b]);
        }
#pragma unroll
        for (int u = 0; u < UR; ++u)
#pragma unroll
            for (int b = 0; b < TB; ++b) {
                float y = acc[u][b];
                y += __shfl_xor(y, 1); y += __shfl_xor(y, 2); y += __shfl_xor(y, 4); y += __shfl_xor(y, 8);
                if (piece == 0 && v + u * ROWS < v1 && t0 + b < T) {
                    const size_t at = ((size_t)(t0 + b) * s.heads + h) * s.v_pad + v + u * ROWS;
                    if (a.out_bf16) a.out_bf16[at] = f32_to_bf16_bits(y * gate[b]);
                    else a.out[at] = y * gate[b];
                }
            }
    }
}

// ---- many tokens of one sequence
// grid (heads, T), 64 threads
__global__ __launch_bounds__(64) void latent_chunk_query_kernel(const LatentShape s, const LatentRotary rot, const float *q, const int32_t *pos, float *out) {
    const int h = blockIdx.x, t = blockIdx.y;
    const float *p = q + ((size_t)t * s.heads + h) * (s.dim + s.rot_dim);
    float *o = out + ((size_t)t * s.heads + h) * s.chunk_k;
    for (int i = threadIdx.x; i < s.dim; i += 64) o[i] = p[i];
    for (int i = threadIdx.x; i < s.rot_dim / 2; i += 64) {
        const float2 w = lt_turn(pos[t], rot.freq[i], rot.gain);
        const float x = p[s.dim + 2 * i], y = p[s.dim + 2 * i + 1];
        o[s.dim + 2 * i] = x * w.x - y * w.y;
        o[s.dim + 2 * i + 1] = y * w.x + x * w.y;
    }
    for (int i = s.dim + s.rot_dim + threadIdx.x; i < s.chunk_k; i += 64) o[i] = 0.f;
}

// one workgroup per position
__global__ __launch_bounds__(LT_THREADS) void latent_chunk_rows_kernel(const uint16_t *rows, int row, int rank, uint16_t *out, int ld) {
    const uint16_t *p = rows + (size_t)blockIdx.x * row;
    for (int i = threadIdx.x; i < ld; i += LT_THREADS) out[(size_t)blockIdx.x * ld + i] = i < rank ? f32_to_bf16_bits(f16_bits_to_f32(p[i])) : 0;
}

// grid (position, groups of heads); pairs of neighbouring elements
__global__ __launch_bounds__(LT_THREADS) void latent_chunk_pack_kernel(const LatentShape s, const uint16_t *rows, int n_ctx, int k0, const float *kv, uint16_t *k16, uint16_t *v16, unsigned *sat) {
    const int key = k0 + blockIdx.x, per = s.chunk_k + s.chunk_v, H = s.heads;
    const float *y = kv + (size_t)blockIdx.x * H * (s.dim + s.vdim);
    const uint16_t *r = rows + (size_t)blockIdx.x * s.row() + s.rank_pad;
    auto f16 = [&](float v) {
        note_f16_clamp(sat, v, 0.f);
        return f32_to_f16_bits(fminf(fmaxf(v, -65504.f), 65504.f));
    };
    for (int i = (blockIdx.y * LT_THREADS + threadIdx.x) * 2; i < H * per; i += gridDim.y * LT_THREADS * 2) {
        const int h = i / per, e0 = i % per;
        uint16_t o[2];
#pragma unroll
        for (int j = 0; j < 2; ++j) {
            const int e = e0 + j;
            if (e0 < s.chunk_k) o[j] = e < s.dim ? f16(y[h * s.dim + e]) : e < s.dim + s.rot_dim ? r[e - s.dim] : 0;
            else o[j] = e - s.chunk_k < s.vdim ? f16(y[H * s.dim + h * s.vdim + e - s.chunk_k]) : 0;
        }
        uint16_t *dst = e0 < s.chunk_k ? k16 + ((size_t)h * n_ctx + key) * s.chunk_k + e0 : v16 + ((size_t)h * n_ctx + key) * s.chunk_v + e0 - s.chunk_k;
        *reinterpret_cast<uint32_t *>(dst) = (uint32_t)o[0] | ((uint32_t)o[1] << 16);
    }
}

// ------------------------------------------------------------------------------------------------ host
static size_t attn_lds(ActType act, const LatentShape &s) {
    const size_t k = (size_t)LT_KEYS * lt_pitch(act, s.row()) * (act == ACT_F32 ? 4 : 2);
    return act == ACT_F32 ? k : k + (size_t)s.rank_pad * LT_VPITCH * 4;
}

bool latent_shape(LatentShape &s) {
    if (s.heads < 1 || s.dim < 1 || s.vdim < 1 || s.rank < 1 || s.rot_dim < 2 || s.rot_dim % 2) return false;
    s.rank_pad = 64;
    while (s.rank_pad < s.rank) s.rank_pad *= 2;
    s.rot_pad = (s.rot_dim + 31) / 32 * 32;
    s.dim_pad = (s.dim + 7) / 8 * 8;
    const int k = s.dim + s.rot_dim;
    s.chunk_k = s.chunk_v = 0;
    if (s.vdim <= 128 && k <= 192) {
        s.chunk_k = k <= 64 && s.vdim <= 64 ? 64 : k <= 128 ? 128 : 192;
        s.chunk_v = s.vdim <= 64 && s.chunk_k < 192 ? 64 : 128;
    }
    s.v_pad = s.chunk_v ? s.chunk_v : (s.vdim + 63) / 64 * 64;
    return s.rank_pad <= 1024 && s.dim_pad <= 4096 && attn_lds(ACT_BF16, s) <= LT_LDS_MAX && attn_lds(ACT_F32, s) <= LT_LDS_MAX;
}

int latent_rows(const LatentShape &s, const LatentCache &cache, ActType act, const float *in, int ld, const float *gain, int n, void *out, int ld_out, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!in || !gain || !out || ld < n || ld_out < n || (cache.in && (!cache.rows || !cache.gain || !cache.rot.freq))) return fail(MESH_ERR_INVALID, "latent_rows: bad operands");
    if (act == ACT_BF16) MESH_LAUNCH((latent_rows_kernel<ACT_BF16>), dim3((unsigned)T), dim3(LT_THREADS), 0, stream, s, cache, in, ld, gain, n, out, ld_out);
    else MESH_LAUNCH((latent_rows_kernel<ACT_F32>), dim3((unsigned)T), dim3(LT_THREADS), 0, stream, s, cache, in, ld, gain, n, out, ld_out);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int latent_query(const LatentShape &s, const LatentCache &cache, ActType act, const float *q, const uint16_t *w_uk_t, float scale, bool append, void *qa, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!q || !w_uk_t || !qa || !cache.rot.freq || (append && (!cache.in || !cache.rows || !cache.gain))) return fail(MESH_ERR_INVALID, "latent_query: bad operands");
    const int tb = T == 1 ? 1 : LT_QUERY_TOKENS, groups = (T + tb - 1) / tb;
    // enough workgroups to fill the chip, at least one pass of rows each
    const int slices = std::max(1, std::min(s.rank_pad / (LT_THREADS / 8), 512 / std::max(1, s.heads * groups)));
    const dim3 grid((unsigned)(s.heads + (append ? 1 : 0)), (unsigned)slices, (unsigned)groups), block(LT_THREADS);
    const size_t lds = (size_t)tb * s.dim_pad * sizeof(float);
    if (act == ACT_BF16 && tb == 1) MESH_LAUNCH((latent_query_kernel<ACT_BF16, 1>), grid, block, lds, stream, s, cache, q, w_uk_t, scale, qa, T);
    else if (act == ACT_BF16) MESH_LAUNCH((latent_query_kernel<ACT_BF16, LT_QUERY_TOKENS>), grid, block, lds, stream, s, cache, q, w_uk_t, scale, qa, T);
    else if (tb == 1) MESH_LAUNCH((latent_query_kernel<ACT_F32, 1>), grid, block, lds, stream, s, cache, q, w_uk_t, scale, qa, T);
    else MESH_LAUNCH((latent_query_kernel<ACT_F32, LT_QUERY_TOKENS>), grid, block, lds, stream, s, cache, q, w_uk_t, scale, qa, T);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int latent_group(const LatentShape &s, int T, bool one_run) { return one_run && T > 1 && s.rank_pad <= 512 ? LATENT_GROUP : 1; }

int latent_splits(const LatentShape &s, int T, int group, int max_keys, int target) {
    const int wgs = (T + group - 1) / group * latent_head_tiles(s);
    const int n = std::min((target ? target : 256) / std::max(1, wgs), (max_keys + LT_KEYS - 1) / LT_KEYS);
    return std::max(1, std::min(n, ATTN_SPLITS_CAP));
}

template <ActType ACT, int NR, int TOK>
static int launch_attn(const LatentShape &s, const LatentAttnArgs &a, int T, hipStream_t stream) {
    static bool ready = false;        // (hosts are single-threaded per session; a second thread sets the same attribute)
    if (!ready) {
        MESH_HIP_TRY(hipFuncSetAttribute(reinterpret_cast<const void *>(latent_attn_kernel<ACT, NR, TOK>), hipFuncAttributeMaxDynamicSharedMemorySize, (int)LT_LDS_MAX));
        ready = true;
    }
    MESH_LAUNCH((latent_attn_kernel<ACT, NR, TOK>), dim3((unsigned)a.n_splits, (unsigned)latent_head_tiles(s), (unsigned)((T + TOK - 1) / TOK)), dim3(LT_THREADS), attn_lds(ACT, s), stream, a,
                s.heads, s.rot_pad, T);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}
template <ActType ACT, int NR>
static int launch_attn_group(const LatentShape &s, const LatentAttnArgs &a, int T, hipStream_t stream) {
    if (a.group == 1) return launch_attn<ACT, NR, 1>(s, a, T, stream);
    if constexpr (NR <= 8) return launch_attn<ACT, NR, LATENT_GROUP>(s, a, T, stream);
    return fail(MESH_ERR_UNSUPPORTED, "latent_attention: no grouped kernel for a rank of %d", s.rank);
}
template <ActType ACT>
static int launch_attn_rank(const LatentShape &s, const LatentAttnArgs &a, int T, hipStream_t stream) {
    switch (s.rank_pad) {
        case 64: return launch_attn_group<ACT, 1>(s, a, T, stream);
        case 128: return launch_attn_group<ACT, 2>(s, a, T, stream);
        case 256: return launch_attn_group<ACT, 4>(s, a, T, stream);
        case 512: return launch_attn_group<ACT, 8>(s, a, T, stream);
        case 1024: return launch_attn_group<ACT, 16>(s, a, T, stream);
        default: return fail(MESH_ERR_UNSUPPORTED, "latent_attention: no kernel for a rank of %d", s.rank);
    }
}

int latent_attention(const LatentShape &s, const LatentAttnArgs &a, ActType act, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!a.qa || !a.rows || !a.part || !a.ml || a.n_splits < 1 || a.n_splits > ATTN_SPLITS_CAP || T > 65535 || (a.group != 1 && a.group != LATENT_GROUP))
        return fail(MESH_ERR_INVALID, "latent_attention: bad operands");
    return act == ACT_BF16 ? launch_attn_rank<ACT_BF16>(s, a, T, stream) : launch_attn_rank<ACT_F32>(s, a, T, stream);
}

int latent_out(const LatentShape &s, const LatentAttnArgs &a, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!a.w_uv || !a.gate || (!a.out && !a.out_bf16) || a.n_splits > ATTN_SPLITS_CAP || T > 65535) return fail(MESH_ERR_INVALID, "latent_out: bad operands");
    const int tb = T == 1 ? 1 : LT_QUERY_TOKENS, groups = (T + tb - 1) / tb;
    const int slices = std::max(1, std::min(s.v_pad / (LT_THREADS / 16), 256 / std::max(1, s.heads * groups)));
    const dim3 grid((unsigned)s.heads, (unsigned)slices, (unsigned)groups), block(LT_THREADS);
    const size_t lds = (size_t)tb * s.rank_pad * sizeof(float);
    if (tb == 1) MESH_LAUNCH((latent_out_kernel<1>), grid, block, lds, stream, s, a, T);
    else MESH_LAUNCH((latent_out_kernel<LT_QUERY_TOKENS>), grid, block, lds, stream, s, a, T);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int latent_chunk_query(const LatentShape &s, const LatentRotary &rot, const float *q, const int32_t *pos, float *out, int T, hipStream_t stream) {
    if (T <= 0) return MESH_OK;
    if (!s.chunk_k || T > 65535) return fail(MESH_ERR_INVALID, "latent_chunk_query: bad operands");
    MESH_LAUNCH(latent_chunk_query_kernel, dim3((unsigned)s.heads, (unsigned)T), dim3(64), 0, stream, s, rot, q, pos, out);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int latent_chunk_rows(const LatentShape &s, const void *rows, int n_ctx, int seq, int k0, int n, uint16_t *out, int ld, hipStream_t stream) {
    if (n <= 0) return MESH_OK;
    if (k0 < 0 || k0 + n > n_ctx || ld < s.rank) return fail(MESH_ERR_INVALID, "latent_chunk_rows: bad operands");
    const uint16_t *p = static_cast<const uint16_t *>(rows) + ((size_t)seq * n_ctx + k0) * s.row();
    MESH_LAUNCH(latent_chunk_rows_kernel, dim3((unsigned)n), dim3(LT_THREADS), 0, stream, p, s.row(), s.rank, out, ld);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

int latent_chunk_pack(const LatentShape &s, const void *rows, int n_ctx, int seq, int k0, int n, const float *kv, uint16_t *k16, uint16_t *v16, unsigned *sat, hipStream_t stream) {
    if (n <= 0) return MESH_OK;
    if (!s.chunk_k || k0 < 0 || k0 + n > n_ctx) return fail(MESH_ERR_INVALID, "latent_chunk_pack: bad operands");
    const uint16_t *p = static_cast<const uint16_t *>(rows) + ((size_t)seq * n_ctx + k0) * s.row();
    const int cols = s.heads * (s.chunk_k + s.chunk_v) / 2;
    MESH_LAUNCH(latent_chunk_pack_kernel, dim3((unsigned)n, (unsigned)std::max(1, std::min(4, cols / LT_THREADS))), dim3(LT_THREADS), 0, stream, s, p, n_ctx, k0, kv, k16, v16, sat);
    MESH_LAUNCH_CHECK();
    return MESH_OK;
}

}  // namespace mesh
