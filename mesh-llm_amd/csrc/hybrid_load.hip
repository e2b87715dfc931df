// Weights of a model folder on the device (hybrid.hpp).
#include <algorithm>
#include <cmath>
#include <cstring>

#include "hybrid.hpp"
#include "registry.hpp"
#include "safetensors.hpp"
#include "stage.hpp"

namespace mesh {

namespace {

typedef std::vector<uint64_t> Shape;

struct FolderLoader {
    const SafetensorsFile &f;
    mesh_stage &st;

    int dev_alloc(void **p, size_t bytes) {
        hipError_t e = hipMalloc(p, bytes ? bytes : 16);
        if (e != hipSuccess) return fail(e == hipErrorOutOfMemory ? MESH_ERR_NOMEM : MESH_ERR_DEVICE, "hipMalloc(%zu) failed: %s", bytes, hipGetErrorString(e));
        st.allocations.push_back(*p);
        return MESH_OK;
    }
    // bf16 tensor of exactly this shape
    int get(const std::string &name, const Shape &shape, const uint16_t *&data) {
        const SafeTensor *t = f.find(name);
        if (!t) return fail(MESH_ERR_FORMAT, "model.safetensors: tensor '%s' not found", name.c_str());
        if (t->dtype != "BF16") return fail(MESH_ERR_UNSUPPORTED, "model.safetensors: tensor '%s' is %s (BF16 expected)", name.c_str(), t->dtype.c_str());
        if (t->shape != shape) {
            std::string have, want;
            for (uint64_t d : t->shape) have += std::to_string(d) + " ";
            for (uint64_t d : shape) want += std::to_string(d) + " ";
            return fail(MESH_ERR_FORMAT, "model.safetensors: tensor '%s' has shape [ %s], expected [ %s]", name.c_str(), have.c_str(), want.c_str());
        }
        data = reinterpret_cast<const uint16_t *>(f.data(*t));       // (read with memcpy only: the file does not promise alignment)
        st.weight_bytes += t->nbytes;
        return MESH_OK;
    }
    // the tensor as f32 on the host
    int floats(const std::string &name, const Shape &shape, std::vector<float> &out) {
        const uint16_t *d = nullptr;
        int rc = get(name, shape, d);
        if (rc != MESH_OK) return rc;
        size_t n = 1;
        for (uint64_t v : shape) n *= v;
        out.resize(n);
        for (size_t i = 0; i < n; ++i) {
            uint16_t b;
            memcpy(&b, reinterpret_cast<const uint8_t *>(d) + 2 * i, 2);
            const uint32_t u = (uint32_t)b << 16;
            memcpy(&out[i], &u, 4);
        }
        return MESH_OK;
    }
    int upload(const std::vector<float> &v, float **out) {
        void *p = nullptr;
        int rc = dev_alloc(&p, v.size() * sizeof(float));
        if (rc != MESH_OK) return rc;
        MESH_HIP_TRY(hipMemcpy(p, v.data(), v.size() * sizeof(float), hipMemcpyHostToDevice));
        *out = static_cast<float *>(p);
        return MESH_OK;
    }
    int raw(const std::string &name, const Shape &shape, uint16_t **out) {
        const uint16_t *d = nullptr;
        int rc = get(name, shape, d);
        if (rc != MESH_OK) return rc;
        size_t n = 2;
        for (uint64_t v : shape) n *= v;
        void *p = nullptr;
        if ((rc = dev_alloc(&p, n)) != MESH_OK) return rc;
        MESH_HIP_TRY(hipMemcpy(p, d, n, hipMemcpyHostToDevice));
        *out = static_cast<uint16_t *>(p);
        return MESH_OK;
    }
    int matrix_alloc(LinearWeight &W, int M, int K) {
        W.M = M; W.K = K; W.Mp = linear_rows_padded(M); W.Kp = linear_k_padded(K);
        void *p = nullptr;
        int rc = dev_alloc(&p, (size_t)W.Mp * W.Kp * 2);
        if (rc != MESH_OK) return rc;
        MESH_HIP_TRY(hipMemset(p, 0, (size_t)W.Mp * W.Kp * 2));
        W.w = static_cast<const uint16_t *>(p);
        return MESH_OK;
    }
    static int copy(uint16_t *dst, size_t dpitch, const uint8_t *src, size_t spitch, size_t width, size_t rows) {
        if (dpitch == spitch && width == spitch) MESH_HIP_TRY(hipMemcpy(dst, src, width * rows, hipMemcpyHostToDevice));
        else MESH_HIP_TRY(hipMemcpy2D(dst, dpitch, src, spitch, width, rows, hipMemcpyHostToDevice));
        return MESH_OK;
    }
    // [rows][cols] into W from row `row0` on; blocks of rb rows are placed rp rows apart, blocks of cb columns cp columns apart
    int place(LinearWeight &W, const std::string &name, int rows, int cols, int row0, int rb, int rp, int cb, int cp) {
        const uint16_t *d = nullptr;
        int rc = get(name, {(uint64_t)rows, (uint64_t)cols}, d);
        if (rc != MESH_OK) return rc;
        if (rb == rp) { rb = rp = rows; }
        if (cb == cp) { cb = cp = cols; }
        uint16_t *w = const_cast<uint16_t *>(W.w);
        for (int r = 0, br = 0; r < rows; r += rb, ++br)
            for (int c = 0, bc = 0; c < cols; c += cb, ++bc) {
                rc = copy(w + (size_t)(row0 + br * rp) * W.Kp + (size_t)bc * cp, (size_t)W.Kp * 2, reinterpret_cast<const uint8_t *>(d) + ((size_t)r * cols + c) * 2, (size_t)cols * 2,
                          (size_t)cb * 2, (size_t)rb);
                if (rc != MESH_OK) return rc;
            }
        return MESH_OK;
    }
    int matrix(LinearWeight &W, const std::string &name, int M, int K) {
        int rc = matrix_alloc(W, M, K);
        return rc != MESH_OK ? rc : place(W, name, M, K, 0, M, M, K, K);
    }
    int vector(const std::string &name, int n, float **out, float factor = 1.f) {
        std::vector<float> v;
        int rc = floats(name, {(uint64_t)n}, v);
        if (rc != MESH_OK) return rc;
        for (float &x : v) x *= factor;
        return upload(v, out);
    }
    // output norm (one number) times the layer scale
    int scaled_rms(const std::string &norm, const std::string &scale, int n, RowNorm &out) {
        std::vector<float> g, s;
        float *p = nullptr;
        int rc;
        if ((rc = floats(norm, {}, g)) || (rc = floats(scale, {(uint64_t)n}, s))) return rc;
        for (float &v : s) v *= g[0];
        out.kind = NORM_RMS;
        rc = upload(s, &p);
        out.gain = p;
        return rc;
    }
    // layer norm whose result is multiplied by `factor`
    int layer_norm(const std::string &name, int n, float factor, RowNorm &out) {
        float *g = nullptr, *b = nullptr;
        int rc;
        if ((rc = vector(name, n, &g, factor)) || (rc = vector(name + ".b", n, &b, factor))) return rc;
        out.kind = NORM_LAYER;
        out.gain = g; out.bias = b;
        return MESH_OK;
    }
    // bf16 matrices [heads][rows][cols] of a tensor [heads * rows][cols], transposed or not, as [heads][R][C] with zeros around
    int per_head(const std::string &name, int heads, int rows, int cols, bool transposed, int R, int C, uint16_t **out) {
        const uint16_t *d = nullptr;
        int rc = get(name, {(uint64_t)heads * rows, (uint64_t)cols}, d);
        if (rc != MESH_OK) return rc;
        std::vector<uint16_t> v((size_t)heads * R * C, 0);
        for (int h = 0; h < heads; ++h)
            for (int r = 0; r < rows; ++r)
                for (int c = 0; c < cols; ++c) {
                    uint16_t b;
                    memcpy(&b, reinterpret_cast<const uint8_t *>(d) + 2 * (((size_t)h * rows + r) * cols + c), 2);
                    v[((size_t)h * R + (transposed ? c : r)) * C + (transposed ? r : c)] = b;
                }
        void *p = nullptr;
        if ((rc = dev_alloc(&p, v.size() * 2)) != MESH_OK) return rc;
        MESH_HIP_TRY(hipMemcpy(p, v.data(), v.size() * 2, hipMemcpyHostToDevice));
        *out = static_cast<uint16_t *>(p);
        return MESH_OK;
    }
    // rows of several tensors, one below the other
    int stacked(LinearWeight &W, const std::vector<std::pair<std::string, int>> &parts, int K) {
        int M = 0, rc;
        for (const auto &p : parts) M += p.second;
        if ((rc = matrix_alloc(W, M, K)) != MESH_OK) return rc;
        int row = 0;
        for (const auto &p : parts) {
            if ((rc = place(W, p.first, p.second, K, row, p.second, p.second, K, K)) != MESH_OK) return rc;
            row += p.second;
        }
        return MESH_OK;
    }
    int latent_layer(HybridLayer &L, const ModelSpec &s, int index, int local, const std::string &mx) {
        const MixerSpec &m = L.spec.mixer;
        const int E = s.width, H = m.heads;
        LatentShape &ls = L.latent;
        ls.heads = H; ls.dim = m.dim; ls.rot_dim = m.rot_dim; ls.vdim = m.vdim; ls.rank = m.kv_rank;
        if (!latent_shape(ls))
            return fail(MESH_ERR_UNSUPPORTED, "layer %d: latent attention of rank %d with %d + %d key entries has no kernel", index, m.kv_rank, m.dim, m.rot_dim);
        L.cache_layer = m.kv_from >= 0 ? local - (index - m.kv_from) : local;
        if (L.cache_layer < 0)
            return fail(MESH_ERR_UNSUPPORTED, "layer %d reads the cache of layer %d, which lies before the stage's layers", index, m.kv_from);
        std::vector<std::pair<std::string, int>> in = {{mx + "dq", m.q_rank}};
        if (m.kv_from < 0) in.push_back({mx + "dkv", m.kv_rank + m.rot_dim});
        in.push_back({mx + "g", H});
        int rc;
        if ((rc = stacked(L.in, in, E)) || (rc = vector(mx + "dq.norm", m.q_rank, &L.cq_norm)) || (rc = matrix(L.uq, mx + "uq", H * (m.dim + m.rot_dim), m.q_rank)) ||
            (rc = per_head(mx + "uk", H, m.dim, m.kv_rank, true, ls.rank_pad, ls.dim_pad, &L.w_uk_t)) ||
            (rc = per_head(mx + "uv", H, m.vdim, m.kv_rank, false, m.vdim, ls.rank_pad, &L.w_uv)))
            return rc;
        if (m.kv_from < 0 && (rc = vector(mx + "dkv.norm", m.kv_rank, &L.c_norm)) != MESH_OK) return rc;
        if (ls.chunk_k && st.hybrid->act == ACT_BF16) {
            const size_t counted = st.weight_bytes;           // (a second copy)
            rc = stacked(L.ukv, {{mx + "uk", H * m.dim}, {mx + "uv", H * m.vdim}}, m.kv_rank);
            st.weight_bytes = counted;
            if (rc != MESH_OK) return rc;
        }
        std::vector<double> f((size_t)m.rot_dim / 2);
        for (size_t i = 0; i < f.size(); ++i) f[i] = m.rot.freq((int)i);
        void *p = nullptr;
        if ((rc = dev_alloc(&p, f.size() * sizeof(double))) != MESH_OK) return rc;
        MESH_HIP_TRY(hipMemcpy(p, f.data(), f.size() * sizeof(double), hipMemcpyHostToDevice));
        L.rot.freq = static_cast<const double *>(p);
        L.rot.gain = m.rot.gain();
        if ((rc = matrix_alloc(L.out, E, H * ls.v_pad)) != MESH_OK) return rc;
        return place(L.out, mx + "o", E, H * m.vdim, 0, E, E, m.vdim, ls.v_pad);
    }
    int gated_layer(HybridLayer &L, const ModelSpec &s, int index, const std::string &mx) {
        const MixerSpec &m = L.spec.mixer;
        const int E = s.width, qk = m.kv_heads * m.dim, v = m.heads * m.vdim;
        GatedStateArgs &g = L.gated;
        if (!gated_state_supported(m.dim, m.vdim))
            return fail(MESH_ERR_UNSUPPORTED, "layer %d: states of %d x %d have no kernel (%d at most)", index, m.dim, m.vdim, STATE_DIM_MAX);
        g.delta = m.kind == MIXER_DELTA;
        g.heads = m.heads; g.kv_heads = m.kv_heads; g.dim = m.dim; g.vdim = m.vdim; g.eps = s.eps;
        g.at_q = 0; g.at_k = qk; g.at_v = 2 * qk; g.at_g = 2 * qk + v;
        std::vector<std::pair<std::string, int>> in = {{mx + "q", qk}, {mx + "k", qk}, {mx + "v", v}, {mx + "g", v}};
        int rc;
        float *p = nullptr, *q = nullptr, *r = nullptr;
        if (g.delta) {
            g.taps = m.taps;
            g.at_b = g.at_g + v; g.at_a = g.at_b + m.heads;
            in.push_back({mx + "b", m.heads});
            in.push_back({mx + "a", m.heads});
            std::vector<float> A;
            if ((rc = floats(mx + "A_log", {(uint64_t)m.heads}, A)) != MESH_OK) return rc;
            for (float &x : A) x = expf(x);
            if ((rc = upload(A, &p)) || (rc = vector(mx + "dt_bias", m.heads, &q))) return rc;
            g.A = p; g.dt_bias = q;
            if ((rc = table(mx + "q.conv", qk, m.taps, &p)) || (rc = table(mx + "k.conv", qk, m.taps, &q)) || (rc = table(mx + "v.conv", v, m.taps, &r))) return rc;
            g.conv_q = p; g.conv_k = q; g.conv_v = r;
        } else {
            const SafeTensor *a1 = f.find(mx + "a1");
            if (!a1 || a1->shape.size() != 2 || a1->shape[0] < 1 || a1->shape[0] > 4096) return fail(MESH_ERR_FORMAT, "model.safetensors: tensor '%sa1' not found or not a matrix", mx.c_str());
            g.rank = (int)a1->shape[0];
            if (g.rank > STATE_RANK_MAX) return fail(MESH_ERR_UNSUPPORTED, "layer %d: a decay projection of rank %d has no kernel (%d at most)", index, g.rank, STATE_RANK_MAX);
            g.at_a = g.at_g + v;
            g.inv_tau = 1.0f / m.tau;
            in.push_back({mx + "a1", g.rank});
            if ((rc = table(mx + "a2", qk, g.rank, &p)) || (rc = vector(mx + "a2.b", qk, &q))) return rc;
            g.a2 = p; g.a2_bias = q;
        }
        if ((rc = stacked(L.in, in, E)) || (rc = vector(mx + "norm", m.vdim, &p)) || (rc = matrix(L.out, mx + "o", E, v))) return rc;
        g.norm = p;
        g.ld = L.in.M;
        g.ld_out = L.out.Kp;
        return MESH_OK;
    }
    int table(const std::string &name, int rows, int cols, float **out) {
        std::vector<float> v;
        const int rc = floats(name, {(uint64_t)rows, (uint64_t)cols}, v);
        return rc != MESH_OK ? rc : upload(v, out);
    }
    int head_norm(const std::string &name, int heads, int dim, int pad, float **out) {
        std::vector<float> g, p((size_t)heads * pad, 0.f);
        int rc = floats(name, {(uint64_t)heads * dim}, g);
        if (rc != MESH_OK) return rc;
        for (int h = 0; h < heads; ++h)
            for (int i = 0; i < dim; ++i) p[(size_t)h * pad + i] = g[(size_t)h * dim + i];
        return upload(p, out);
    }
    int layer(HybridLayer &L, const ModelSpec &s, int index, int local) {
        const std::string p = "l" + std::to_string(index) + ".", mx = p + "mix.";
        const MixerSpec &m = L.spec.mixer;
        const int E = s.width;
        int rc;
        if (m.kind == MIXER_ATTENTION) {
            L.head_pad = m.dim <= 64 ? 64 : m.dim <= 128 ? 128 : 256;
            if (m.dim > 256) return fail(MESH_ERR_UNSUPPORTED, "layer %d: attention heads of %d entries have no kernel (256 at most)", index, m.dim);
            const int HP = m.heads * L.head_pad, GP = m.kv_heads * L.head_pad;
            if ((rc = matrix_alloc(L.in, HP + GP, E)) || (rc = place(L.in, mx + "q", m.heads * m.dim, E, 0, m.dim, L.head_pad, E, E)) ||
                (rc = place(L.in, mx + "k", m.kv_heads * m.dim, E, HP, m.dim, L.head_pad, E, E)) ||
                (rc = head_norm(mx + "q.norm", m.heads, m.dim, L.head_pad, &L.q_norm)) || (rc = head_norm(mx + "k.norm", m.kv_heads, m.dim, L.head_pad, &L.k_norm)) ||
                (rc = matrix_alloc(L.out, E, HP)) || (rc = place(L.out, mx + "o", E, m.heads * m.dim, 0, E, E, m.dim, L.head_pad)))
                return rc;
        } else if (m.kind == MIXER_LATENT) {
            if ((rc = latent_layer(L, s, index, local, mx)) != MESH_OK) return rc;
        } else if (m.has_matrix_state()) {
            if ((rc = gated_layer(L, s, index, mx)) != MESH_OK) return rc;
        } else {
            const int W = m.width;
            std::vector<float> bz, bx;
            if ((rc = matrix_alloc(L.in, 3 * W, E)) || (rc = place(L.in, mx + "z", W, E, 0, W, W, E, E)) || (rc = place(L.in, mx + "x", W, E, W, W, W, E, E)) ||
                (rc = place(L.in, mx + "g", W, E, 2 * W, W, W, E, E)) || (rc = floats(mx + "z.b", {(uint64_t)W}, bz)) || (rc = floats(mx + "x.b", {(uint64_t)W}, bx)) ||
                (rc = upload(bz, &L.bias_z)) || (rc = upload(bx, &L.bias_x)) || (rc = matrix(L.out, mx + "o", E, W)))
                return rc;
        }
        const bool ln = s.out_norm == NORM_LAYER;
        if (s.in_norm == NORM_LAYER && ((rc = layer_norm(p + "norm1", E, 1.f, L.pre1)) || (L.spec.ff && (rc = layer_norm(p + "norm2", E, 1.f, L.pre2))))) return rc;
        if ((rc = ln ? layer_norm(p + "norm1b", E, s.residual_mult, L.post1) : scaled_rms(p + "norm1", p + "ls1", E, L.post1)) != MESH_OK) return rc;
        if (L.spec.ff) {
            if ((rc = matrix(L.up, p + "mlp.up", L.spec.ff, E)) || (rc = matrix(L.down, p + "mlp.down", E, L.spec.ff)) ||
                (rc = ln ? layer_norm(p + "norm2b", E, s.residual_mult, L.post2) : scaled_rms(p + "norm2", p + "ls2", E, L.post2)))
                return rc;
            if (s.ff == FF_POLY_NORM && (rc = vector(p + "mlp.act", 4, &L.coef)) != MESH_OK) return rc;
        }
        if (s.side_dim) {
            float *g = nullptr;
            if ((rc = matrix(L.side_gate, p + "side.gate", s.side_dim, E)) || (rc = matrix(L.side_proj, p + "side.proj", E, s.side_dim)) || (rc = vector(p + "side.norm", E, &g))) return rc;
            L.post_side.kind = NORM_RMS;
            L.post_side.gain = g;
        }
        return MESH_OK;
    }
};

}  // namespace

int hybrid_open(const char *folder, int layer_begin, int layer_end, const mesh_stage_opts *opts, mesh_stage *st) {
    st->hybrid.reset(new HybridModel());
    HybridModel &hm = *st->hybrid;
    ModelSpec &s = hm.spec;
    int rc = model_spec_from_folder(folder, s);
    if (rc != MESH_OK) return rc;
    hparams_from_spec(s, st->hp);
    const int n_layer = (int)s.layers.size();
    if (layer_end < 0) layer_end = n_layer;
    if (layer_begin < 0 || layer_begin >= layer_end || layer_end > n_layer)
        return fail(MESH_ERR_INVALID, "mesh_stage_open: layer range [%d,%d) does not fit a %d-layer model", layer_begin, layer_end, n_layer);
    st->layer_begin = layer_begin;
    st->layer_end = layer_end;
    if (opts && (opts->kv_type || opts->kv_type_v))
        return fail(MESH_ERR_UNSUPPORTED, "mesh_stage_open: the cache rows of architecture '%s' follow its precision (no kv_type)", s.arch.c_str());
    hm.act = opts && opts->precision == MESH_PRECISION_F32 ? ACT_F32 : ACT_BF16;
    st->k_type = st->v_type = hm.act == ACT_F32 ? MESH_F32 : MESH_F16;
    SafetensorsFile f;
    if ((rc = f.open((std::string(folder) + "/model.safetensors").c_str())) != MESH_OK) return rc;
    if ((rc = stage_select_device(opts, st)) != MESH_OK) return rc;

    FolderLoader ld{f, *st};
    const int E = s.width;
    hm.width_pad = linear_k_padded(E);
    hm.layers.resize((size_t)(layer_end - layer_begin));
    for (int i = layer_begin; i < layer_end; ++i) {
        HybridLayer &L = hm.layers[(size_t)(i - layer_begin)];
        L.spec = s.layers[(size_t)i];
        if ((rc = ld.layer(L, s, i, i - layer_begin)) != MESH_OK) return rc;
        const MixerSpec &m = L.spec.mixer;
        hm.in_max = std::max({hm.in_max, L.in.M, s.ff == FF_POLY_NORM ? L.up.M : 0, L.side_gate.M * LINEAR_SLICES_MAX});
        hm.act_max = std::max({hm.act_max, L.out.Kp, L.down.Kp, L.side_proj.Kp, L.uq.Kp, L.ukv.Kp, s.ff == FF_RELU2 ? L.up.M : 0});
        if (m.kind == MIXER_ATTENTION) {
            hm.q_max = std::max(hm.q_max, m.heads * L.head_pad);
            hm.part_max = std::max(hm.part_max, (size_t)m.heads * L.head_pad);
        } else if (m.kind == MIXER_LATENT) {
            const LatentShape &ls = L.latent;
            hm.q_max = std::max(hm.q_max, m.heads * (m.dim + m.rot_dim));
            hm.part_max = std::max(hm.part_max, (size_t)m.heads * std::max(ls.rank_pad, ls.chunk_v));
            hm.qx_max = std::max(hm.qx_max, (size_t)m.heads * ls.row() * (hm.act == ACT_F32 ? 4 : 2));
            if (L.ukv.present()) {
                hm.qx_max = std::max(hm.qx_max, (size_t)m.heads * ls.chunk_k * sizeof(float));
                hm.kvx_max = std::max(hm.kvx_max, (size_t)L.ukv.M);
                hm.kv16_max = std::max(hm.kv16_max, (size_t)m.heads * (ls.chunk_k + ls.chunk_v));
            }
        } else if (m.has_matrix_state()) {
            hm.has_chunks = true;
            hm.q_max = std::max(hm.q_max, m.heads * m.vdim);
            hm.gated_ws_max = std::max(hm.gated_ws_max, gated_state_workspace(1, m.heads, m.dim, m.vdim));
        } else {
            hm.state_max = std::max(hm.state_max, m.width);
        }
        if (m.has_state()) hm.has_state = true;
        for (const LinearWeight *w : {&L.in, &L.out, &L.up, &L.down, &L.side_gate, &L.side_proj, &L.uq})
            if (w->present() && !linear_step_supported(*w)) hm.step_ok = false;
    }
    if (hm.side() && (rc = ld.raw("side.embed", {(uint64_t)s.vocab, (uint64_t)n_layer * s.side_dim}, &hm.side_embed)) != MESH_OK) return rc;
    const bool begins = layer_begin == 0, ends = layer_end == n_layer;
    if (ends) {
        if ((rc = ld.matrix(hm.head, s.tied_head ? "embed" : "head", s.vocab, E)) != MESH_OK) return rc;
        if (s.out_norm == NORM_LAYER) {
            if ((rc = ld.layer_norm("final.norm", E, s.logit_scale, hm.final_norm)) != MESH_OK) return rc;
        } else {
            std::vector<float> g;
            if ((rc = ld.floats("final.norm", {}, g)) || (rc = ld.upload(g, &hm.final_gain))) return rc;
        }
        if (!linear_step_supported(hm.head)) hm.step_ok = false;
        st->output.data = const_cast<uint16_t *>(hm.head.w); st->output.K = E; st->output.M = s.vocab;
    }
    if (begins) {
        if (ends && s.tied_head) {
            hm.embed = const_cast<uint16_t *>(hm.head.w);
            hm.embed_ld = hm.head.Kp;
        } else {
            if ((rc = ld.raw("embed", {(uint64_t)s.vocab, (uint64_t)E}, &hm.embed)) != MESH_OK) return rc;
            hm.embed_ld = E;
        }
        if (s.sinusoid) {
            std::vector<float> fr((size_t)(E + 1) / 2);
            for (size_t i = 0; i < fr.size(); ++i) fr[i] = (float)pow(10000.0, -2.0 * (double)i / E);
            if ((rc = ld.upload(fr, &hm.freq)) != MESH_OK) return rc;
        }
        st->tok_embd.data = hm.embed; st->tok_embd.K = E; st->tok_embd.M = s.vocab;
    }
    MESH_HIP_TRY(hipDeviceSynchronize());
    return MESH_OK;
}

}  // namespace mesh
