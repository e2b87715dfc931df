// See hybrid.hpp.
#include "hybrid.hpp"

#include <algorithm>
#include <cmath>
#include <cstring>

#include "attn.hpp"
#include "registry.hpp"
#include "safetensors.hpp"
#include "stage.hpp"

namespace mesh {

// ------------------------------------------------------------------------------------------------ loading
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
    // output norm (one number) times the layer scale
    int gain(const std::string &norm, const std::string &scale, int n, float **out) {
        std::vector<float> g, s;
        int rc;
        if ((rc = floats(norm, {}, g)) || (rc = floats(scale, {(uint64_t)n}, s))) return rc;
        for (float &v : s) v *= g[0];
        return upload(s, out);
    }
    int head_norm(const std::string &name, int heads, int dim, int pad, float **out) {
        std::vector<float> g, p((size_t)heads * pad, 0.f);
        int rc = floats(name, {(uint64_t)heads * dim}, g);
        if (rc != MESH_OK) return rc;
        for (int h = 0; h < heads; ++h)
            for (int i = 0; i < dim; ++i) p[(size_t)h * pad + i] = g[(size_t)h * dim + i];
        return upload(p, out);
    }
    int layer(HybridLayer &L, const ModelSpec &s, int index) {
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
        } else {
            const int W = m.width;
            std::vector<float> bz, bx;
            if ((rc = matrix_alloc(L.in, 3 * W, E)) || (rc = place(L.in, mx + "z", W, E, 0, W, W, E, E)) || (rc = place(L.in, mx + "x", W, E, W, W, W, E, E)) ||
                (rc = place(L.in, mx + "g", W, E, 2 * W, W, W, E, E)) || (rc = floats(mx + "z.b", {(uint64_t)W}, bz)) || (rc = floats(mx + "x.b", {(uint64_t)W}, bx)) ||
                (rc = upload(bz, &L.bias_z)) || (rc = upload(bx, &L.bias_x)) || (rc = matrix(L.out, mx + "o", E, W)))
                return rc;
        }
        if ((rc = gain(p + "norm1", p + "ls1", E, &L.gain1)) != MESH_OK) return rc;
        if (L.spec.ff) {
            std::vector<float> c;
            if ((rc = matrix(L.up, p + "mlp.up", L.spec.ff, E)) || (rc = matrix(L.down, p + "mlp.down", E, L.spec.ff)) || (rc = floats(p + "mlp.act", {4}, c)) ||
                (rc = upload(c, &L.coef)) || (rc = gain(p + "norm2", p + "ls2", E, &L.gain2)))
                return rc;
        }
        std::vector<float> g;
        if ((rc = matrix(L.side_gate, p + "side.gate", s.side_dim, E)) || (rc = matrix(L.side_proj, p + "side.proj", E, s.side_dim)) ||
            (rc = floats(p + "side.norm", {(uint64_t)E}, g)) || (rc = upload(g, &L.gain_side)))
            return rc;
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
        if ((rc = ld.layer(L, s, i)) != MESH_OK) return rc;
        hm.in_max = std::max({hm.in_max, L.in.M, L.up.M, L.side_gate.M * LINEAR_SLICES_MAX});
        hm.act_max = std::max({hm.act_max, L.out.Kp, L.down.Kp, L.side_proj.Kp});
        if (L.spec.mixer.kind == MIXER_ATTENTION) hm.q_max = std::max(hm.q_max, L.spec.mixer.heads * L.head_pad);
        else { hm.has_state = true; hm.state_max = std::max(hm.state_max, L.spec.mixer.width); }
        for (const LinearWeight *w : {&L.in, &L.out, &L.up, &L.down, &L.side_gate, &L.side_proj})
            if (w->present() && !linear_step_supported(*w)) hm.step_ok = false;
    }
    if ((rc = ld.raw("side.embed", {(uint64_t)s.vocab, (uint64_t)n_layer * s.side_dim}, &hm.side)) != MESH_OK) return rc;
    if (layer_begin == 0) {
        if ((rc = ld.raw("embed", {(uint64_t)s.vocab, (uint64_t)E}, &hm.embed)) != MESH_OK) return rc;
        std::vector<float> fr((size_t)(E + 1) / 2);
        for (size_t i = 0; i < fr.size(); ++i) fr[i] = (float)pow(10000.0, -2.0 * (double)i / E);
        if ((rc = ld.upload(fr, &hm.freq)) != MESH_OK) return rc;
        st->tok_embd.data = hm.embed; st->tok_embd.K = E; st->tok_embd.M = s.vocab;
    }
    if (layer_end == n_layer) {
        std::vector<float> g;
        if ((rc = ld.floats("final.norm", {}, g)) || (rc = ld.upload(g, &hm.final_gain)) || (rc = ld.matrix(hm.head, "head", s.vocab, E))) return rc;
        if (!linear_step_supported(hm.head)) hm.step_ok = false;
        st->output.data = const_cast<uint16_t *>(hm.head.w); st->output.K = E; st->output.M = s.vocab;
    }
    MESH_HIP_TRY(hipDeviceSynchronize());
    return MESH_OK;
}

// ------------------------------------------------------------------------------------------------ session
int hybrid_session_alloc(mesh_session *s) {
    mesh_stage *st = s->stage;
    const HybridModel &hm = *st->hybrid;
    s->hybrid.reset(new HybridSession());
    HybridSession &h = *s->hybrid;
    const size_t B = (size_t)st->n_batch_max, E = (size_t)hm.spec.width, ab = act_bytes(hm.act);
    int rc = MESH_OK;
    // every buffer starts as zeros: what no kernel has written yet is read in places and discarded there, and has to be finite
    auto buf = [&](size_t bytes) -> void * {
        void *p = nullptr;
        if (rc == MESH_OK) rc = sess_alloc(s, &p, bytes);
        if (rc == MESH_OK && hipMemsetAsync(p, 0, bytes ? bytes : 16, s->stream) != hipSuccess) rc = fail(MESH_ERR_DEVICE, "hipMemsetAsync failed");
        return p;
    };
    auto fbuf = [&](size_t n) { return static_cast<float *>(buf(n * sizeof(float))); };
    s->x = fbuf(B * E);
    h.x2 = fbuf(E);
    h.xa = buf(B * (size_t)hm.width_pad * ab);
    h.acta = buf(B * (size_t)hm.act_max * std::max(ab, sizeof(float)));        // (the single-token step keeps f32 vectors in it)
    h.big = fbuf(B * (size_t)hm.in_max);
    h.y = fbuf(B * E);
    h.q = fbuf(B * (size_t)hm.q_max);
    h.part = fbuf(2 * 3 * STEP_PARTS_MAX);
    h.ws = fbuf(hm.state_max ? min_gru_workspace((int)B, hm.state_max) : 0);
    s->attn_part_rows = std::max<size_t>(B, 512);
    if (hm.q_max) {
        int heads = 0;
        for (const HybridLayer &L : hm.layers) heads = std::max(heads, L.spec.mixer.heads);
        s->attn_part = fbuf(s->attn_part_rows * (size_t)hm.q_max);
        s->attn_ml = fbuf(s->attn_part_rows * (size_t)heads * 2);
    }
    void *sat = buf(256);
    s->f16_sat = static_cast<unsigned *>(sat);
    for (const HybridLayer &L : hm.layers) {
        const MixerSpec &m = L.spec.mixer;
        uint8_t *k = nullptr, *v = nullptr;
        float *state = nullptr;
        if (m.kind == MIXER_ATTENTION) {
            const size_t bytes = (size_t)st->n_seq_max * m.kv_heads * (size_t)st->n_ctx * (size_t)kv_row_bytes(st->k_type, L.head_pad);
            k = static_cast<uint8_t *>(buf(bytes));
            v = static_cast<uint8_t *>(buf(bytes));
        } else {
            state = fbuf((size_t)st->n_seq_max * m.width);
        }
        h.k.push_back(k); h.v.push_back(v); h.state.push_back(state);
    }
    h.seq_len.assign((size_t)st->n_seq_max, 0);
    return rc;
}

int hybrid_check_batch(const mesh_session *s, const mesh_batch *b) {
    const HybridModel &hm = *s->stage->hybrid;
    const HybridSession &h = *s->hybrid;
    std::vector<char> seen(h.seq_len.size(), 0);
    for (int i = 0; i < b->n_tokens; ++i) {
        const int q = b->seq_id ? b->seq_id[i] : 0;
        const bool follows = i > 0 && (b->seq_id ? b->seq_id[i - 1] : 0) == q;
        if (follows) {
            if (b->pos[i] != b->pos[i - 1] + 1)
                return fail(MESH_ERR_INVALID, "mesh_stage_decode: token %d of sequence %d is at position %d, its neighbour before it at %d (one by one expected)", i, q, b->pos[i], b->pos[i - 1]);
            continue;
        }
        if (seen[(size_t)q]) return fail(MESH_ERR_INVALID, "mesh_stage_decode: the tokens of sequence %d are not neighbours in the call", q);
        seen[(size_t)q] = 1;
        if (hm.has_state && b->pos[i] != 0 && b->pos[i] != h.seq_len[(size_t)q])
            return fail(MESH_ERR_INVALID, "mesh_stage_decode: sequence %d stands at %d tokens, but the call goes on at position %d (0 starts it anew)", q, h.seq_len[(size_t)q], b->pos[i]);
    }
    return MESH_OK;
}

void hybrid_note_batch(mesh_session *s, const mesh_batch *b, bool ok) {
    for (int i = 0; i < b->n_tokens; ++i) s->hybrid->seq_len[(size_t)(b->seq_id ? b->seq_id[i] : 0)] = ok ? b->pos[i] + 1 : -1;
}

// ------------------------------------------------------------------------------------------------ layers
bool hybrid_single_step(const mesh_session *s, int T) { return T == 1 && s->tune.step_fused && s->stage->hybrid->step_ok; }

static int keys_seen(const MixerSpec &m, int max_keys) { return m.window > 0 ? std::min(m.window, max_keys) : max_keys; }

static int layer_splits(const mesh_session *s, const MixerSpec &m, int T, int max_keys) {
    return T < 64 ? attn_splits_for(s->tune, T, m.kv_heads, keys_seen(m, max_keys), false) : 1;
}

uint64_t hybrid_graph_key(const mesh_session *s, int T, int max_keys) {
    uint64_t key = 1469598103934665603ull ^ (uint64_t)T;
    for (const HybridLayer &L : s->stage->hybrid->layers)
        if (L.spec.mixer.kind == MIXER_ATTENTION) key = (key ^ (uint64_t)layer_splits(s, L.spec.mixer, T, max_keys)) * 1099511628211ull;
    return key;
}

int hybrid_embed(mesh_session *s, int T) {
    const HybridModel &hm = *s->stage->hybrid;
    ProfScope ps(s, MESH_PROF_CODEC);
    return embed_rows(hm.embed, s->d_tok, s->d_pos, hm.freq, hm.spec.embed_scale, T, hm.spec.width, s->x, s->stream);
}

// q, k of the call in h.big -> attention output in h.acta: f32 rows for the single-token step, else the product's activations
static int run_attention(mesh_session *s, size_t il, int T, int max_keys, bool f32_out) {
    mesh_stage *st = s->stage;
    const HybridModel &hm = *st->hybrid;
    HybridSession &h = *s->hybrid;
    const HybridLayer &L = hm.layers[il];
    const MixerSpec &m = L.spec.mixer;
    int rc;
    {
        QkAppendArgs a;
        a.qk = h.big; a.q = h.q; a.kcache = h.k[il]; a.vcache = h.v[il]; a.kv_type = st->k_type;
        a.q_norm = L.q_norm; a.k_norm = L.k_norm; a.pos = s->d_pos; a.seq = s->d_seq; a.sat = s->f16_sat;
        a.eps = hm.spec.eps; a.n_head = m.heads; a.n_kv = m.kv_heads; a.dim = m.dim; a.hd = L.head_pad; a.n_ctx = st->n_ctx;
        ProfScope ps(s, MESH_PROF_ROPE);
        if ((rc = qk_norm_append(a, T, s->stream)) != MESH_OK) return rc;
    }
    AttnArgs aa;
    aa.q = h.q; aa.kcache = h.k[il]; aa.vcache = h.v[il]; aa.k_type = st->k_type; aa.v_type = st->v_type; aa.pos = s->d_pos; aa.seq = s->d_seq;
    aa.part = s->attn_part; aa.ml = s->attn_ml;
    if (f32_out || hm.act == ACT_F32) aa.out = static_cast<float *>(h.acta);
    else aa.out_bf16 = static_cast<uint16_t *>(h.acta);
    aa.window = m.window;
    aa.scale = m.scale;
    aa.n_head = m.heads; aa.n_kv = m.kv_heads; aa.group = m.heads / m.kv_heads; aa.head_dim = L.head_pad; aa.n_ctx = st->n_ctx;
    aa.n_splits = layer_splits(s, m, T, max_keys);
    ProfScope ps(s, MESH_PROF_ATTN);
    if (hm.act == ACT_F32) return attention(aa, T, s->stream);
    if (T >= s->tune.gemm_min_tokens && s->chunk_pos0 >= 0 && L.head_pad <= 128) {
        aa.part_rows = s->tune.attn_chunk_ksplit ? s->attn_part_rows : 0;
        return attention_chunk(aa, T, s->chunk_pos0, s->chunk_seq, s->stream);
    }
    if (T >= s->tune.attn_mma_min_tokens && attention_mma_supported(aa)) return attention_mma(aa, T, s->stream);
    return attention(aa, T, s->stream);
}

// One token: every product derives its input from what the launch before it left (linear.hpp).
static int run_step(mesh_session *s, int max_keys) {
    mesh_stage *st = s->stage;
    const HybridModel &hm = *st->hybrid;
    HybridSession &h = *s->hybrid;
    hipStream_t stream = s->stream;
    float *inner = static_cast<float *>(h.acta);       // a sublayer's vector: attention output, recurrence output, side vector
    HybridPending pend;
    pend.x = s->x;
    int set = 0, rc;
    auto base = [&](const LinearWeight &W, float *out, StepOut kind) {
        StepArgs a;
        a.W = W; a.eps = hm.spec.eps; a.out = out; a.out_kind = kind;
        a.pos = s->d_pos; a.seq = s->d_seq; a.tok = s->d_tok;
        return a;
    };
    // a product that reads the residual stream, completing it first
    auto from_stream = [&](StepArgs a) {
        a.in = pend.x;
        if (pend.y) {
            a.in_kind = STEP_IN_RESIDUAL;
            a.y = pend.y; a.gain = pend.gain; a.part = pend.part; a.n_part = pend.n_part;
            a.x_out = pend.x == s->x ? h.x2 : s->x;
        }
        ProfScope ps(s, MESH_PROF_GEMV);
        const int r = linear_step(a, stream);
        if (pend.y) pend.x = a.x_out;
        pend.y = nullptr;
        return r;
    };
    // a sublayer's last product: its result waits to be normed and added
    auto to_stream = [&](StepArgs a, const float *gain) {
        a.out = h.y; a.out_kind = STEP_OUT_SUMSQ;
        a.out_part = h.part + (size_t)set * 3 * STEP_PARTS_MAX;
        set ^= 1;
        pend.y = h.y; pend.gain = gain; pend.part = a.out_part; pend.n_part = linear_step_grid(a);
        ProfScope ps(s, MESH_PROF_GEMV);
        return linear_step(a, stream);
    };
    for (size_t il = 0; il < hm.layers.size(); ++il) {
        const HybridLayer &L = hm.layers[il];
        if (L.spec.mixer.kind == MIXER_ATTENTION) {
            if ((rc = from_stream(base(L.in, h.big, STEP_OUT_PLAIN))) != MESH_OK) return rc;
            if ((rc = run_attention(s, il, 1, max_keys, true)) != MESH_OK) return rc;
        } else {
            StepArgs a = base(L.in, inner, STEP_OUT_MIN_GRU);
            a.width = L.spec.mixer.width; a.bias_z = L.bias_z; a.bias_x = L.bias_x; a.state = h.state[il];
            if ((rc = from_stream(a)) != MESH_OK) return rc;
        }
        StepArgs o = base(L.out, nullptr, STEP_OUT_SUMSQ);
        o.in = inner;
        if ((rc = to_stream(o, L.gain1)) != MESH_OK) return rc;
        if (L.spec.ff) {
            StepArgs u = base(L.up, h.big, STEP_OUT_POWERS);
            u.out_part = h.part + (size_t)set * 3 * STEP_PARTS_MAX;
            const float *powers = u.out_part;
            const int n_powers = linear_step_grid(u);
            set ^= 1;
            if ((rc = from_stream(u)) != MESH_OK) return rc;
            StepArgs d = base(L.down, nullptr, STEP_OUT_SUMSQ);
            d.in_kind = STEP_IN_POLY; d.in = h.big; d.part = powers; d.n_part = n_powers; d.coef = L.coef;
            if ((rc = to_stream(d, L.gain2)) != MESH_OK) return rc;
        }
        StepArgs g = base(L.side_gate, inner, STEP_OUT_SIDE);
        g.side = hm.side; g.side_stride = (int)hm.spec.layers.size() * hm.spec.side_dim; g.side_offset = (st->layer_begin + (int)il) * hm.spec.side_dim;
        if ((rc = from_stream(g)) != MESH_OK) return rc;
        StepArgs p = base(L.side_proj, nullptr, STEP_OUT_SUMSQ);
        p.in = inner;
        if ((rc = to_stream(p, L.gain_side)) != MESH_OK) return rc;
    }
    h.tail = pend;
    return MESH_OK;
}

int hybrid_run_layers(mesh_session *s, int T, int max_keys) {
    mesh_stage *st = s->stage;
    const HybridModel &hm = *st->hybrid;
    HybridSession &h = *s->hybrid;
    if (hybrid_single_step(s, T)) return run_step(s, max_keys);
    hipStream_t stream = s->stream;
    const int E = hm.spec.width;
    const float eps = hm.spec.eps;
    const ActType act = hm.act;
    int rc;
    auto product = [&](const LinearWeight &W, const void *x, float *y, int ldy) {
        ProfScope ps(s, MESH_PROF_GEMV);
        return linear(W, x, act, T, y, ldy, s->tune.linear_tile_min_tokens, stream);
    };
    auto add = [&](const float *gain) {
        ProfScope ps(s, MESH_PROF_PREP);
        return residual_norm_rows(s->x, h.y, gain, eps, T, E, h.xa, act, hm.width_pad, stream);
    };
    {
        ProfScope ps(s, MESH_PROF_PREP);
        if ((rc = residual_norm_rows(s->x, nullptr, nullptr, eps, T, E, h.xa, act, hm.width_pad, stream)) != MESH_OK) return rc;
    }
    for (size_t il = 0; il < hm.layers.size(); ++il) {
        const HybridLayer &L = hm.layers[il];
        const MixerSpec &m = L.spec.mixer;
        if ((rc = product(L.in, h.xa, h.big, L.in.M)) != MESH_OK) return rc;
        if (m.kind == MIXER_ATTENTION) {
            if ((rc = run_attention(s, il, T, max_keys, false)) != MESH_OK) return rc;
        } else {
            MinGruArgs a;
            a.zxg = h.big; a.bias_z = L.bias_z; a.bias_x = L.bias_x; a.state = h.state[il]; a.pos = s->d_pos; a.seq = s->d_seq; a.ws = h.ws;
            a.out = h.acta; a.act = act; a.ld = L.out.Kp; a.width = m.width;
            ProfScope ps(s, MESH_PROF_PREP);
            if ((rc = min_gru(a, T, stream)) != MESH_OK) return rc;
        }
        if ((rc = product(L.out, h.acta, h.y, E)) != MESH_OK || (rc = add(L.gain1)) != MESH_OK) return rc;
        if (L.spec.ff) {
            if ((rc = product(L.up, h.xa, h.big, L.spec.ff)) != MESH_OK) return rc;
            {
                ProfScope ps(s, MESH_PROF_PREP);
                if ((rc = poly_norm_rows(h.big, L.coef, eps, T, L.spec.ff, h.acta, act, L.down.Kp, stream)) != MESH_OK) return rc;
            }
            if ((rc = product(L.down, h.acta, h.y, E)) != MESH_OK || (rc = add(L.gain2)) != MESH_OK) return rc;
        }
        int slices;
        const size_t slice = (size_t)T * hm.spec.side_dim;
        {
            ProfScope ps(s, MESH_PROF_GEMV);
            if ((slices = linear_sliced(L.side_gate, h.xa, act, T, h.big, slice, s->tune.linear_tile_min_tokens, stream)) < 0) return slices;
        }
        {
            ProfScope ps(s, MESH_PROF_PREP);
            if ((rc = side_gate_rows(h.big, slices, slice, hm.side, s->d_tok, (int)hm.spec.layers.size() * hm.spec.side_dim, (st->layer_begin + (int)il) * hm.spec.side_dim, T,
                                     hm.spec.side_dim, h.acta, act, L.side_proj.Kp, stream)) != MESH_OK)
                return rc;
        }
        if ((rc = product(L.side_proj, h.acta, h.y, E)) != MESH_OK || (rc = add(L.gain_side)) != MESH_OK) return rc;
    }
    return MESH_OK;
}

int hybrid_finish(mesh_session *s, int T, float **x) {
    const HybridModel &hm = *s->stage->hybrid;
    HybridSession &h = *s->hybrid;
    *x = s->x;
    if (!hybrid_single_step(s, T)) return MESH_OK;
    *x = h.tail.x;
    ProfScope ps(s, MESH_PROF_PREP);
    return residual_norm_rows(h.tail.x, h.tail.y, h.tail.gain, hm.spec.eps, 1, hm.spec.width, h.xa, hm.act, hm.width_pad, s->stream);
}

int hybrid_logits(mesh_session *s, int T, const int32_t *d_rows, int n_rows, float *d_out) {
    const HybridModel &hm = *s->stage->hybrid;
    HybridSession &h = *s->hybrid;
    int rc;
    if (hybrid_single_step(s, T)) {
        StepArgs a;
        a.W = hm.head; a.in_kind = STEP_IN_RESIDUAL_NORM; a.out_kind = STEP_OUT_PLAIN;
        a.in = h.tail.x; a.y = h.tail.y; a.gain = h.tail.gain; a.part = h.tail.part; a.n_part = h.tail.n_part;
        a.x_out = h.tail.x == s->x ? h.x2 : s->x;
        a.norm_gain = hm.final_gain; a.eps = hm.spec.eps; a.out = d_out;
        ProfScope ps(s, MESH_PROF_GEMV);
        return linear_step(a, s->stream);
    }
    {
        ProfScope ps(s, MESH_PROF_PREP);
        if ((rc = scalar_norm_rows(s->x, d_rows, hm.final_gain, hm.spec.eps, n_rows, hm.spec.width, h.xa, hm.act, hm.width_pad, s->stream)) != MESH_OK) return rc;
    }
    ProfScope ps(s, MESH_PROF_GEMV);
    return linear(hm.head, h.xa, hm.act, n_rows, d_out, hm.head.M, s->tune.linear_tile_min_tokens, s->stream);
}

}  // namespace mesh
