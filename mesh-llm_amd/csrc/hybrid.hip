// See hybrid.hpp.
#include "hybrid.hpp"

#include <algorithm>

#include "attn.hpp"
#include "stage.hpp"

namespace mesh {

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
    s->attn_part_rows = std::max<size_t>(B, 256 * LATENT_GROUP);
    if (hm.part_max) {
        int heads = 0;
        for (const HybridLayer &L : hm.layers) heads = std::max(heads, L.spec.mixer.heads);
        s->attn_part = fbuf(s->attn_part_rows * hm.part_max);
        s->attn_ml = fbuf(s->attn_part_rows * (size_t)heads * 2);
    }
    h.qx = buf(B * hm.qx_max);
    h.kvx = fbuf(B * hm.kvx_max);
    h.kv16 = static_cast<uint16_t *>(buf((size_t)st->n_ctx * hm.kv16_max * 2));
    h.chunk_cap = (int)B / STATE_CHUNK + std::min((int)B, st->n_seq_max) + 1;        // (a sequence's tokens leave one chunk that is not whole)
    h.gated_ws = fbuf((size_t)(hm.has_chunks ? h.chunk_cap : 0) * hm.gated_ws_max);
    void *sat = buf(256);
    s->f16_sat = static_cast<unsigned *>(sat);
    for (const HybridLayer &L : hm.layers) {
        const MixerSpec &m = L.spec.mixer;
        uint8_t *k = nullptr, *v = nullptr;
        float *state = nullptr, *tail = nullptr;
        if (m.kind == MIXER_ATTENTION) {
            const size_t bytes = (size_t)st->n_seq_max * m.kv_heads * (size_t)st->n_ctx * (size_t)kv_row_bytes(st->k_type, L.head_pad);
            k = static_cast<uint8_t *>(buf(bytes));
            v = static_cast<uint8_t *>(buf(bytes));
        } else if (m.kind == MIXER_LATENT) {
            if (m.kv_from < 0) k = static_cast<uint8_t *>(buf((size_t)st->n_seq_max * (size_t)st->n_ctx * L.latent.row() * (hm.act == ACT_F32 ? 4 : 2)));
        } else if (m.has_matrix_state()) {
            state = fbuf((size_t)st->n_seq_max * m.heads * m.dim * m.vdim);
            if (L.gated.delta) tail = fbuf((size_t)st->n_seq_max * m.taps * gated_state_channels(L.gated));
        } else {
            state = fbuf((size_t)st->n_seq_max * m.width);
        }
        h.k.push_back(k); h.v.push_back(v); h.state.push_back(state); h.tail.push_back(tail);
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

bool hybrid_needs_ids(const mesh_stage *st) { return st->hybrid->side(); }

size_t hybrid_chunk_table(mesh_session *s, const mesh_batch *b, int32_t *table, const int32_t *d_table) {
    HybridSession &h = *s->hybrid;
    if (!s->stage->hybrid->has_chunks) return 0;
    const size_t B = (size_t)s->stage->n_batch_max;
    int32_t *chunk = table, *first = chunk + B + 1, *run = first + B;
    int nc = 0, nr = 0, start = 0;
    for (int i = 0; i < b->n_tokens; ++i) {
        const bool opens = i == 0 || (b->seq_id && b->seq_id[i] != b->seq_id[i - 1]);
        if (opens) { start = i; run[nr++] = nc; }
        if (opens || (i - start) % STATE_CHUNK == 0) { chunk[nc] = i; first[nc++] = start; }
    }
    chunk[nc] = b->n_tokens;
    run[nr] = nc;
    h.chunks.chunk = d_table; h.chunks.first = d_table + B + 1; h.chunks.run = h.chunks.first + B;
    h.chunks.n_chunks = nc; h.chunks.n_runs = nr;
    return nr == b->n_tokens ? 0 : 2 * B + 1 + (size_t)nr + 1;
}

// ------------------------------------------------------------------------------------------------ layers
bool hybrid_single_step(const mesh_session *s, int T) { return T == 1 && s->tune.step_fused && s->stage->hybrid->step_ok; }

static int keys_seen(const MixerSpec &m, int max_keys) { return m.window > 0 ? std::min(m.window, max_keys) : max_keys; }

static int layer_splits(const mesh_session *s, const MixerSpec &m, int T, int max_keys) {
    return T < 64 ? attn_splits_for(s->tune, T, m.kv_heads, keys_seen(m, max_keys), false) : 1;
}

// (the partial sums have room for 1024 (token, split) rows at least)
static int latent_layer_splits(const mesh_session *s, const LatentShape &ls, int T, int max_keys) {
    return latent_splits(ls, T, latent_group(ls, T, s->chunk_pos0 >= 0), max_keys, std::min(s->tune.attn_split_target, 256));
}

uint64_t hybrid_graph_key(const mesh_session *s, int T, int max_keys) {
    uint64_t key = 1469598103934665603ull ^ (uint64_t)T;
    auto mix = [&](uint64_t v) { key = (key ^ v) * 1099511628211ull; };
    for (const HybridLayer &L : s->stage->hybrid->layers) {
        if (L.spec.mixer.kind == MIXER_ATTENTION) mix((uint64_t)layer_splits(s, L.spec.mixer, T, max_keys));
        if (L.spec.mixer.kind == MIXER_LATENT) mix((uint64_t)latent_layer_splits(s, L.latent, T, max_keys) << 1 | (s->chunk_pos0 >= 0 ? 1 : 0));
    }
    if (s->stage->hybrid->has_chunks) mix(((uint64_t)s->hybrid->chunks.n_chunks << 32) | (uint64_t)s->hybrid->chunks.n_runs);
    return key;
}

int hybrid_embed(mesh_session *s, int T) {
    const HybridModel &hm = *s->stage->hybrid;
    ProfScope ps(s, MESH_PROF_CODEC);
    return embed_rows(hm.embed, hm.embed_ld, s->d_tok, s->d_pos, hm.freq, hm.spec.embed_scale, T, hm.spec.width, s->x, s->stream);
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

// What the layer's recurrence needs beside its weights.
static GatedStateArgs gated_args(mesh_session *s, size_t il, void *out, ActType act) {
    HybridSession &h = *s->hybrid;
    GatedStateArgs a = s->stage->hybrid->layers[il].gated;
    a.in = h.big; a.state = h.state[il]; a.tail = h.tail[il]; a.pos = s->d_pos; a.seq = s->d_seq;
    a.chunks = h.chunks; a.ws = h.gated_ws; a.o = h.q; a.out = out; a.act = act;
    return a;
}

static LatentCache latent_cache(mesh_session *s, size_t il) {
    const HybridModel &hm = *s->stage->hybrid;
    HybridSession &h = *s->hybrid;
    const HybridLayer &L = hm.layers[il];
    LatentCache c;
    c.rows = h.k[(size_t)L.cache_layer]; c.n_ctx = s->stage->n_ctx;
    if (L.own_cache((int)il)) { c.in = h.big + L.spec.mixer.q_rank; c.ld = L.in.M; c.gain = L.c_norm; }
    c.rot = L.rot; c.pos = s->d_pos; c.seq = s->d_seq; c.sat = s->f16_sat; c.eps = hm.spec.eps;
    return c;
}

// queries in h.q, this call's rows in the cache unless `append` -> attention output in h.acta (f32 rows for the single-token
// step, else the product's activations)
static int run_latent_rows(mesh_session *s, size_t il, int T, int max_keys, bool append, bool f32_out) {
    mesh_stage *st = s->stage;
    const HybridModel &hm = *st->hybrid;
    HybridSession &h = *s->hybrid;
    const HybridLayer &L = hm.layers[il];
    const MixerSpec &m = L.spec.mixer;
    const LatentCache c = latent_cache(s, il);
    int rc;
    {
        ProfScope ps(s, MESH_PROF_ROPE);
        if ((rc = latent_query(L.latent, c, hm.act, h.q, L.w_uk_t, m.scale, append && c.in, h.qx, T, s->stream)) != MESH_OK) return rc;
    }
    LatentAttnArgs a;
    a.qa = h.qx; a.rows = c.rows; a.pos = s->d_pos; a.seq = s->d_seq; a.part = s->attn_part; a.ml = s->attn_ml; a.n_ctx = st->n_ctx;
    a.group = latent_group(L.latent, T, s->chunk_pos0 >= 0);
    a.n_splits = latent_layer_splits(s, L.latent, T, max_keys);
    a.w_uv = L.w_uv; a.gate = h.big + L.in.M - m.heads; a.gate_ld = L.in.M;
    if (f32_out || hm.act == ACT_F32) a.out = static_cast<float *>(h.acta);
    else a.out_bf16 = static_cast<uint16_t *>(h.acta);
    ProfScope ps(s, MESH_PROF_ATTN);
    if ((rc = latent_attention(L.latent, a, hm.act, T, s->stream)) != MESH_OK) return rc;
    return latent_out(L.latent, a, T, s->stream);
}

// the same for a long chunk of one sequence: keys and values of all its positions are projected, then attended to
static int run_latent_chunk(mesh_session *s, size_t il, int T) {
    mesh_stage *st = s->stage;
    const HybridModel &hm = *st->hybrid;
    HybridSession &h = *s->hybrid;
    const HybridLayer &L = hm.layers[il];
    const LatentShape &ls = L.latent;
    const void *rows = h.k[(size_t)L.cache_layer];
    uint16_t *k16 = h.kv16, *v16 = k16 + (size_t)ls.heads * st->n_ctx * ls.chunk_k;
    int rc;
    {
        ProfScope ps(s, MESH_PROF_ROPE);
        if ((rc = latent_chunk_query(ls, L.rot, h.q, s->d_pos, static_cast<float *>(h.qx), T, s->stream)) != MESH_OK) return rc;
    }
    const int n_keys = s->chunk_pos0 + T;
    for (int k0 = 0; k0 < n_keys; k0 += st->n_batch_max) {
        const int n = std::min(st->n_batch_max, n_keys - k0);
        {
            ProfScope ps(s, MESH_PROF_PREP);
            if ((rc = latent_chunk_rows(ls, rows, st->n_ctx, s->chunk_seq, k0, n, static_cast<uint16_t *>(h.acta), L.ukv.Kp, s->stream)) != MESH_OK) return rc;
        }
        {
            ProfScope ps(s, MESH_PROF_GEMV);
            if ((rc = linear(L.ukv, h.acta, ACT_BF16, n, h.kvx, L.ukv.M, s->tune.linear_tile_min_tokens, s->stream)) != MESH_OK) return rc;
        }
        ProfScope ps(s, MESH_PROF_PREP);
        if ((rc = latent_chunk_pack(ls, rows, st->n_ctx, s->chunk_seq, k0, n, h.kvx, k16, v16, s->f16_sat, s->stream)) != MESH_OK) return rc;
    }
    AttnArgs a;
    a.q = static_cast<const float *>(h.qx); a.kcache = reinterpret_cast<const uint8_t *>(k16); a.vcache = reinterpret_cast<const uint8_t *>(v16);
    a.part = s->attn_part; a.ml = s->attn_ml; a.part_rows = s->tune.attn_chunk_ksplit ? s->attn_part_rows : 0;
    a.out_bf16 = static_cast<uint16_t *>(h.acta);
    a.scale = L.spec.mixer.scale;
    a.n_head = a.n_kv = ls.heads; a.head_dim = ls.chunk_k; a.v_dim = ls.chunk_v; a.n_ctx = st->n_ctx;
    a.head_gate = h.big + L.in.M - ls.heads; a.gate_ld = L.in.M;
    ProfScope ps(s, MESH_PROF_ATTN);
    return attention_chunk(a, T, s->chunk_pos0, 0, s->stream);
}

static int run_latent(mesh_session *s, size_t il, int T, int max_keys) {
    const HybridModel &hm = *s->stage->hybrid;
    HybridSession &h = *s->hybrid;
    const HybridLayer &L = hm.layers[il];
    int rc;
    {
        ProfScope ps(s, MESH_PROF_PREP);
        if ((rc = latent_rows(L.latent, latent_cache(s, il), hm.act, h.big, L.in.M, L.cq_norm, L.spec.mixer.q_rank, h.acta, L.uq.Kp, T, s->stream)) != MESH_OK) return rc;
    }
    {
        ProfScope ps(s, MESH_PROF_GEMV);
        if ((rc = linear(L.uq, h.acta, hm.act, T, h.q, L.uq.M, s->tune.linear_tile_min_tokens, s->stream)) != MESH_OK) return rc;
    }
    if (L.ukv.present() && s->chunk_pos0 >= 0 && T >= s->tune.latent_chunk_min_tokens) return run_latent_chunk(s, il, T);
    return run_latent_rows(s, il, T, max_keys, false, false);
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
    const bool ln = hm.spec.out_norm == NORM_LAYER;
    auto base = [&](const LinearWeight &W, float *out, StepOut kind) {
        StepArgs a;
        a.W = W; a.eps = hm.spec.eps; a.out = out; a.out_kind = kind;
        a.pos = s->d_pos; a.seq = s->d_seq; a.tok = s->d_tok;
        return a;
    };
    auto run = [&](const StepArgs &a) {
        ProfScope ps(s, MESH_PROF_GEMV);
        return linear_step(a, stream);
    };
    // a product that reads the residual stream, completing it first
    auto from_stream = [&](StepArgs a, const RowNorm &pre) {
        a.in = pend.x;
        if (pre.kind == NORM_LAYER) { a.in_kind = STEP_IN_LAYER; a.norm_gain = pre.gain; a.norm_bias = pre.bias; }
        if (pend.y) {
            if (!ln) a.in_kind = STEP_IN_RESIDUAL;
            a.y = pend.y; a.gain = pend.post.gain; a.bias = pend.post.bias; a.part = pend.part; a.n_part = pend.n_part;
            a.x_out = pend.x == s->x ? h.x2 : s->x;
        }
        const int r = run(a);
        if (pend.y) pend.x = a.x_out;
        pend.y = nullptr;
        return r;
    };
    // a sublayer's last product: its result waits to be normed and added
    auto to_stream = [&](StepArgs a, const RowNorm &post) {
        a.out = h.y;
        pend.y = h.y; pend.post = post;
        if (!ln) {
            a.out_kind = STEP_OUT_SUMSQ;
            a.out_part = h.part + (size_t)set * 3 * STEP_PARTS_MAX;
            set ^= 1;
            pend.part = a.out_part; pend.n_part = linear_step_grid(a);
        }
        return run(a);
    };
    for (size_t il = 0; il < hm.layers.size(); ++il) {
        const HybridLayer &L = hm.layers[il];
        const MixerSpec &m = L.spec.mixer;
        if (m.kind == MIXER_MIN_GRU) {
            StepArgs a = base(L.in, inner, STEP_OUT_MIN_GRU);
            a.width = m.width; a.bias_z = L.bias_z; a.bias_x = L.bias_x; a.state = h.state[il];
            if ((rc = from_stream(a, L.pre1)) != MESH_OK) return rc;
        } else {
            if ((rc = from_stream(base(L.in, h.big, STEP_OUT_PLAIN), L.pre1)) != MESH_OK) return rc;
            if (m.kind == MIXER_ATTENTION) {
                if ((rc = run_attention(s, il, 1, max_keys, true)) != MESH_OK) return rc;
            } else if (m.kind == MIXER_LATENT) {
                StepArgs q = base(L.uq, h.q, STEP_OUT_PLAIN);
                q.in_kind = STEP_IN_UNIT_RMS; q.in = h.big; q.gain = L.cq_norm;
                if ((rc = run(q)) != MESH_OK || (rc = run_latent_rows(s, il, 1, max_keys, true, true)) != MESH_OK) return rc;
            } else {
                ProfScope ps(s, MESH_PROF_PREP);
                if ((rc = gated_state_step(gated_args(s, il, inner, ACT_F32), 1, stream)) != MESH_OK) return rc;
            }
        }
        StepArgs o = base(L.out, nullptr, STEP_OUT_PLAIN);
        o.in = inner;
        if ((rc = to_stream(o, L.post1)) != MESH_OK) return rc;
        if (L.spec.ff) {
            StepArgs u = base(L.up, h.big, STEP_OUT_PLAIN), d = base(L.down, nullptr, STEP_OUT_PLAIN);
            d.in = h.big;
            if (hm.spec.ff == FF_POLY_NORM) {
                u.out_kind = STEP_OUT_POWERS;
                u.out_part = h.part + (size_t)set * 3 * STEP_PARTS_MAX;
                set ^= 1;
                d.in_kind = STEP_IN_POLY; d.part = u.out_part; d.n_part = linear_step_grid(u); d.coef = L.coef;
            } else {
                u.out = inner;
                d.in_kind = STEP_IN_RELU2; d.in = inner;
            }
            if ((rc = from_stream(u, L.pre2)) != MESH_OK || (rc = to_stream(d, L.post2)) != MESH_OK) return rc;
        }
        if (hm.side()) {
            StepArgs g = base(L.side_gate, inner, STEP_OUT_SIDE);
            g.side = hm.side_embed; g.side_stride = (int)hm.spec.layers.size() * hm.spec.side_dim; g.side_offset = (st->layer_begin + (int)il) * hm.spec.side_dim;
            if ((rc = from_stream(g, RowNorm{})) != MESH_OK) return rc;
            StepArgs p = base(L.side_proj, nullptr, STEP_OUT_PLAIN);
            p.in = inner;
            if ((rc = to_stream(p, L.post_side)) != MESH_OK) return rc;
        }
    }
    h.tail_step = pend;
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
    // the residual stream after a sublayer, and the next one's input
    auto add = [&](const float *y, const RowNorm &post, const RowNorm &pre) {
        ProfScope ps(s, MESH_PROF_PREP);
        return residual_norm_rows(s->x, y, post, pre, eps, T, E, h.xa, act, hm.width_pad, stream);
    };
    if ((rc = add(nullptr, RowNorm{}, hm.layers[0].pre1)) != MESH_OK) return rc;
    for (size_t il = 0; il < hm.layers.size(); ++il) {
        const HybridLayer &L = hm.layers[il];
        const MixerSpec &m = L.spec.mixer;
        const RowNorm after = hm.side() || il + 1 == hm.layers.size() ? RowNorm{} : hm.layers[il + 1].pre1;
        if ((rc = product(L.in, h.xa, h.big, L.in.M)) != MESH_OK) return rc;
        if (m.kind == MIXER_ATTENTION) {
            if ((rc = run_attention(s, il, T, max_keys, false)) != MESH_OK) return rc;
        } else if (m.kind == MIXER_LATENT) {
            if ((rc = run_latent(s, il, T, max_keys)) != MESH_OK) return rc;
        } else if (m.has_matrix_state()) {
            const GatedStateArgs a = gated_args(s, il, h.acta, act);
            ProfScope ps(s, MESH_PROF_PREP);
            if ((rc = h.chunks.n_runs == T ? gated_state_step(a, T, stream) : gated_state_chunks(a, T, stream)) != MESH_OK) return rc;
        } else {
            MinGruArgs a;
            a.zxg = h.big; a.bias_z = L.bias_z; a.bias_x = L.bias_x; a.state = h.state[il]; a.pos = s->d_pos; a.seq = s->d_seq; a.ws = h.ws;
            a.out = h.acta; a.act = act; a.ld = L.out.Kp; a.width = m.width;
            ProfScope ps(s, MESH_PROF_PREP);
            if ((rc = min_gru(a, T, stream)) != MESH_OK) return rc;
        }
        if ((rc = product(L.out, h.acta, h.y, E)) != MESH_OK || (rc = add(h.y, L.post1, L.spec.ff ? L.pre2 : after)) != MESH_OK) return rc;
        if (L.spec.ff) {
            if (hm.spec.ff == FF_POLY_NORM) {
                if ((rc = product(L.up, h.xa, h.big, L.spec.ff)) != MESH_OK) return rc;
                ProfScope ps(s, MESH_PROF_PREP);
                if ((rc = poly_norm_rows(h.big, L.coef, eps, T, L.spec.ff, h.acta, act, L.down.Kp, stream)) != MESH_OK) return rc;
            } else {
                ProfScope ps(s, MESH_PROF_GEMV);
                if ((rc = linear_relu2(L.up, h.xa, act, T, h.acta, L.down.Kp, s->tune.linear_tile_min_tokens, stream)) != MESH_OK) return rc;
            }
            if ((rc = product(L.down, h.acta, h.y, E)) != MESH_OK || (rc = add(h.y, L.post2, after)) != MESH_OK) return rc;
        }
        if (!hm.side()) continue;
        int slices;
        const size_t slice = (size_t)T * hm.spec.side_dim;
        {
            ProfScope ps(s, MESH_PROF_GEMV);
            if ((slices = linear_sliced(L.side_gate, h.xa, act, T, h.big, slice, s->tune.linear_tile_min_tokens, stream)) < 0) return slices;
        }
        {
            ProfScope ps(s, MESH_PROF_PREP);
            if ((rc = side_gate_rows(h.big, slices, slice, hm.side_embed, s->d_tok, (int)hm.spec.layers.size() * hm.spec.side_dim, (st->layer_begin + (int)il) * hm.spec.side_dim, T,
                                     hm.spec.side_dim, h.acta, act, L.side_proj.Kp, stream)) != MESH_OK)
                return rc;
        }
        if ((rc = product(L.side_proj, h.acta, h.y, E)) != MESH_OK || (rc = add(h.y, L.post_side, RowNorm{})) != MESH_OK) return rc;
    }
    return MESH_OK;
}

int hybrid_finish(mesh_session *s, int T, float **x) {
    const HybridModel &hm = *s->stage->hybrid;
    HybridSession &h = *s->hybrid;
    *x = s->x;
    if (!hybrid_single_step(s, T)) return MESH_OK;
    *x = h.tail_step.x;
    ProfScope ps(s, MESH_PROF_PREP);
    return residual_norm_rows(h.tail_step.x, h.tail_step.y, h.tail_step.post, RowNorm{}, hm.spec.eps, 1, hm.spec.width, h.xa, hm.act, hm.width_pad, s->stream);
}

int hybrid_logits(mesh_session *s, int T, const int32_t *d_rows, int n_rows, float *d_out) {
    const HybridModel &hm = *s->stage->hybrid;
    HybridSession &h = *s->hybrid;
    int rc;
    if (hybrid_single_step(s, T)) {
        StepArgs a;
        a.W = hm.head; a.in_kind = STEP_IN_RESIDUAL_NORM; a.out_kind = STEP_OUT_PLAIN;
        a.in = h.tail_step.x; a.y = h.tail_step.y; a.gain = h.tail_step.post.gain; a.bias = h.tail_step.post.bias; a.part = h.tail_step.part; a.n_part = h.tail_step.n_part;
        a.x_out = h.tail_step.x == s->x ? h.x2 : s->x;
        if (hm.final_norm.kind == NORM_LAYER) { a.in_kind = STEP_IN_LAYER; a.norm_gain = hm.final_norm.gain; a.norm_bias = hm.final_norm.bias; }
        else a.norm_gain = hm.final_gain;
        a.eps = hm.spec.eps; a.out = d_out;
        ProfScope ps(s, MESH_PROF_GEMV);
        return linear_step(a, s->stream);
    }
    {
        ProfScope ps(s, MESH_PROF_PREP);
        rc = hm.final_norm.kind == NORM_LAYER ? layer_norm_rows(s->x, d_rows, hm.final_norm, hm.spec.eps, n_rows, hm.spec.width, h.xa, hm.act, hm.width_pad, s->stream)
                                              : scalar_norm_rows(s->x, d_rows, hm.final_gain, hm.spec.eps, n_rows, hm.spec.width, h.xa, hm.act, hm.width_pad, s->stream);
        if (rc != MESH_OK) return rc;
    }
    ProfScope ps(s, MESH_PROF_GEMV);
    return linear(hm.head, h.xa, hm.act, n_rows, d_out, hm.head.M, s->tune.linear_tile_min_tokens, s->stream);
}

}  // namespace mesh
