// See model_config.hpp.  Host-only.
#include "model_config.hpp"

#include <sys/stat.h>

#include <algorithm>
#include <cmath>
#include <cstdio>

#include "json.hpp"
#include "mesh_common.hpp"
#include "registry.hpp"

namespace mesh {

namespace {

constexpr uint64_t MAX_VOCAB = 1u << 22, MAX_ROWS = 1u << 18, MAX_LAYERS = 4096, MAX_HEADS = 1u << 12, MAX_DIM = 1u << 12, MAX_WINDOW = 1u << 30, MAX_TAPS = 64;

bool read_file(const std::string &path, std::string &out) {
    FILE *f = fopen(path.c_str(), "rb");
    if (!f) return false;
    char buf[65536];
    size_t n;
    while ((n = fread(buf, 1, sizeof buf, f)) > 0 && out.size() < (64u << 20)) out.append(buf, n);
    const bool ok = !ferror(f);
    fclose(f);
    return ok;
}

// `where.name` as a whole number in [1, max]
int need_count(const JsonValue &v, const char *name, const std::string &where, uint64_t max, int &out) {
    const JsonValue *f = v.get(name);
    uint64_t n = 0;
    if (!f || !f->as_count(max, n) || n == 0) return fail(MESH_ERR_FORMAT, "config.json: %s%s missing or not a whole number in [1, %llu]", where.c_str(), name, (unsigned long long)max);
    out = (int)n;
    return MESH_OK;
}

int need_number(const JsonValue *v, const char *name, const std::string &where, float &out) {
    const JsonValue *f = v ? v->get(name) : nullptr;
    if (!f || f->kind != JsonValue::NUMBER) return fail(MESH_ERR_FORMAT, "config.json: %s%s missing or not a number", where.c_str(), name);
    out = (float)f->num;
    return MESH_OK;
}

int need_real(const JsonValue *v, const char *name, const std::string &where, double &out) {
    const JsonValue *f = v ? v->get(name) : nullptr;
    if (!f || f->kind != JsonValue::NUMBER) return fail(MESH_ERR_FORMAT, "config.json: %s%s missing or not a number", where.c_str(), name);
    out = f->num;
    return MESH_OK;
}

int rotary_of(const JsonValue *rot, const std::string &where, RotarySpec &r) {
    if (!rot || rot->kind != JsonValue::OBJECT) return fail(MESH_ERR_FORMAT, "config.json: %srot missing", where.c_str());
    const std::string w = where + "rot.";
    int rc;
    if ((rc = need_count(*rot, "dims", w, MAX_DIM, r.dims)) || (rc = need_real(rot, "base", w, r.base))) return rc;
    if (r.dims % 2 || !(r.base > 1.0)) return fail(MESH_ERR_FORMAT, "config.json: %sdims %d is odd, or base %g is not above 1", w.c_str(), r.dims, r.base);
    const JsonValue *s = rot->get("scaling");
    if (!s || s->is_null()) return MESH_OK;
    const std::string ws = w + "scaling.";
    if ((rc = need_real(s, "factor", ws, r.factor)) || (rc = need_real(s, "original", ws, r.original)) || (rc = need_real(s, "fast", ws, r.fast)) || (rc = need_real(s, "slow", ws, r.slow)))
        return rc;
    if (!(r.factor > 0 && r.original > 0 && r.fast > 0 && r.slow > 0)) return fail(MESH_ERR_FORMAT, "config.json: %s: a number is not positive", (w + "scaling").c_str());
    r.scaled = true;
    return MESH_OK;
}

int latent_of(const JsonValue &mx, const std::string &w, MixerSpec &m) {
    int rc;
    m.kind = MIXER_LATENT;
    if ((rc = need_count(mx, "heads", w, MAX_HEADS, m.heads)) || (rc = need_count(mx, "dim", w, MAX_DIM, m.dim)) || (rc = need_count(mx, "vdim", w, MAX_DIM, m.vdim)) ||
        (rc = need_count(mx, "rot_dim", w, MAX_DIM, m.rot_dim)) || (rc = need_count(mx, "kv_rank", w, MAX_ROWS, m.kv_rank)) ||
        (rc = need_count(mx, "q_rank", w, MAX_ROWS, m.q_rank)) || (rc = need_number(&mx, "scale", w, m.scale)) || (rc = rotary_of(mx.get("rot"), w, m.rot)))
        return rc;
    m.kv_heads = 1;
    if (m.rot.dims != m.rot_dim) return fail(MESH_ERR_FORMAT, "config.json: %srot.dims %d differs from rot_dim %d", w.c_str(), m.rot.dims, m.rot_dim);
    const JsonValue *from = mx.get("kv_from");
    if (from && !from->is_null()) {
        uint64_t n = 0;
        if (!from->as_count(MAX_LAYERS, n)) return fail(MESH_ERR_FORMAT, "config.json: %skv_from is not a layer", w.c_str());
        m.kv_from = (int)n;
    }
    return MESH_OK;
}

int matrix_state_of(const JsonValue &mx, const std::string &w, MixerSpec &m) {
    int rc;
    if ((rc = need_count(mx, "heads", w, MAX_HEADS, m.heads)) || (rc = need_count(mx, "dim", w, MAX_DIM, m.dim)) || (rc = need_count(mx, "vdim", w, MAX_DIM, m.vdim))) return rc;
    m.kv_heads = m.heads;
    if (m.kind == MIXER_GLA) {
        if ((rc = need_number(&mx, "tau", w, m.tau)) != MESH_OK) return rc;
        return m.tau > 0.f ? MESH_OK : fail(MESH_ERR_FORMAT, "config.json: %stau is not positive", w.c_str());
    }
    if ((rc = need_count(mx, "kv_heads", w, MAX_HEADS, m.kv_heads)) || (rc = need_count(mx, "conv", w, MAX_TAPS, m.taps))) return rc;
    if (m.heads % m.kv_heads) return fail(MESH_ERR_FORMAT, "config.json: %sheads %d is not a multiple of kv_heads %d", w.c_str(), m.heads, m.kv_heads);
    return MESH_OK;
}

int mixer_of(const JsonValue &layer, const std::string &where, MixerSpec &m) {
    const JsonValue *type = layer.get("type"), *mx = layer.get("mixer");
    if (!type || type->kind != JsonValue::STRING || !mx || mx->kind != JsonValue::OBJECT) return fail(MESH_ERR_FORMAT, "config.json: %stype / mixer missing", where.c_str());
    const std::string w = where + "mixer.";
    int rc;
    if (type->str == "mingru") {
        m.kind = MIXER_MIN_GRU;
        return need_count(*mx, "width", w, MAX_ROWS, m.width);
    }
    if (type->str == "latent_attention") return latent_of(*mx, w, m);
    if (type->str == "delta" || type->str == "gla") {
        m.kind = type->str == "delta" ? MIXER_DELTA : MIXER_GLA;
        return matrix_state_of(*mx, w, m);
    }
    if (type->str != "attention")
        return fail(MESH_ERR_UNSUPPORTED, "config.json: %stype '%s' has no mixer (attention, mingru, latent_attention, delta and gla do)", where.c_str(), type->str.c_str());
    m.kind = MIXER_ATTENTION;
    int vdim = 0;
    if ((rc = need_count(*mx, "heads", w, MAX_HEADS, m.heads)) || (rc = need_count(*mx, "kv_heads", w, MAX_HEADS, m.kv_heads)) ||
        (rc = need_count(*mx, "dim", w, MAX_DIM, m.dim)) || (rc = need_number(mx, "scale", w, m.scale)))
        return rc;
    vdim = m.dim;
    if (mx->get("vdim") && (rc = need_count(*mx, "vdim", w, MAX_DIM, vdim)) != MESH_OK) return rc;
    m.vdim = vdim;
    if (vdim != m.dim) return fail(MESH_ERR_FORMAT, "config.json: %svdim %d differs from dim %d, but the values are the keys", w.c_str(), vdim, m.dim);
    if (m.heads % m.kv_heads) return fail(MESH_ERR_FORMAT, "config.json: %sheads %d is not a multiple of kv_heads %d", w.c_str(), m.heads, m.kv_heads);
    const JsonValue *mask = mx->get("mask");
    if (mask && !mask->is_null() && (rc = need_count(*mask, "size", w + "mask.", MAX_WINDOW, m.window)) != MESH_OK) return rc;
    return MESH_OK;
}

}  // namespace

double RotarySpec::freq(int pair) const {
    const double f = pow(base, -2.0 * pair / dims);
    if (!scaled) return f;
    // (fractional) pair that turns `t` times over the original context
    auto turns = [&](double t) { return dims * log(original / (2.0 * M_PI * t)) / (2.0 * log(base)); };
    const double lo = std::max(floor(turns(fast)), 0.0), hi = std::min(ceil(turns(slow)), (double)dims - 1.0);
    const double ramp = std::min(std::max((pair - lo) / std::max(hi - lo, 0.001), 0.0), 1.0);
    return f / factor * ramp + f * (1.0 - ramp);
}

float RotarySpec::gain() const { return scaled ? (float)(0.1 * log(factor) + 1.0) : 1.f; }

bool is_model_folder(const char *path) {
    struct stat st;
    return path && stat(path, &st) == 0 && S_ISDIR(st.st_mode);
}

int model_spec_from_folder(const char *folder, ModelSpec &s) {
    const std::string path = std::string(folder) + "/config.json";
    std::string text, err;
    if (!read_file(path, text)) return fail(MESH_ERR_IO, "cannot read '%s'", path.c_str());
    JsonValue root;
    if (!json_parse(text.data(), text.size(), root, err)) return fail(MESH_ERR_FORMAT, "'%s': %s", path.c_str(), err.c_str());
    const JsonValue *arch = root.get("architecture"), *layers = root.get("layers"), *side = root.get("token_side");
    if (!arch || arch->kind != JsonValue::STRING) return fail(MESH_ERR_FORMAT, "config.json: architecture missing");
    s.arch = arch->str;
    if (!find_arch(s.arch, CONTAINER_FOLDER))
        return fail(MESH_ERR_UNSUPPORTED, "architecture '%s' is not supported in a model folder (%s)", s.arch.c_str(), arch_names(CONTAINER_FOLDER).c_str());
    int rc;
    if ((rc = need_count(root, "vocab", "", MAX_VOCAB, s.vocab)) || (rc = need_count(root, "width", "", MAX_ROWS, s.width)) ||
        (rc = need_number(root.get("norm"), "eps", "norm.", s.eps)))
        return rc;
    // what the design fixes around its layers
    if (s.arch == "Nadosun") {
        s.sinusoid = true;
        if ((rc = need_number(root.get("embedding"), "scale", "embedding.", s.embed_scale)) != MESH_OK) return rc;
        if (!side || (rc = need_count(*side, "dim", "token_side.", MAX_ROWS, s.side_dim)) != MESH_OK)
            return side ? rc : fail(MESH_ERR_FORMAT, "config.json: token_side missing");
    } else {
        s.in_norm = s.out_norm = NORM_LAYER;
        s.ff = FF_RELU2;
        s.tied_head = true;
        if ((rc = need_number(&root, "residual_mult", "", s.residual_mult)) || (rc = need_number(&root, "logit_scale", "", s.logit_scale))) return rc;
    }
    if (!layers || layers->kind != JsonValue::ARRAY || layers->items.empty() || layers->items.size() > MAX_LAYERS)
        return fail(MESH_ERR_FORMAT, "config.json: layers missing or empty");
    for (size_t i = 0; i < layers->items.size(); ++i) {
        const JsonValue &l = layers->items[i];
        const std::string where = "layers[" + std::to_string(i) + "].";
        LayerSpec ls;
        if ((rc = mixer_of(l, where, ls.mixer)) != MESH_OK) return rc;
        const JsonValue *mlp = l.get("mlp");
        if (mlp && !mlp->is_null()) {
            const JsonValue *kind = mlp->get("kind");
            if (!kind || kind->kind != JsonValue::STRING || kind->str != "dense")
                return fail(MESH_ERR_UNSUPPORTED, "config.json: %smlp.kind is not 'dense'", where.c_str());
            if ((rc = need_count(*mlp, "ff", where + "mlp.", MAX_ROWS, ls.ff)) != MESH_OK) return rc;
        }
        const MixerSpec &m = ls.mixer;
        if ((uint64_t)m.heads * (uint64_t)std::max(m.dim + m.rot_dim, m.vdim) > MAX_ROWS)
            return fail(MESH_ERR_UNSUPPORTED, "config.json: %smixer has %d heads of %d", where.c_str(), m.heads, std::max(m.dim + m.rot_dim, m.vdim));
        if (m.kv_from >= 0) {
            const MixerSpec *j = m.kv_from < (int)i ? &s.layers[(size_t)m.kv_from].mixer : nullptr;
            if (!j || j->kind != MIXER_LATENT || j->kv_from >= 0)
                return fail(MESH_ERR_FORMAT, "config.json: %smixer.kv_from %d is not an earlier latent_attention layer with a cache of its own", where.c_str(), m.kv_from);
            if (j->kv_rank != m.kv_rank || j->rot_dim != m.rot_dim || !(j->rot == m.rot))
                return fail(MESH_ERR_FORMAT, "config.json: %smixer.kv_rank, rot_dim or rot differ from those of layer %d, whose cache it reads", where.c_str(), m.kv_from);
        }
        s.layers.push_back(ls);
    }
    return MESH_OK;
}

}  // namespace mesh
