// See model_config.hpp.  Host-only.
#include "model_config.hpp"

#include <sys/stat.h>

#include <cmath>
#include <cstdio>

#include "json.hpp"
#include "mesh_common.hpp"
#include "registry.hpp"

namespace mesh {

namespace {

constexpr uint64_t MAX_VOCAB = 1u << 22, MAX_ROWS = 1u << 18, MAX_LAYERS = 4096, MAX_HEADS = 1u << 12, MAX_DIM = 1u << 12, MAX_WINDOW = 1u << 30;

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

int mixer_of(const JsonValue &layer, const std::string &where, MixerSpec &m) {
    const JsonValue *type = layer.get("type"), *mx = layer.get("mixer");
    if (!type || type->kind != JsonValue::STRING || !mx || mx->kind != JsonValue::OBJECT) return fail(MESH_ERR_FORMAT, "config.json: %stype / mixer missing", where.c_str());
    const std::string w = where + "mixer.";
    int rc;
    if (type->str == "mingru") {
        m.kind = MIXER_MIN_GRU;
        return need_count(*mx, "width", w, MAX_ROWS, m.width);
    }
    if (type->str != "attention") return fail(MESH_ERR_UNSUPPORTED, "config.json: %stype '%s' has no mixer (attention and mingru do)", where.c_str(), type->str.c_str());
    m.kind = MIXER_ATTENTION;
    int vdim = 0;
    if ((rc = need_count(*mx, "heads", w, MAX_HEADS, m.heads)) || (rc = need_count(*mx, "kv_heads", w, MAX_HEADS, m.kv_heads)) ||
        (rc = need_count(*mx, "dim", w, MAX_DIM, m.dim)) || (rc = need_number(mx, "scale", w, m.scale)))
        return rc;
    vdim = m.dim;
    if (mx->get("vdim") && (rc = need_count(*mx, "vdim", w, MAX_DIM, vdim)) != MESH_OK) return rc;
    if (vdim != m.dim) return fail(MESH_ERR_FORMAT, "config.json: %svdim %d differs from dim %d, but the values are the keys", w.c_str(), vdim, m.dim);
    if (m.heads % m.kv_heads) return fail(MESH_ERR_FORMAT, "config.json: %sheads %d is not a multiple of kv_heads %d", w.c_str(), m.heads, m.kv_heads);
    const JsonValue *mask = mx->get("mask");
    if (mask && !mask->is_null() && (rc = need_count(*mask, "size", w + "mask.", MAX_WINDOW, m.window)) != MESH_OK) return rc;
    return MESH_OK;
}

}  // namespace

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
        (rc = need_number(root.get("norm"), "eps", "norm.", s.eps)) || (rc = need_number(root.get("embedding"), "scale", "embedding.", s.embed_scale)))
        return rc;
    if (!side || (rc = need_count(*side, "dim", "token_side.", MAX_ROWS, s.side_dim)) != MESH_OK)
        return side ? rc : fail(MESH_ERR_FORMAT, "config.json: token_side missing");
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
        if (ls.mixer.kind == MIXER_ATTENTION && (uint64_t)ls.mixer.heads * ls.mixer.dim > MAX_ROWS)
            return fail(MESH_ERR_UNSUPPORTED, "config.json: %smixer has %d heads of %d", where.c_str(), ls.mixer.heads, ls.mixer.dim);
        s.layers.push_back(ls);
    }
    return MESH_OK;
}

}  // namespace mesh
