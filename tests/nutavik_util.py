"""Small random Nutavik models for the tests: configurations and weights (as the bf16 values a file can hold)."""
import numpy as np

from folder_util import bf16


def latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale=None, base=10000.0, scaling=None, kv_from=None, ff=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
         "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": {"dims": rot_dim, "base": base}}
    if scaling:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def delta(heads, kv_heads, dim, vdim, conv, ff=None):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def gla(heads, dim, vdim, tau, ff=None):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def config(vocab, width, layers, eps=1e-5, residual=1.0, logit=1.0):
    return {"architecture": "Nutavik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": residual, "logit_scale": logit, "layers": layers}


YARN = (4.0, 64, 8.0, 0.5)

CONFIGS = {
    # no size is a multiple of a tile, none equals another; a cache shared over two layers, layers without a feed-forward
    "mixed": config(211, 136, [latent(5, 24, 10, 36, 44, 52, base=5000.0, scaling=YARN, ff=100), delta(6, 2, 20, 28, 4, ff=90), gla(3, 26, 40, 5.0),
                               latent(3, 30, 10, 20, 44, 28, scale=0.2, base=5000.0, scaling=YARN, kv_from=0), delta(2, 2, 33, 17, 2), gla(4, 18, 24, 16.0, ff=33)],
                    eps=1e-4, residual=0.6, logit=1.7),
    # every pair of row lengths the chunk kernel has, and heads beyond it
    "wide-heads": config(150, 256, [latent(2, 128, 64, 128, 300, 200, ff=128), latent(3, 64, 32, 48, 128, 64, scaling=(2.0, 100, 32.0, 1.0)), latent(2, 72, 40, 80, 64, 96),
                                    latent(1, 100, 80, 30, 520, 40), latent(20, 16, 6, 12, 70, 33, kv_from=None), latent(2, 150, 64, 140, 40, 24)], residual=0.8),
    "wide-states": config(97, 98, [delta(2, 1, 130, 200, 4), gla(2, 200, 70, 8.0, ff=65), delta(1, 1, 256, 256, 3), gla(1, 70, 256, 1.0), delta(3, 3, 64, 16, 1)], eps=1e-6, logit=0.5),
    "ones": config(40, 64, [latent(1, 1, 2, 1, 1, 1, ff=1), delta(1, 1, 1, 1, 1), gla(1, 1, 1, 1.0), latent(2, 1, 2, 3, 1, 2, kv_from=0)], eps=1e-3),
    "latent-only": config(64, 128, [latent(4, 32, 16, 24, 48, 40, ff=128), latent(4, 16, 16, 32, 48, 40, kv_from=0, ff=64), latent(4, 16, 16, 32, 48, 40, kv_from=0)]),
    "states-only": config(64, 64, [delta(4, 2, 16, 24, 4, ff=64), gla(2, 32, 16, 16.0)]),
}


def random_weights(cfg, seed, rank=7):
    rng = np.random.Generator(np.random.PCG64(seed))
    E, V = cfg["width"], cfg["vocab"]
    w = {"embed": rng.standard_normal((V, E))}

    def mat(name, rows, cols, gain=1.0):
        w[name] = rng.standard_normal((rows, cols)) * (gain / np.sqrt(cols))

    def norm(name, n, bias=True):
        w[name] = 1.0 + 0.3 * rng.standard_normal(n)
        if bias:
            w[name + ".b"] = 0.2 * rng.standard_normal(n)

    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        x = p + "mix."
        H, v = m["heads"], m["heads"] * m["vdim"]
        if l["type"] == "latent_attention":
            mat(x + "dq", m["q_rank"], E)
            norm(x + "dq.norm", m["q_rank"], False)
            mat(x + "uq", H * (m["dim"] + m["rot_dim"]), m["q_rank"], 1.5)
            if "kv_from" not in m:
                mat(x + "dkv", m["kv_rank"] + m["rot_dim"], E)
                norm(x + "dkv.norm", m["kv_rank"], False)
            mat(x + "uk", H * m["dim"], m["kv_rank"], 1.5)
            mat(x + "uv", v, m["kv_rank"])
            mat(x + "g", H, E)
        else:
            qk = m.get("kv_heads", H) * m["dim"]
            mat(x + "q", qk, E)
            mat(x + "k", qk, E, 1.0 if l["type"] == "delta" else m["dim"] ** -0.5)
            mat(x + "v", v, E)
            mat(x + "g", v, E)
            norm(x + "norm", m["vdim"], False)
            if l["type"] == "delta":
                for t, n in (("q", qk), ("k", qk), ("v", v)):
                    w[x + t + ".conv"] = rng.standard_normal((n, m["conv"])) * m["conv"] ** -0.5
                mat(x + "b", H, E)
                mat(x + "a", H, E)
                w[x + "A_log"] = rng.uniform(-2.0, 1.0, H)
                w[x + "dt_bias"] = rng.uniform(-4.0, 0.0, H)
            else:
                mat(x + "a1", rank, E)
                mat(x + "a2", qk, rank)
                w[x + "a2.b"] = rng.uniform(-1.0, 4.0, qk)
        mat(x + "o", E, v)
        for nm in ("norm1", "norm1b"):
            norm(p + nm, E)
        if l["mlp"]:
            mat(p + "mlp.up", l["mlp"]["ff"], E)
            mat(p + "mlp.down", E, l["mlp"]["ff"])
            for nm in ("norm2", "norm2b"):
                norm(p + nm, E)
    norm("final.norm", E)
    return {k: bf16(a).reshape(np.shape(a)) for k, a in w.items()}


def only(w, cfg, keep):
    """The weights with every addition to the residual stream but those of `keep` (a layer type, "ff" or "") made nothing."""
    w = dict(w)
    for i, l in enumerate(cfg["layers"]):
        for name, part in (("norm1b", l["type"]), ("norm2b", "ff")):
            for k in ("l%d.%s" % (i, name), "l%d.%s.b" % (i, name)):
                if part != keep and k in w:
                    w[k] = np.zeros_like(w[k])
    return w


def needle_weights(cfg, seed, needle, asker, score=14.0):
    """Random weights in which every latent layer's query of token `asker` finds the key of token `needle` with a score far above
    all others: the two tokens' embeddings stand out in a coordinate each, which the first projections turn into one latent each,
    and the query projection maps the one latent onto the other's keys."""
    w = random_weights(cfg, seed)
    e = w["embed"].copy() * 0.3
    e[:, :2] = 0
    e[needle, 0] = e[asker, 1] = 6.0
    w["embed"] = bf16(e)
    for k in ("final.norm", "final.norm.b"):              # (logits from the same table: without what stands out there)
        w[k] = w[k].copy()
        w[k][:2] = 0
    for i, l in enumerate(cfg["layers"]):
        if l["type"] != "latent_attention":
            continue
        m, p = l["mixer"], "l%d.mix." % i
        src = "l%d.mix." % m.get("kv_from", i)
        rng = np.random.Generator(np.random.PCG64(seed + 100 + m.get("kv_from", i)))
        dc, dq = rng.standard_normal(m["kv_rank"]), rng.standard_normal(m["q_rank"])
        w["l%d.norm1" % i] = np.ones(cfg["width"])
        w["l%d.norm1.b" % i] = np.zeros(cfg["width"])
        w[p + "dq"] = w[p + "dq"] * 0.2
        w[p + "dq"][:, 0] = 0
        w[p + "dq"][:, 1] = dq
        w[p + "dq.norm"] = np.ones(m["q_rank"])
        if src == p:
            w[p + "dkv"] = w[p + "dkv"] * 0.2
            w[p + "dkv"][:, :2] = 0
            w[p + "dkv"][:m["kv_rank"], 0] = dc
            w[p + "dkv.norm"] = np.ones(m["kv_rank"])
        c, cq = dc / np.sqrt(np.mean(dc ** 2)), dq / np.sqrt(np.mean(dq ** 2))
        # (keys mostly measure how much of the needle's latent a token has)
        uk = w[p + "uk"] * 0.2 + np.outer(rng.standard_normal(len(w[p + "uk"])), c) * (2.0 / (c @ c))
        w[p + "uk"] = uk
        k = (uk @ c).reshape(m["heads"], m["dim"])
        uq = w[p + "uq"].reshape(m["heads"], m["dim"] + m["rot_dim"], m["q_rank"]) * 0.2
        for h in range(m["heads"]):
            uq[h, :m["dim"]] += np.outer(k[h], cq) * (score / m["scale"] / (k[h] @ k[h]) / (cq @ cq))
        w[p + "uq"] = uq.reshape(w[p + "uq"].shape)
    return {k: bf16(a).reshape(np.shape(a)) for k, a in w.items()}
