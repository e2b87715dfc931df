"""Small random Nadosun models for the tests: configurations, weights (as the bf16 values a file can hold) and the folder
with config.json and model.safetensors, written byte by byte."""
import numpy as np

from folder_util import bf16, error, prompt, safetensors_bytes, write_folder  # noqa: F401


def attention(heads, kv_heads, dim, window, scale=None, ff=None):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": ff} if ff else None,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale, "mask": {"size": window}}}


def mingru(width, ff=None):
    return {"type": "mingru", "mlp": {"kind": "dense", "ff": ff} if ff else None, "mixer": {"width": width}}


def config(vocab, width, side, layers, eps=1e-5, scale=1.0):
    return {"architecture": "Nadosun", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "token_side": {"dim": side}, "layers": layers}


CONFIGS = {
    # widths that are no multiple of a tile, heads smaller than a cache row, a feed-forward behind a recurrent layer
    "mixed": config(211, 136, 12, [mingru(72, ff=100), attention(6, 2, 24, 9), attention(4, 4, 64, 33, scale=0.2, ff=90), mingru(200)], eps=1e-4, scale=0.3),
    "wide-heads": config(150, 256, 32, [attention(8, 1, 128, 70, ff=300), mingru(64), attention(5, 5, 96, 20, scale=0.15)], scale=2.0),
    "odd-shapes": config(97, 98, 7, [attention(3, 1, 160, 40, ff=33), attention(20, 1, 16, 150), mingru(31, ff=65), attention(14, 2, 40, 65)], eps=1e-6, scale=0.7),
    "ones": config(40, 64, 1, [attention(1, 1, 8, 1, ff=1), mingru(1), attention(2, 1, 4, 2, scale=1.0)], eps=1e-3),
    "recurrent-only": config(64, 64, 8, [mingru(64), mingru(128, ff=64)]),
    "attention-only": config(64, 128, 16, [attention(2, 2, 64, 16, ff=128), attention(4, 2, 32, 300)]),
}


def random_weights(cfg, seed):
    rng = np.random.Generator(np.random.PCG64(seed))
    E, S, V, n = cfg["width"], cfg["token_side"]["dim"], cfg["vocab"], len(cfg["layers"])
    w = {"embed": rng.standard_normal((V, E)), "side.embed": rng.standard_normal((V, n * S)), "final.norm": np.float32(1.3), "head": rng.standard_normal((V, E)) / np.sqrt(E)}

    def mat(name, rows, cols, gain=1.0):
        w[name] = rng.standard_normal((rows, cols)) * (gain / np.sqrt(cols))

    for i, l in enumerate(cfg["layers"]):
        p, m = "l%d." % i, l["mixer"]
        if l["type"] == "attention":
            hd, gd = m["heads"] * m["dim"], m["kv_heads"] * m["dim"]
            mat(p + "mix.q", hd, E)
            mat(p + "mix.k", gd, E)
            mat(p + "mix.o", E, hd)
            w[p + "mix.q.norm"] = 1.5 + 0.5 * rng.standard_normal(hd)
            w[p + "mix.k.norm"] = 1.5 + 0.5 * rng.standard_normal(gd)
        else:
            W = m["width"]
            for t in "zxg":
                mat(p + "mix." + t, W, E, 0.6)
            mat(p + "mix.o", E, W)
            w[p + "mix.z.b"] = -1.5 + rng.standard_normal(W)
            w[p + "mix.x.b"] = 0.3 * rng.standard_normal(W)
        w[p + "norm1"] = np.float32(0.5 + rng.random())
        w[p + "ls1"] = 0.5 + 0.5 * rng.random(E)
        if l["mlp"]:
            mat(p + "mlp.up", l["mlp"]["ff"], E)
            mat(p + "mlp.down", E, l["mlp"]["ff"])
            w[p + "mlp.act"] = 0.2 + rng.random(4)
            w[p + "norm2"] = np.float32(0.5 + rng.random())
            w[p + "ls2"] = 0.5 + 0.5 * rng.random(E)
        mat(p + "side.gate", S, E)
        mat(p + "side.proj", E, S)
        w[p + "side.norm"] = 0.5 * rng.standard_normal(E)
    return {k: bf16(v).reshape(np.shape(v)) for k, v in w.items()}


def only(w, cfg, keep):
    """The weights with every addition to the residual stream but `keep` ("mixer", "ff", "side" or "") scaled to nothing."""
    w = dict(w)
    for i, l in enumerate(cfg["layers"]):
        p = "l%d." % i
        for part, name in (("mixer", "ls1"), ("ff", "ls2"), ("side", "side.norm")):
            if part != keep and p + name in w:
                w[p + name] = np.zeros_like(w[p + name])
    return w


def needle_weights(cfg, seed, needle, asker, strength):
    """Random weights in which every attention layer's query of token `asker` finds the key of token `needle` with a score
    far above all others: the two tokens' embeddings stand out in two coordinates, which the projections turn into one common
    direction per head."""
    w = random_weights(cfg, seed)
    e = w["embed"].copy() * 0.3
    e[:, :2] = 0
    e[needle, 0] = strength
    e[asker, 1] = strength
    w["embed"] = bf16(e)
    for i, l in enumerate(cfg["layers"]):
        if l["type"] != "attention":
            continue
        m, p = l["mixer"], "l%d.mix." % i
        rng = np.random.Generator(np.random.PCG64(seed + 100 + i))
        d = rng.standard_normal(m["dim"])
        q, k = w[p + "q"].copy(), w[p + "k"].copy()
        q[:, :2] = 0
        k[:, :2] = 0
        q[:, 1] = np.tile(d, m["heads"])
        k[:, 0] = np.tile(d, m["kv_heads"])
        w[p + "q"], w[p + "k"] = bf16(q), bf16(k)
        w[p + "q.norm"] = np.ones_like(w[p + "q.norm"])
        w[p + "k.norm"] = np.ones_like(w[p + "k.norm"])
        w["l%d.norm1" % i] = np.float32(8.0)         # what attention finds outweighs the embeddings' own size
    return w
