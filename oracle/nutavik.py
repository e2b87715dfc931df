"""Plain restatement of the Nutavik design in float64 numpy: one function per mechanism, token positions as array rows.

Test infrastructure only: nothing of it is shared with the product path.  A model is a `config` dict (the parsed
config.json) and a dict of float arrays by tensor name.

Notation: rms(v) = sqrt(mean(v^2) + eps).  W x is `x @ W.T` for a matrix stored [out, in].
"""
import math

import numpy as np

from oracle.nadosun import sigmoid, silu, unit_rms

UNIT_EPS = 1e-6      # inside the root of the delta rule's unit vectors


def softplus(z):
    return np.maximum(z, 0.0) + np.log1p(np.exp(-np.abs(z)))


def layer_norm(v, gain, bias, eps):
    c = v - v.mean(axis=-1, keepdims=True)
    return c / np.sqrt(np.mean(c * c, axis=-1, keepdims=True) + eps) * gain + bias


def rotation(rot):
    """Angular frequency of every pair, and the factor on cos and sin (1 without frequency scaling)."""
    dims, base = rot["dims"], rot["base"]
    i = np.arange(dims // 2, dtype=np.float64)
    f = float(base) ** (-2.0 * i / dims)
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def turns(t):        # the (fractional) dimension whose pair turns t times over the original context
        return dims * math.log(s["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(turns(s["fast"])), 0), min(math.ceil(turns(s["slow"])), dims - 1)
    ramp = np.clip((i - lo) / max(hi - lo, 0.001), 0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def rotate(v, pos, rot):
    """v [T, ..., rot_dim]: pairs of neighbours turned by position times frequency."""
    f, gain = rotation(rot)
    n = 2 * len(f)
    a = np.asarray(pos, np.float64)[:, None] * f
    a = a.reshape((len(pos),) + (1,) * (v.ndim - 2) + (-1,))
    c, s = np.cos(a) * gain, np.sin(a) * gain
    out = v.copy()
    out[..., 0:n:2] = v[..., 0:n:2] * c - v[..., 1:n:2] * s
    out[..., 1:n:2] = v[..., 1:n:2] * c + v[..., 0:n:2] * s
    return out


def latent_rows(w, p, m, eps, h, pos):
    """What a layer caches: the latent [T, kv_rank] (normed) and the rotated key part [T, rot_dim] that all heads share."""
    y = h @ w[p + ".dkv"].T
    R = m["kv_rank"]
    return unit_rms(y[:, :R], eps) * w[p + ".dkv.norm"], rotate(y[:, R:], pos, m["rot"])


def latent_attention(w, p, m, eps, h, latent, shared, pos):
    """latent / shared: rows of all positions up to pos[-1], this call's included."""
    H, D, P, V, T = m["heads"], m["dim"], m["rot_dim"], m["vdim"], len(h)
    cq = unit_rms(h @ w[p + ".dq"].T, eps) * w[p + ".dq.norm"]
    q = (cq @ w[p + ".uq"].T).reshape(T, H, D + P)
    qn, qr = q[..., :D], rotate(q[..., D:], pos, m["rot"])
    k = (latent @ w[p + ".uk"].T).reshape(-1, H, D)
    v = (latent @ w[p + ".uv"].T).reshape(-1, H, V)
    gate = sigmoid(h @ w[p + ".g"].T)
    out = np.empty((T, H, V))
    for t in range(T):
        n = pos[t] + 1
        for hd in range(H):
            s = (k[:n, hd] @ qn[t, hd] + shared[:n] @ qr[t, hd]) * m["scale"]
            e = np.exp(s - s.max())
            out[t, hd] = (e / e.sum()) @ v[:n, hd] * gate[t, hd]
    return out.reshape(T, H * V) @ w[p + ".o"].T


def short_conv(y, taps, before):
    """Causal convolution per channel, then silu.  y [T, n], taps [n, K] (last: current token), before [K - 1, n]: the inputs
    ahead of y.  Returns (output, the last K - 1 inputs)."""
    K = taps.shape[1]
    z = np.concatenate([before, y])
    out = sum(z[i:i + len(y)] * taps[:, i] for i in range(K))
    return silu(out), z[len(z) - (K - 1):]


def unit(v):
    return v / np.sqrt(np.sum(v * v, axis=-1, keepdims=True) + UNIT_EPS)


def delta(w, p, m, eps, h, state):
    """state: (S [heads, dim, vdim], three convolution tails)."""
    H, G, D, V, T = m["heads"], m["kv_heads"], m["dim"], m["vdim"], len(h)
    S, tails = state[0].copy(), list(state[1:])
    y = []
    for i, name in enumerate("qkv"):
        c, tails[i] = short_conv(h @ w[p + "." + name].T, w[p + "." + name + ".conv"], tails[i])
        y.append(c)
    q, k = unit(y[0].reshape(T, G, D)) * D ** -0.5, unit(y[1].reshape(T, G, D))
    v = y[2].reshape(T, H, V)
    beta = sigmoid(h @ w[p + ".b"].T)
    g = np.exp(-np.exp(w[p + ".A_log"]) * softplus(h @ w[p + ".a"].T + w[p + ".dt_bias"]))
    out = np.empty((T, H, V))
    for t in range(T):
        for hd in range(H):
            kk, qq = k[t, hd // (H // G)], q[t, hd // (H // G)]
            s = S[hd] * g[t, hd]
            u = beta[t, hd] * (v[t, hd] - s.T @ kk)
            S[hd] = s + np.outer(kk, u)
            out[t, hd] = S[hd].T @ qq
    o = unit_rms(out, eps) * w[p + ".norm"]
    return (o.reshape(T, H * V) * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T, (S, *tails)


def gla(w, p, m, eps, h, S):
    """S [heads, dim, vdim]; every key channel (row of S) has a decay of its own."""
    H, D, V, T = m["heads"], m["dim"], m["vdim"], len(h)
    q = (h @ w[p + ".q"].T * D ** -0.5).reshape(T, H, D)
    k, v = (h @ w[p + ".k"].T).reshape(T, H, D), (h @ w[p + ".v"].T).reshape(T, H, V)
    z = (h @ w[p + ".a1"].T) @ w[p + ".a2"].T + w[p + ".a2.b"]
    alpha = np.exp(-softplus(-z) / m["tau"]).reshape(T, H, D)
    S = S.copy()
    out = np.empty((T, H, V))
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = np.einsum("hdv,hd->hv", S, q[t])
    o = unit_rms(out, eps) * w[p + ".norm"]
    return (o.reshape(T, H * V) * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T, S


def feed_forward(w, p, h):
    return np.maximum(h @ w[p + ".up"].T, 0.0) ** 2 @ w[p + ".down"].T


class NutavikOracle:
    """One sequence.  forward(tokens) continues where the last call stopped and returns the logits [T, vocab]; .layers
    then holds the residual stream after every layer, [n_layers, T, width]."""

    def __init__(self, cfg, tensors):
        self.cfg = cfg
        self.w = {k: np.asarray(v, np.float64) for k, v in tensors.items()}
        self.reset()

    def reset(self):
        self.n = 0
        self.state = []
        for l in self.cfg["layers"]:
            m = l["mixer"]
            if l["type"] == "latent_attention":
                self.state.append(None if "kv_from" in m else (np.zeros((0, m["kv_rank"])), np.zeros((0, m["rot_dim"]))))
            elif l["type"] == "delta":
                qk, K = m["kv_heads"] * m["dim"], m["conv"] - 1
                self.state.append((np.zeros((m["heads"], m["dim"], m["vdim"])), np.zeros((K, qk)), np.zeros((K, qk)), np.zeros((K, m["heads"] * m["vdim"]))))
            else:
                self.state.append(np.zeros((m["heads"], m["dim"], m["vdim"])))

    def mixer(self, i, h, pos):
        layer, w, eps = self.cfg["layers"][i], self.w, self.cfg["norm"]["eps"]
        m, p = layer["mixer"], "l%d.mix" % i
        if layer["type"] == "delta":
            y, self.state[i] = delta(w, p, m, eps, h, self.state[i])
        elif layer["type"] == "gla":
            y, self.state[i] = gla(w, p, m, eps, h, self.state[i])
        else:
            j = m.get("kv_from", i)
            if j == i:
                self.state[i] = tuple(np.concatenate([a, b]) for a, b in zip(self.state[i], latent_rows(w, p, m, eps, h, pos)))
            y = latent_attention(w, p, m, eps, h, *self.state[j], pos)
        return y

    def forward(self, tokens):
        cfg, w, eps, r = self.cfg, self.w, self.cfg["norm"]["eps"], self.cfg["residual_mult"]
        pos = np.arange(self.n, self.n + len(tokens))

        def norm(v, name):
            return layer_norm(v, w[name], w[name + ".b"], eps)

        x = w["embed"][np.asarray(tokens, np.int64)]
        self.layers = []
        for i, layer in enumerate(cfg["layers"]):
            p = "l%d." % i
            x = x + r * norm(self.mixer(i, norm(x, p + "norm1"), pos), p + "norm1b")
            if layer["mlp"] is not None:
                x = x + r * norm(feed_forward(w, p + "mlp", norm(x, p + "norm2")), p + "norm2b")
            self.layers.append(x)
        self.n += len(tokens)
        self.layers = np.stack(self.layers)
        return norm(x, "final.norm") @ w["embed"].T * cfg["logit_scale"]
