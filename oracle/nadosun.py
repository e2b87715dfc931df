"""Plain restatement of the Nadosun design in float64 numpy: one function per mechanism, token positions as array rows.

Test infrastructure only: nothing of it is shared with the product path.  A model is a `config` dict (the parsed
config.json) and a dict of float arrays by tensor name.

Notation: rms(v) = sqrt(mean(v^2) + eps).  W x is `x @ W.T` for a matrix stored [out, in].
"""
import math

import numpy as np


def sigmoid(z):
    return np.where(z >= 0, 1.0 / (1.0 + np.exp(-np.abs(z))), np.exp(-np.abs(z)) / (1.0 + np.exp(-np.abs(z))))


def silu(z):
    return z * sigmoid(z)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def unit_rms(v, eps):
    """v / rms(v) along the last axis."""
    return v / np.sqrt(np.mean(v * v, axis=-1, keepdims=True) + eps)


def sinusoid(pos, width):
    """Position vectors [T, width]: pair i holds sin and cos of pos / 10000^(2i / width)."""
    pos = np.asarray(pos, np.float64)
    out = np.empty((len(pos), width))
    for i in range(width):
        angle = pos * 10000.0 ** (-2.0 * (i // 2) / width)
        out[:, i] = np.sin(angle) if i % 2 == 0 else np.cos(angle)
    return out


def embed(w, cfg, tokens, pos):
    return w["embed"][tokens] * cfg["embedding"]["scale"] + sinusoid(pos, cfg["width"])


def min_gru(w, p, h, state):
    """h [T, n], state [width] -> (output [T, n], new state): S_t = (1 - z_t) S_{t-1} + z_t c_t, gates from h_t alone."""
    z = sigmoid(h @ w[p + ".z"].T + w[p + ".z.b"])
    u = h @ w[p + ".x"].T + w[p + ".x.b"]
    cand = np.where(u >= 0, u + 0.5, sigmoid(u))
    s = state.copy()
    states = np.empty_like(cand)
    for t in range(len(h)):
        s = (1.0 - z[t]) * s + z[t] * cand[t]
        states[t] = s
    return (states * silu(h @ w[p + ".g"].T)) @ w[p + ".o"].T, s


def attention(w, p, spec, eps, h, keys, values, pos):
    """Windowed grouped-query attention without rotation; the values are the un-normalised keys.

    keys / values: [n_past, kv_heads, dim] of the positions before pos[0]; returns (output, keys, values) extended."""
    H, G, dim = spec["heads"], spec["kv_heads"], spec["dim"]
    T = len(h)
    raw = h @ w[p + ".k"].T
    q = (unit_rms(h @ w[p + ".q"].T, eps) * w[p + ".q.norm"]).reshape(T, H, dim)
    k = (unit_rms(raw, eps) * w[p + ".k.norm"]).reshape(T, G, dim)
    keys = np.concatenate([keys, k])
    values = np.concatenate([values, raw.reshape(T, G, dim)])
    window = spec["mask"]["size"]
    out = np.empty((T, H, dim))
    for t in range(T):
        lo = max(0, pos[t] - window + 1)
        for hd in range(H):
            g = hd // (H // G)
            s = keys[lo:pos[t] + 1, g] @ q[t, hd] * spec["scale"]
            e = np.exp(s - s.max())
            out[t, hd] = (e / e.sum()) @ values[lo:pos[t] + 1, g]
    return out.reshape(T, H * dim) @ w[p + ".o"].T, keys, values


def poly_norm(u, coef, eps):
    a, b, c, e = coef
    return a * unit_rms(u, eps) + b * unit_rms(u ** 2, eps) + c * unit_rms(u ** 3, eps) + e


def feed_forward(w, p, eps, h):
    return poly_norm(h @ w[p + ".up"].T, w[p + ".act"], eps) @ w[p + ".down"].T


def out_norm(y, gain, eps):
    """RMS norm with one number for all coordinates."""
    return unit_rms(y, eps) * gain


def token_side(w, p, dim, layer, eps, x, tokens):
    e = w["side.embed"][tokens][:, layer * dim:(layer + 1) * dim]
    y = (gelu_tanh(x @ w[p + ".side.gate"].T) * e) @ w[p + ".side.proj"].T
    return unit_rms(y, eps) * w[p + ".side.norm"]


class NadosunOracle:
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
            if l["type"] == "mingru":
                self.state.append(np.zeros(m["width"]))
            else:
                self.state.append((np.zeros((0, m["kv_heads"], m["dim"])), np.zeros((0, m["kv_heads"], m["dim"]))))

    def forward(self, tokens):
        cfg, w, eps = self.cfg, self.w, self.cfg["norm"]["eps"]
        tokens = np.asarray(tokens, np.int64)
        pos = np.arange(self.n, self.n + len(tokens))
        x = embed(w, cfg, tokens, pos)
        self.layers = []
        for i, layer in enumerate(cfg["layers"]):
            p = "l%d" % i
            if layer["type"] == "mingru":
                y, self.state[i] = min_gru(w, p + ".mix", x, self.state[i])
            else:
                k, v = self.state[i]
                y, k, v = attention(w, p + ".mix", layer["mixer"], eps, x, k, v, pos)
                self.state[i] = (k, v)
            x = x + out_norm(y, w[p + ".norm1"], eps) * w[p + ".ls1"]
            if layer["mlp"] is not None:
                x = x + out_norm(feed_forward(w, p + ".mlp", eps, x), w[p + ".norm2"], eps) * w[p + ".ls2"]
            x = x + token_side(w, p, cfg["token_side"]["dim"], i, eps, x, tokens)
            self.layers.append(x)
        self.n += len(tokens)
        self.layers = np.stack(self.layers)
        return out_norm(x, w["final.norm"], eps) @ w["head"].T
