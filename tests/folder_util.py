"""Model folders for the tests, written byte by byte, and sequences fed through a stage in portions."""
import json
import os

import numpy as np

from util import mesh


def bf16(a):
    """Rounded to bfloat16 (nearest, ties to even), as float32."""
    u = np.ascontiguousarray(a, np.float32).view(np.uint32)
    return ((u + 0x7FFF + ((u >> 16) & 1)) & np.uint32(0xFFFF0000)).view(np.float32)


def safetensors_bytes(tensors):
    """Weights as BF16 entries."""
    head, blobs, at = {}, [], 0
    for name, a in tensors.items():
        b = (np.ascontiguousarray(a, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[name] = {"dtype": "BF16", "shape": list(np.shape(a)), "data_offsets": [at, at + len(b)]}
        blobs.append(b)
        at += len(b)
    h = json.dumps(head).encode()
    return len(h).to_bytes(8, "little") + h + b"".join(blobs)


def write_folder(path, cfg, tensors):
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    with open(os.path.join(path, "model.safetensors"), "wb") as f:
        f.write(safetensors_bytes(tensors))
    return path


def prompt(cfg, n, seed, avoid=()):
    t = np.random.Generator(np.random.PCG64(seed)).integers(0, cfg["vocab"], n).astype(np.int32)
    while np.isin(t, avoid).any():
        t = np.where(np.isin(t, avoid), (t + 1) % cfg["vocab"], t).astype(np.int32)
    return t


def error(got, want):
    """Largest over the rows: rms of the difference (its mean taken off) over the rms of all of `want`."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d -= d.mean(axis=-1, keepdims=True)
    return float(np.sqrt((d ** 2).mean(axis=-1)).max() / np.sqrt((want ** 2).mean()))


def open_stage(folder, prec, begin=0, end=-1, n_ctx=512, n_seq=4, batch=256, **kw):
    m = mesh()
    return m.Stage(folder, begin, end, n_ctx=n_ctx, n_seq_max=n_seq, n_batch_max=batch, precision=m.PRECISION_F32 if prec == "f32" else m.PRECISION_DEFAULT, **kw)


class Seq:
    """One sequence of a session, fed in portions."""

    def __init__(self, stage, session, seq=0):
        self.st, self.ses, self.seq, self.n = stage, session, seq, 0

    def feed(self, tokens, out=None, want=None):
        m = mesh()
        pos = np.arange(self.n, self.n + len(tokens), dtype=np.int32)
        raw = self.ses.decode(np.asarray(tokens, np.int32), pos, seq=np.full(len(tokens), self.seq, np.int32), in_fmt=m.TOKENS,
                              out_fmt=m.LOGITS if out is None else out, want=want)
        self.n += len(tokens)
        return raw.view(np.float32).reshape(-1, self.st.info.n_vocab if out is None else self.st.info.n_embd)


def run(stage, tokens, portions, seq=0, session=None, last=10 ** 9, **options):
    """Logits of the last `last` tokens, fed in portions to a sequence that starts with them."""
    ses = session or stage.session(**options)
    s = Seq(stage, ses, seq)
    rows, at = [], 0
    for p in portions:
        rows.append(s.feed(tokens[at:at + p], want=np.arange(at, at + p) >= len(tokens) - last))
        at += p
    assert at == len(tokens)
    if session is None:
        ses.close()
    return np.concatenate(rows)


def oracle_greedy(orc, prompt, n, forced=None):
    orc.reset()
    lg = orc.forward(prompt)[-1]
    toks, margins = [], []
    for i in range(n):
        top = np.sort(lg)[-2:]
        toks.append(int(lg.argmax()))
        margins.append(float(top[1] - top[0]))
        lg = orc.forward([toks[-1] if forced is None else forced[i]])[-1]
    return toks, margins


def check_greedy(orc, prompt, got, tol):
    """Every generated token is the oracle's argmax, or one the precision cannot tell from it."""
    toks, margins = oracle_greedy(orc, prompt, len(got), forced=got)
    for a, b, mg in zip(got, toks, margins):
        assert a == b or mg < tol, (a, b, mg)
    assert sum(a == b for a, b in zip(got, toks)) >= 0.9 * len(got)
