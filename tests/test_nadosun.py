"""Nadosun on the CPU: the oracle's mechanisms against closed forms, and what the library does with a model folder before it
touches a device (config.json, safetensors, registry)."""
import json
import os

import numpy as np
import pytest

import nadosun_util as N
from oracle import nadosun as O
from util import mesh


@pytest.mark.parametrize("name", sorted(N.CONFIGS))
def test_oracle_token_by_token_equals_whole(name):
    cfg = N.CONFIGS[name]
    w = N.random_weights(cfg, 3)
    t = N.prompt(cfg, 50, 1)
    whole = O.NadosunOracle(cfg, w).forward(t)
    o = O.NadosunOracle(cfg, w)
    parts = np.concatenate([o.forward(t[i:i + 1]) for i in range(20)] + [o.forward(t[20:22]), o.forward(t[22:])])
    assert np.abs(parts - whole).max() < 1e-10


def test_min_gru_closed_form():
    """Constant gates: S_n is the geometric sum of the candidates; the candidate's two branches meet at 1/2."""
    W, n = 4, 6
    w = {"m.z": np.zeros((W, n)), "m.z.b": np.log([1.0, 3.0, 0.25, 1.0]), "m.x": np.zeros((W, n)), "m.x.b": np.array([0.7, 0.0, -0.4, -50.0]),
         "m.g": np.zeros((W, n)), "m.o": np.eye(W)}
    w["m.g"][:, 0] = 1.0
    h = np.zeros((5, n))
    h[:, 0] = 2.0
    out, s = O.min_gru(w, "m", h, np.zeros(W))
    z = np.array([0.5, 0.75, 0.2, 0.5])
    cand = np.array([1.2, 0.5, 1 / (1 + np.exp(0.4)), 1 / (1 + np.exp(50.0))])
    want = np.array([cand * (1 - (1 - z) ** (t + 1)) for t in range(5)])
    assert np.allclose(s, want[-1], rtol=1e-12) and np.allclose(out, want * 2.0 / (1 + np.exp(-2.0)), rtol=1e-12)


def test_attention_window_and_shared_values():
    """With equal scores the output is the mean of the un-normalised keys inside the window."""
    spec = {"heads": 2, "kv_heads": 1, "dim": 3, "scale": 0.5, "mask": {"size": 4}}
    rng = np.random.Generator(np.random.PCG64(0))
    w = {"m.q": np.zeros((6, 5)), "m.k": rng.standard_normal((3, 5)), "m.o": np.eye(6), "m.q.norm": np.ones(6), "m.k.norm": np.ones(3)}
    h = rng.standard_normal((9, 5))
    none = np.zeros((0, 1, 3))
    out, _, _ = O.attention(w, "m", spec, 1e-5, h, none, none, np.arange(9))
    raw = h @ w["m.k"].T
    for t in range(9):
        want = raw[max(0, t - 3):t + 1].mean(axis=0)
        assert np.allclose(out[t], np.tile(want, 2), atol=1e-12)


def test_poly_norm_and_norms():
    u = np.array([[1.0, -2.0, 3.0, 0.5]])
    got = O.poly_norm(u, (2.0, 0.5, -1.0, 0.25), 0.0)
    want = 2 * u / np.sqrt(np.mean(u ** 2)) + 0.5 * u ** 2 / np.sqrt(np.mean(u ** 4)) - u ** 3 / np.sqrt(np.mean(u ** 6)) + 0.25
    assert np.allclose(got, want)
    assert np.allclose(O.out_norm(np.array([3.0, 4.0]), 2.0, 0.5), np.array([3.0, 4.0]) * 2 / np.sqrt(13.0))
    assert np.allclose(O.gelu_tanh(np.array([0.0, 1.0, -30.0, 30.0])), [0.0, 0.8411919906, 0.0, 30.0], atol=1e-9)
    s = O.sinusoid([0, 3], 6)
    assert np.allclose(s[0], [0, 1, 0, 1, 0, 1]) and np.allclose(s[1, 2:4], [np.sin(3 * 10000 ** (-2 / 6)), np.cos(3 * 10000 ** (-2 / 6))])


def test_needle_weights_make_the_window_edge_show():
    """The models of the window tests: one token further away, the needle is out of sight and the asker's output another."""
    cfg = N.config(60, 64, 4, [N.attention(2, 1, 32, 11, scale=0.7)])
    w = N.only(N.needle_weights(cfg, 5, 7, 9, 40.0), cfg, "mixer")
    outs = {}
    for dist in (1, 10, 11, 12):
        t = N.prompt(cfg, 40, 2, avoid=(7, 9))
        t[30], t[30 - dist] = 9, 7
        full = dict(cfg, layers=[N.attention(2, 1, 32, dist + 1, scale=0.7)])
        outs[dist] = (O.NadosunOracle(cfg, w).forward(t)[30], O.NadosunOracle(full, w).forward(t)[30])
    assert N.error(*[a[None] for a in outs[10]]) < 0.02
    assert N.error(*[a[None] for a in outs[11]]) > 0.3 and N.error(*[a[None] for a in outs[12]]) > 0.3


# ------------------------------------------------------------------------------------------------ the library
def test_probe_reads_the_folder(tmp_path):
    m = mesh()
    cfg = N.CONFIGS["mixed"]
    p = N.write_folder(str(tmp_path / "model"), cfg, N.random_weights(cfg, 1))
    i = m.model_probe(p)
    assert (i.arch, i.n_layer, i.n_embd, i.n_vocab, i.n_head, i.n_head_kv, i.head_dim, i.n_ff) == (b"Nadosun", 4, 136, 211, 6, 4, 64, 100)
    assert abs(i.rms_eps - 1e-4) < 1e-10
    with pytest.raises(m.MeshError) as e:
        m.model_probe(str(tmp_path / "absent"))
    assert e.value.code == m.ERR_IO


def broken(cfg, path, value):
    c = json.loads(json.dumps(cfg))
    at = c
    for k in path[:-1]:
        at = at[k]
    if value is None:
        del at[path[-1]]
    else:
        at[path[-1]] = value
    return c


@pytest.mark.parametrize("path,value,code,fragment", [
    (("architecture",), "Sadonun", "ERR_UNSUPPORTED", "'Sadonun' is not supported"),
    (("vocab",), 0, "ERR_FORMAT", "vocab"),
    (("width",), 12.5, "ERR_FORMAT", "width"),
    (("norm", "eps"), None, "ERR_FORMAT", "norm.eps"),
    (("embedding", "scale"), "1", "ERR_FORMAT", "embedding.scale"),
    (("token_side",), None, "ERR_FORMAT", "token_side"),
    (("layers",), [], "ERR_FORMAT", "layers"),
    (("layers", 1, "type"), "lstm", "ERR_UNSUPPORTED", "layers[1].type 'lstm'"),
    (("layers", 1, "mixer", "kv_heads"), 4, "ERR_FORMAT", "not a multiple"),
    (("layers", 1, "mixer", "vdim"), 25, "ERR_FORMAT", "vdim 25"),
    (("layers", 1, "mixer", "mask", "size"), -3, "ERR_FORMAT", "mask.size"),
    (("layers", 0, "mixer", "width"), None, "ERR_FORMAT", "layers[0].mixer.width"),
    (("layers", 0, "mlp", "kind"), "sparse", "ERR_UNSUPPORTED", "layers[0].mlp.kind"),
])
def test_inconsistent_config_is_refused(tmp_path, path, value, code, fragment):
    m = mesh()
    cfg = broken(N.CONFIGS["mixed"], path, value)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    with pytest.raises(m.MeshError) as e:
        m.model_probe(str(tmp_path))
    assert e.value.code == getattr(m, code) and fragment in e.value.message, e.value.message


@pytest.mark.parametrize("text", ["", "{", "{\"a\" 1}", "[1,]", "{} x", "{\"a\": 1e999}", "{\"a\": \"\\x\"}", "[" * 100 + "]" * 100, "nul"])
def test_malformed_json_is_refused(tmp_path, text):
    m = mesh()
    (tmp_path / "config.json").write_text(text)
    with pytest.raises(m.MeshError) as e:
        m.model_probe(str(tmp_path))
    assert e.value.code == m.ERR_FORMAT


def test_json_details_are_read(tmp_path):
    m = mesh()
    cfg = N.CONFIGS["ones"]
    text = json.dumps(cfg, indent=1).replace("Nadosun", "Na\\u0064osun").replace("0.001", "1.0E-3")
    (tmp_path / "config.json").write_text(text)
    i = m.model_probe(str(tmp_path))
    assert i.arch == b"Nadosun" and abs(i.rms_eps - 1e-3) < 1e-9


@pytest.mark.parametrize("damage", ["short", "header beyond file", "bad json", "offsets", "size", "shape"])
def test_damaged_weights_are_refused_before_any_device_call(tmp_path, damage):
    m = mesh()
    cfg = N.CONFIGS["ones"]
    p = N.write_folder(str(tmp_path), cfg, N.random_weights(cfg, 1))
    f = os.path.join(p, "model.safetensors")
    b = open(f, "rb").read()
    n = int.from_bytes(b[:8], "little")
    head = json.loads(b[8:8 + n])
    if damage == "short":
        b = b[:5]
    elif damage == "header beyond file":
        b = (1 << 40).to_bytes(8, "little") + b[8:]
    elif damage == "bad json":
        b = b[:8] + b"]" + b[9:]
    else:
        if damage == "offsets":
            head["head"]["data_offsets"][1] += 1 << 30
        elif damage == "size":
            head["head"]["data_offsets"][1] -= 2
        else:
            head["head"]["shape"] = [-1]
        h = json.dumps(head).encode()
        b = len(h).to_bytes(8, "little") + h + b[8 + n:]
    open(f, "wb").write(b)
    with pytest.raises(m.MeshError) as e:
        m.Stage(p, 0)
    assert e.value.code == m.ERR_FORMAT and "safetensors" in e.value.message


def test_options_that_do_not_fit_are_refused(tmp_path):
    m = mesh()
    cfg = N.CONFIGS["ones"]
    p = N.write_folder(str(tmp_path / "m"), cfg, N.random_weights(cfg, 1))
    for kw, code in ((dict(kv_types=(m.Q8_0, m.Q4_0)), m.ERR_UNSUPPORTED), (dict(precision=7), m.ERR_INVALID), (dict(tuning="step_fused=2"), m.ERR_INVALID)):
        with pytest.raises(m.MeshError) as e:
            m.Stage(p, 0, **kw)
        assert e.value.code == code
    with pytest.raises(m.MeshError) as e:
        m.Stage(p, 1, 9)
    assert e.value.code == m.ERR_INVALID and "layer range" in e.value.message
    import models
    g = os.path.join(str(tmp_path), "t.gguf")
    models.write_model(g, models.CONFIGS["tiny-llama"], [0], seed=1)
    with pytest.raises(m.MeshError) as e:
        m.Stage(g, 0, 1, precision=m.PRECISION_F32)
    assert e.value.code == m.ERR_UNSUPPORTED
    assert m.model_probe(g).arch == b"llama"


def test_portions_of_a_trace_step():
    """A step longer than a call may carry, or with more wanted rows than one returns, is cut without losing a place."""
    m = mesh()
    from mesh_llm_amd import trace
    r = trace.Replayer.__new__(trace.Replayer)
    r.mesh, r.batch_max = m, 300
    want = list(range(0, 260)) + [700, 999]
    parts = list(r._portions(np.zeros(1000, np.int32), want))
    assert parts[0][0] == 0 and parts[-1][1] == 1000 and all(a[1] == b[0] for a, b in zip(parts, parts[1:]))
    assert all(e - b <= 300 and f.sum() <= m.LOGITS_TOKENS_MAX and len(f) == e - b for b, e, f in parts)
    assert [b + int(i) for b, _, f in parts for i in np.flatnonzero(f)] == want
