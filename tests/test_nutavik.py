"""Nutavik on the CPU: the oracle's mechanisms against closed forms, and what the library does with such a model folder before
it touches a device."""
import json

import numpy as np
import pytest

import nutavik_util as N
from folder_util import error, prompt, write_folder
from oracle import nutavik as O
from test_nadosun import broken
from util import mesh


@pytest.mark.parametrize("name", sorted(N.CONFIGS))
def test_oracle_token_by_token_equals_whole(name):
    cfg = N.CONFIGS[name]
    w = N.random_weights(cfg, 3)
    t = prompt(cfg, 40, 1)
    whole = O.NutavikOracle(cfg, w).forward(t)
    o = O.NutavikOracle(cfg, w)
    parts = np.concatenate([o.forward(t[i:i + 1]) for i in range(20)] + [o.forward(t[20:22]), o.forward(t[22:])])
    assert np.abs(parts - whole).max() < 1e-8


def test_rotation_depends_on_distance_only_and_scaling_meets_its_ends():
    rot = {"dims": 8, "base": 100.0}
    rng = np.random.Generator(np.random.PCG64(1))
    a, b = rng.standard_normal((1, 8)), rng.standard_normal((1, 8))
    s = [float((O.rotate(a, [p + 5], rot) @ O.rotate(b, [p], rot).T)[0, 0]) for p in (0, 3, 1000)]
    assert np.allclose(s, s[0]) and np.allclose(O.rotate(a, [0], rot), a)
    u = O.rotate(np.array([[1.0, 0, 1, 0, 0, 0, 0, 0]]), [2], rot)[0]
    assert np.allclose(u[:4], [np.cos(2), np.sin(2), np.cos(2 * 100 ** -0.25), np.sin(2 * 100 ** -0.25)])
    # pairs that turn often keep their frequency, pairs that hardly turn have it divided
    f, one = O.rotation({"dims": 32, "base": 10000.0})
    g, gain = O.rotation({"dims": 32, "base": 10000.0, "scaling": {"factor": 8.0, "original": 512, "fast": 16.0, "slow": 1.0}})
    assert one == 1.0 and np.isclose(gain, 0.1 * np.log(8.0) + 1)
    assert np.isclose(g[0], f[0]) and np.isclose(g[-1], f[-1] / 8) and ((g <= f) & (g >= f / 8 - 1e-15)).all() and len(set(np.round(f / g, 6))) > 3


def test_latent_attention_with_equal_scores_is_the_gated_mean():
    m = {"heads": 2, "dim": 3, "rot_dim": 2, "vdim": 4, "kv_rank": 5, "q_rank": 2, "scale": 0.5, "rot": {"dims": 2, "base": 10.0}}
    rng = np.random.Generator(np.random.PCG64(0))
    h = rng.standard_normal((7, 6))
    w = {"m.dq": np.ones((2, 6)), "m.dq.norm": np.ones(2), "m.uq": np.zeros((10, 2)), "m.dkv": rng.standard_normal((7, 6)), "m.dkv.norm": rng.standard_normal(5),
         "m.uk": rng.standard_normal((6, 5)), "m.uv": rng.standard_normal((8, 5)), "m.g": rng.standard_normal((2, 6)), "m.o": np.eye(8)}
    c, r = O.latent_rows(w, "m", m, 1e-5, h, np.arange(7))
    out = O.latent_attention(w, "m", m, 1e-5, h, c, r, np.arange(7))
    raw = (h @ w["m.dkv"].T)[:, :5]
    lat = raw / np.sqrt((raw ** 2).mean(axis=1, keepdims=True) + 1e-5) * w["m.dkv.norm"]
    gate = 1 / (1 + np.exp(-(h @ w["m.g"].T)))
    for t in range(7):
        want = (lat[:t + 1].mean(axis=0) @ w["m.uv"].T).reshape(2, 4) * gate[t][:, None]
        assert np.allclose(out[t], want.reshape(-1), atol=1e-12)


def test_delta_state_recalls_the_last_value_written_under_a_key():
    """Without decay and with steps of 1 the state maps a unit key to the last value written under it, and forgets the one before."""
    m = {"heads": 1, "kv_heads": 1, "dim": 2, "vdim": 3, "conv": 1}
    big = 40.0
    w = {"m.q": np.eye(2, 8) * big, "m.k": np.eye(2, 8) * big, "m.v": np.eye(3, 8, 2), "m.b": np.full((1, 8), 0.0), "m.a": np.zeros((1, 8)), "m.A_log": np.array([-60.0]),
         "m.dt_bias": np.zeros(1), "m.g": np.zeros((3, 8)), "m.o": np.eye(3), "m.norm": np.ones(3)}
    for n, k in (("q", 2), ("k", 2), ("v", 3)):
        w["m.%s.conv" % n] = np.ones((k, 1))
    w["m.b"][0, 5] = big                                   # coordinate 5 is 1 in every token
    w["m.g"][:, 5] = big
    def token(key, value):
        return np.concatenate([np.eye(2)[key], value, [1.0, 0, 0]])
    h = np.stack([token(0, [3.0, 1, 2]), token(1, [5.0, 4, 9]), token(0, [7.0, 8, 6])])
    _, (S, *_) = O.delta(w, "m", m, 1e-6, h, (np.zeros((1, 2, 3)), np.zeros((0, 2)), np.zeros((0, 2)), np.zeros((0, 3))))
    silu = lambda z: z / (1 + np.exp(-z))                  # noqa: E731
    assert np.allclose(S[0], [silu(np.array([7.0, 8, 6])), silu(np.array([5.0, 4, 9]))], rtol=1e-4)


def test_short_conv_taps():
    y = np.arange(1.0, 6.0)[:, None]
    out, tail = O.short_conv(y, np.array([[100.0, 10.0, 1.0]]), np.zeros((2, 1)))
    lin = np.array([1, 12, 123, 234, 345.0])
    assert np.allclose(out[:, 0], lin / (1 + np.exp(-lin))) and np.allclose(tail[:, 0], [4, 5])


def test_gla_decays_channel_by_channel():
    m = {"heads": 1, "dim": 2, "vdim": 1, "tau": 2.0}
    w = {"m.q": np.array([[1.0, 0]]).repeat(2, 0), "m.k": np.array([[1.0, 0]]).repeat(2, 0), "m.v": np.array([[1.0, 0]]), "m.g": np.array([[50.0, 0]]), "m.o": np.eye(1),
         "m.a1": np.zeros((1, 2)), "m.a2": np.zeros((2, 1)), "m.a2.b": np.log([1.0, 1 / 3]), "m.norm": np.ones(1)}
    h = np.array([[1.0, 0]] * 4)
    _, S = O.gla(w, "m", m, 1e-6, h, np.zeros((1, 2, 1)))
    for d, alpha in enumerate((0.5 ** 0.5, 0.25 ** 0.5)):
        assert np.isclose(S[0, d, 0], sum(alpha ** i for i in range(4)))


def test_norm_and_feed_forward():
    v = np.array([[1.0, 3.0]])
    assert np.allclose(O.layer_norm(v, np.array([2.0, 1.0]), np.array([0.5, 0.0]), 3.0), [[-0.5, 0.5]])
    w = {"f.up": np.array([[1.0, 0], [0, -1]]), "f.down": np.eye(2)}
    assert np.allclose(O.feed_forward(w, "f", np.array([[3.0, 2.0]])), [[9.0, 0.0]])


def test_needle_weights_make_a_far_key_show():
    cfg = N.config(60, 96, [N.latent(2, 16, 8, 16, 24, 20)])
    w = N.needle_weights(cfg, 5, 7, 9)
    t = prompt(cfg, 80, 2, avoid=(7, 9))
    t[79] = 9
    u = t.copy()
    u[3] = 7
    a, b = (O.NutavikOracle(cfg, w).forward(x)[79:] for x in (t, u))
    assert error(a, b) > 0.2


# ------------------------------------------------------------------------------------------------ the library
def test_probe_reads_the_folder(tmp_path):
    m = mesh()
    cfg = N.CONFIGS["mixed"]
    p = write_folder(str(tmp_path / "model"), cfg, N.random_weights(cfg, 1))
    i = m.model_probe(p)
    assert (i.arch, i.n_layer, i.n_embd, i.n_vocab, i.n_head, i.head_dim, i.n_ff) == (b"Nutavik", 6, 136, 211, 6, 33, 100)
    assert abs(i.rms_eps - 1e-4) < 1e-10


@pytest.mark.parametrize("path,value,code,fragment", [
    (("residual_mult",), None, "ERR_FORMAT", "residual_mult"),
    (("logit_scale",), "2", "ERR_FORMAT", "logit_scale"),
    (("norm",), None, "ERR_FORMAT", "norm.eps"),
    (("layers", 0, "mixer", "q_rank"), None, "ERR_FORMAT", "layers[0].mixer.q_rank"),
    (("layers", 0, "mixer", "scale"), None, "ERR_FORMAT", "layers[0].mixer.scale"),
    (("layers", 0, "mixer", "rot"), None, "ERR_FORMAT", "rot missing"),
    (("layers", 0, "mixer", "rot", "dims"), 9, "ERR_FORMAT", "odd"),
    (("layers", 0, "mixer", "rot", "dims"), 8, "ERR_FORMAT", "differs from rot_dim"),
    (("layers", 0, "mixer", "rot", "scaling", "fast"), None, "ERR_FORMAT", "scaling.fast"),
    (("layers", 0, "mixer", "rot", "scaling", "factor"), 0, "ERR_FORMAT", "not positive"),
    (("layers", 3, "mixer", "kv_from"), 1, "ERR_FORMAT", "not an earlier latent_attention layer"),
    (("layers", 3, "mixer", "kv_from"), 3, "ERR_FORMAT", "not an earlier latent_attention layer"),
    (("layers", 3, "mixer", "kv_from"), -1, "ERR_FORMAT", "kv_from"),
    (("layers", 3, "mixer", "kv_rank"), 43, "ERR_FORMAT", "differ from those of layer 0"),
    (("layers", 3, "mixer", "rot", "base"), 5001.0, "ERR_FORMAT", "differ from those of layer 0"),
    (("layers", 1, "mixer", "kv_heads"), 4, "ERR_FORMAT", "not a multiple"),
    (("layers", 1, "mixer", "conv"), None, "ERR_FORMAT", "layers[1].mixer.conv"),
    (("layers", 2, "mixer", "tau"), 0, "ERR_FORMAT", "tau"),
    (("layers", 2, "mixer", "vdim"), 0, "ERR_FORMAT", "layers[2].mixer.vdim"),
    (("layers", 2, "type"), "mamba", "ERR_UNSUPPORTED", "layers[2].type 'mamba'"),
])
def test_inconsistent_config_is_refused(tmp_path, path, value, code, fragment):
    m = mesh()
    (tmp_path / "config.json").write_text(json.dumps(broken(N.CONFIGS["mixed"], path, value)))
    with pytest.raises(m.MeshError) as e:
        m.model_probe(str(tmp_path))
    assert e.value.code == getattr(m, code) and fragment in e.value.message, e.value.message
