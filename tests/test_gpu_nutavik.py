"""Nutavik on the GPU against the plain oracle: each mechanism alone, whole prompts against portions and token-by-token
decoding, far keys that show, sequences side by side and reused, layer ranges, greedy generation through the stage, and the
trace runner."""
import json
import os
import subprocess
import urllib.request

import numpy as np
import pytest

import nutavik_util as N
from folder_util import Seq, check_greedy, error, open_stage, prompt, run, write_folder
from oracle.nutavik import NutavikOracle
from util import ROOT, mesh

pytestmark = pytest.mark.gpu

# rms of a row's difference over the rms of all rows (folder_util.error).  With bf16 single rows may be further off than all
# together: a read-out that is small before its norm, the first tokens' in particular, is rounded more coarsely.
LIMIT = {"bf16": 2e-2, "f32": 3e-5}
LIMIT_ROW = {"bf16": 1e-1, "f32": 3e-5}
BOTH = pytest.mark.parametrize("prec", ["bf16", "f32"])


def made(tmp, name, seed=11, change=None):
    """(config, weights, folder, oracle) of a configuration; `change` rewrites the weights."""
    cfg = N.CONFIGS[name] if isinstance(name, str) else name
    w = N.random_weights(cfg, seed)
    if change:
        w = change(w, cfg)
    return cfg, w, write_folder(str(tmp / "model"), cfg, w), NutavikOracle(cfg, w)


def off(got, want, prec):
    """Distance in units of the limits."""
    d = np.asarray(got, np.float64) - want
    return max(np.sqrt(np.mean(d ** 2)) / np.sqrt(np.mean(np.asarray(want) ** 2)) / LIMIT[prec], error(got, want) / LIMIT_ROW[prec])


# ------------------------------------------------------------------------------------------------ mechanisms
@BOTH
@pytest.mark.parametrize("keep", ["", "latent_attention", "delta", "gla", "ff"])
@pytest.mark.parametrize("name", ["mixed", "wide-heads", "wide-states", "ones"])
def test_each_mechanism_alone(tmp_path, name, keep, prec):
    """The residual stream after the last layer with every other addition made nothing: the embedding (""), one kind of mixer, the
    feed-forwards; many tokens and one."""
    m = mesh()
    cfg = N.CONFIGS[name]
    if keep not in ("", "ff") and not any(l["type"] == keep for l in cfg["layers"]):
        pytest.skip("no such layer")
    cfg, w, folder, orc = made(tmp_path, name, change=lambda w, c: N.only(w, c, keep))
    t = prompt(cfg, 90, 5)
    orc.forward(t)
    want = orc.layers[-1]
    st = open_stage(folder, prec)
    for chunk in (1000, 2):                  # latent attention over cached latents, and over projected keys and values
        ses = st.session(latent_chunk_min_tokens=chunk)
        s = Seq(st, ses)
        got = np.concatenate([s.feed(t[:70], out=m.F32)] + [s.feed(t[i:i + 1], out=m.F32) for i in range(70, 90)])
        assert np.isfinite(got).all()
        base = w["embed"][t]
        added = np.sqrt(np.mean((want - base) ** 2)) if keep else np.sqrt(np.mean(want ** 2))
        err = np.sqrt(np.mean((got - want) ** 2, axis=-1)) / max(added, 1e-3)
        # (bf16: a vector that is small before its output norm is rounded more coarsely than the rest)
        limit, limit_row = (1e-7, 1e-7) if keep == "" else (1e-5, 5e-5) if prec == "f32" else (1.5e-2, 1e-1)
        if name == "ones" and keep:          # (sums of one product: a norm over near-ties and values near zero)
            limit, limit_row = limit * 10, limit_row * 10
        assert np.sqrt(np.mean(err ** 2)) < limit and err.max() < limit_row, (name, keep, prec, chunk, err.max(), np.sqrt(np.mean(err ** 2)))
        ses.close()
    st.close()


@BOTH
@pytest.mark.parametrize("name", sorted(N.CONFIGS))
def test_whole_prompt_portions_and_decoding(tmp_path, name, prec):
    cfg, w, folder, orc = made(tmp_path, name)
    T = 128
    t = prompt(cfg, T, 2)
    want = orc.forward(t)
    st = open_stage(folder, prec)
    limit = 8 if name == "ones" else 1
    cuts = {"whole": [T], "halves": [64, 64], "twos": [2] * 20 + [88], "chunk edges": [31, 2, 32, 33, 30], "uneven": [17, 2, 33, 3, 64, 2, 5, 1, 1], "one by one": [1] * T,
            "decoded": [100] + [1] * 28}
    for how, portions in cuts.items():
        e = off(run(st, t, portions), want, prec)
        assert e < limit, (name, prec, how, e)
    for how in ("whole", "chunk edges", "uneven"):           # short portions over projected keys and values as well
        e = off(run(st, t, cuts[how], latent_chunk_min_tokens=2), want, prec)
        assert e < limit, (name, prec, how, "chunk", e)
    # the same decoding through the many-token launches, and through replayed graphs, also of short portions
    assert off(run(st, t, [100] + [1] * 28, step_fused=0), want, prec) < limit
    ses = st.session(graphs=1)
    for portions in ([40] + [1] * 88, [68] + [2] * 10 + [4] * 10):
        assert off(run(st, t, portions, session=ses), want, prec) < limit
        assert np.array_equal(run(st, t, portions, session=ses), run(st, t, portions))
    assert ses.graph_replays >= 100
    ses.close()
    st.close()


@BOTH
def test_long_prompt_takes_every_kernel(tmp_path, prec):
    """Lengths around the large tile and the chunk kernels' steps, portions behind a long past, rows at both ends."""
    cfg = N.config(300, 192, [N.latent(6, 40, 24, 50, 72, 80, scaling=(2.0, 300, 32.0, 1.0), ff=200), N.delta(4, 2, 48, 32, 4, ff=264), N.gla(3, 36, 48, 8.0),
                              N.latent(4, 96, 24, 100, 72, 40, scaling=(2.0, 300, 32.0, 1.0), kv_from=0)], residual=0.9, logit=3.0)
    cfg, w, folder, orc = made(tmp_path, cfg)
    st = open_stage(folder, prec, n_ctx=1024, batch=1024)
    t = prompt(cfg, 900, 8)
    want = orc.forward(t)
    rows = sorted({0, 1, 30, 31, 32, 33, 63, 64, 127, 128, 129, 255, 256, 511, 512, 640, 899})
    for portions in ([900], [128, 129, 643], [895, 5], [127, 33, 740], [700, 64, 130, 2, 4]):
        s = Seq(st, st.session())
        got, at = [], 0
        for p in portions:
            got.append(s.feed(t[at:at + p], want=np.isin(np.arange(at, at + p), rows)))
            at += p
        s.ses.close()
        e = off(np.concatenate(got), want[rows], prec)
        assert e < 1, (portions, prec, e)
    st.close()
    # a session whose calls are shorter than the context projects keys and values in several blocks
    st = open_stage(folder, prec, n_ctx=1024, batch=200)
    assert off(run(st, t, [200, 200, 200, 150, 150], last=100), want[-100:], prec) < 1
    st.close()


@BOTH
@pytest.mark.parametrize("width", [1032, 3000, 4100, 8300, 1031])
def test_widths_of_every_norm_kernel(tmp_path, width, prec):
    """Rows of one to several groups of a thread, longer than its registers hold, and of a length that is no multiple of four."""
    cfg = N.config(140, width, [N.latent(2, 16, 8, 16, 32, 24, ff=72), N.gla(1, 16, 24, 4.0)], residual=0.5)
    cfg, w, folder, orc = made(tmp_path, cfg)
    st = open_stage(folder, prec, n_ctx=256, batch=256)
    t = prompt(cfg, 150, 8)
    want = orc.forward(t)[-20:]
    for portions in ([150], [130] + [1] * 20):
        e = off(run(st, t, portions, last=20), want, prec)
        assert e < 1, (portions, prec, e)
    st.close()


# ------------------------------------------------------------------------------------------------ far tokens
@BOTH
@pytest.mark.parametrize("layers", [[N.latent(2, 16, 8, 16, 24, 20)], [N.latent(5, 40, 24, 64, 100, 60)], [N.latent(3, 100, 64, 90, 512, 40)], [N.latent(2, 200, 8, 30, 90, 40)],
                                    [N.latent(2, 16, 8, 16, 24, 20), N.latent(18, 24, 8, 20, 24, 30, kv_from=0)]])
def test_a_far_key_shows_from_every_place(tmp_path, layers, prec):
    """One key stands out for the last token, at the sequence's start, at edges of the kernels' steps and splits, just behind; the
    asking token ends a prompt, ends a portion of two, or is decoded alone."""
    needle, asker = 7, 9
    cfg, w, folder, orc = made(tmp_path, N.config(60, 128, layers), change=lambda w, c: N.needle_weights(c, 5, needle, asker))
    st = open_stage(folder, prec, n_ctx=512)
    ses, projected = st.session(), st.session(latent_chunk_min_tokens=2)
    for end, places in ((34, (0, 1, 30, 31, 32)), (200, (0, 1, 31, 32, 63, 64, 127, 128, 160, 197, 198))):
        for at in places:
            t = prompt(cfg, end, 40 + at, avoid=(needle, asker))
            t[end - 1], t[at] = asker, needle
            orc.reset()
            want = orc.forward(t)[-1:]
            for portions in ([end], [end - 2, 2], [end - 1, 1]):
                for s in (ses, projected):
                    e = off(run(st, t, portions, session=s, last=1), want, prec)
                    assert e < 2, (end, at, portions, s is projected, e)
    ses.close(), projected.close()
    st.close()


def slow(w, cfg):
    """States that hardly forget, and a token whose writes are large."""
    for i, l in enumerate(cfg["layers"]):
        p = "l%d.mix." % i
        if l["type"] == "delta":
            w[p + "A_log"] = np.full_like(w[p + "A_log"], -6.0)
        elif l["type"] == "gla":
            w[p + "a2.b"] = np.full_like(w[p + "a2.b"], 12.0)
    return w


@BOTH
def test_far_token_reaches_through_the_state(tmp_path, prec):
    """Changing one token 300 back changes the last logits as the oracle says."""
    cfg, w, folder, orc = made(tmp_path, "states-only", change=slow)
    t = prompt(cfg, 330, 3)
    u = t.copy()
    u[20:24] = (u[20:24] + 5) % cfg["vocab"]
    a = orc.forward(t)[-4:]
    orc.reset()
    b = orc.forward(u)[-4:]
    assert error(a, b) > 4 * LIMIT["f32"]
    st = open_stage(folder, prec)
    for tok, want in ((t, a), (u, b)):
        for portions in ([165, 165], [256, 70, 1, 1, 1, 1], [21, 2, 200, 100, 7]):
            assert off(run(st, tok, portions, last=4), want, prec) < 1
    st.close()


@BOTH
def test_states_that_forget_at_once_stay_finite(tmp_path, prec):
    """Decays far below what a quotient of products over a chunk could hold, next to some that keep everything."""
    def change(w, cfg):
        rng = np.random.Generator(np.random.PCG64(9))
        for i, l in enumerate(cfg["layers"]):
            p = "l%d.mix." % i
            if l["type"] == "delta":
                w[p + "A_log"] = np.linspace(-8.0, 5.0, len(w[p + "A_log"]))
            else:
                w[p + "a2.b"] = N.bf16(rng.choice([-60.0, -5.0, 0.0, 30.0], len(w[p + "a2.b"])))
        return {k: N.bf16(v).reshape(np.shape(v)) for k, v in w.items()}
    cfg, w, folder, orc = made(tmp_path, N.config(64, 64, [N.delta(4, 2, 16, 24, 4, ff=64), N.gla(2, 32, 16, 0.25), N.gla(2, 20, 16, 1.0)]), change=change)
    t = prompt(cfg, 100, 3)
    want = orc.forward(t)
    st = open_stage(folder, prec)
    for portions in ([100], [40, 60], [33] + [1] * 67):
        e = off(run(st, t, portions), want, prec)
        assert e < 2, (portions, e)
    st.close()


# ------------------------------------------------------------------------------------------------ sequences
@BOTH
def test_unequal_requests_in_one_call_equal_each_alone(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec, n_seq=4, batch=256)
    lens = [70, 3, 41, 1]
    toks = [prompt(cfg, n + 40, 20 + i) for i, n in enumerate(lens)]
    want = []
    for t in toks:
        orc.reset()
        want.append(orc.forward(t))
    ses = st.session()
    order = [2, 0, 3, 1]
    at = [0] * 4

    def call(counts):
        ids, pos, seq, rows = [], [], [], []
        for q in order:
            n = counts[q]
            ids += list(toks[q][at[q]:at[q] + n])
            pos += list(range(at[q], at[q] + n))
            seq += [q] * n
            rows.append(want[q][at[q]:at[q] + n])
            at[q] += n
        got = ses.decode(np.array(ids, np.int32), pos, seq=seq, in_fmt=m.TOKENS, out_fmt=m.LOGITS).view(np.float32).reshape(len(ids), -1)
        assert off(got, np.concatenate(rows), prec) < 1, counts

    call(lens)                       # four prompts at once
    call([1, 1, 1, 1])               # a batch of decode steps
    call([2, 1, 5, 3])               # decode steps beside portions
    call([1, 0, 1, 0])
    call([33, 1, 2, 32])
    call([1, 1, 1, 1])
    ses.close()
    st.close()


@BOTH
def test_a_sequence_given_back_starts_clean(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec, n_seq=2)
    ses = st.session()
    a, b = prompt(cfg, 120, 1), prompt(cfg, 50, 2)
    want_b = orc.forward(b)
    run(st, a, [100, 1, 1, 18], session=ses, seq=1)
    ses.seq_reset(1)
    assert off(run(st, b, [40] + [1] * 10, session=ses, seq=1), want_b, prec) < 1
    for portions in ([1] * 50, [2] * 25, [50]):           # starting at position 0 again is enough, also with a token or two
        assert off(run(st, b, portions, session=ses, seq=1), want_b, prec) < 1
    assert off(run(st, b, [50], session=ses, seq=0), want_b, prec) < 1
    with pytest.raises(m.MeshError) as e:
        ses.decode(np.array([3], np.int32), [7], seq=[1], in_fmt=m.TOKENS, out_fmt=m.LOGITS)
    assert e.value.code == m.ERR_INVALID and "stands at 50 tokens" in e.value.message
    more = prompt(cfg, 5, 9)
    orc.reset()
    orc.forward(b)
    got = Seq(st, ses, 1)
    got.n = 50
    assert off(got.feed(more), orc.forward(more), prec) < 1
    ses.close()
    st.close()


@BOTH
def test_layer_ranges_joined_at_an_f32_boundary(tmp_path, prec):
    """A stage in the middle needs no token ids; a layer that reads an earlier layer's cache needs that layer in its stage."""
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    t = prompt(cfg, 60, 6)
    want = orc.forward(t)
    first, second = open_stage(folder, prec, 0, 4), open_stage(folder, prec, 4, 6)
    s1, s2 = first.session(), second.session()
    got, at = [], 0
    for n in (40, 1, 1, 2, 16):
        pos, ids = np.arange(at, at + n), t[at:at + n]
        h = s1.decode(ids, pos, in_fmt=m.TOKENS, out_fmt=m.F32)
        got.append(s2.decode(h, pos, in_fmt=m.F32, out_fmt=m.LOGITS).view(np.float32).reshape(n, -1))
        at += n
    assert off(np.concatenate(got), want, prec) < 1
    for x in (s1, s2, first, second):
        x.close()
    with pytest.raises(m.MeshError) as e:
        open_stage(folder, prec, 1, 6)
    assert e.value.code == m.ERR_UNSUPPORTED and "layer 3 reads the cache of layer 0" in e.value.message


@BOTH
def test_long_decoding(tmp_path, prec):
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec, n_ctx=512)
    t = prompt(cfg, 420, 12)
    want = orc.forward(t)
    assert off(run(st, t, [20] + [1] * 400), want, prec) < 1
    st.close()


def test_missing_or_misshapen_weights_are_refused(tmp_path):
    m = mesh()
    cfg = N.CONFIGS["mixed"]
    w = N.random_weights(cfg, 1)
    for name, shape in (("l0.mix.dkv", None), ("l2.mix.a1", None), ("l2.mix.a2", (78, 6)), ("l1.mix.q.conv", (40, 3)), ("l4.norm1.b", (135,)), ("l0.mix.uk", (120, 43))):
        bad = dict(w)
        if shape is None:
            del bad[name]
        else:
            bad[name] = np.zeros(shape, np.float32)
        with pytest.raises(m.MeshError) as e:
            open_stage(write_folder(str(tmp_path / "bad"), cfg, bad), "bf16")
        assert e.value.code == m.ERR_FORMAT and name in e.value.message


# ------------------------------------------------------------------------------------------------ generation
@BOTH
def test_greedy_generation_through_the_session(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec)
    ses = st.session()
    prompts = [prompt(cfg, n, 60 + n) for n in (30, 5, 18)]
    outs = [[] for _ in prompts]
    for q, p in enumerate(prompts):
        lg = Seq(st, ses, q).feed(p, want=[0] * (len(p) - 1) + [1])
        outs[q].append(int(lg[0].argmax()))
    for _ in range(24):              # all sequences in one call per step
        ids = np.array([o[-1] for o in outs], np.int32)
        pos = [len(p) + len(o) - 1 for p, o in zip(prompts, outs)]
        lg = ses.decode(ids, pos, seq=[0, 1, 2], in_fmt=m.TOKENS, out_fmt=m.LOGITS).view(np.float32).reshape(3, -1)
        for q in range(3):
            outs[q].append(int(lg[q].argmax()))
    for p, o in zip(prompts, outs):
        check_greedy(orc, p, o, 1e-3 if prec == "f32" else 1.0)
    ses.close()
    st.close()


def test_greedy_generation_through_the_plugin_endpoint(tmp_path):
    from plugin_host import PB, PluginHost
    cfg, w, folder, orc = made(tmp_path, "mixed")
    host = PluginHost(os.path.join(ROOT, "mesh-llm_amd", "mesh-stage-plugin"), ["--model", folder, "--precision", "f32", "-c", "128", "--batch", "64"], tmp_path, name="latent")
    info = json.loads(host.initialize().initialize_response.server_info_json)
    assert info["arch"] == "Nutavik" and info["stage_open"] is True
    env = host.request(initialize_request=PB["InitializeRequest"](host_protocol_version=2, host_version="t", host_info_json="{}", mesh_visibility=1))
    address = env.initialize_response.manifest.endpoints[0].address

    def post(ids, pos0):
        req = urllib.request.Request(address + "/stage/decode", data=np.asarray(ids, np.int32).tobytes(), method="POST",
                                     headers={"X-Mesh-Tokens": str(len(ids)), "X-Mesh-Pos0": str(pos0), "X-Mesh-In-Format": "tokens", "X-Mesh-Out-Format": "logits",
                                              "X-Mesh-Want": str(len(ids) - 1)})
        with urllib.request.urlopen(req, timeout=60) as r:
            return np.frombuffer(r.read(), np.float32)

    p = prompt(cfg, 39, 77)
    out = [int(post(p, 0).argmax())]
    for i in range(15):
        out.append(int(post(out[-1:], len(p) + i).argmax()))
    check_greedy(orc, p, out, 1e-3)
    host.request(shutdown_request=PB["ShutdownRequest"](reason="done"))
    host.close()


@BOTH
def test_trace_runner(tmp_path, prec):
    cfg, w, folder, orc = made(tmp_path, "mixed")
    out = tmp_path / "out"
    out.mkdir()
    a, b = prompt(cfg, 45, 1), prompt(cfg, 9, 2)
    steps = [("a", a[:30], [3, 29], []), ("a", a[30:32], [], []), ("a", a[32:33], [0], []), ("a", a[33:], [11, 0], ["a"]), ("b", b, [8], ["b"]), ("a", b[:4], [3], ["a"])]
    lines = [json.dumps({"step": i, "entries": [{"id": e, "tokens": [int(v) for v in t], "want": wn}], "end": end}) for i, (e, t, wn, end) in enumerate(steps)]
    r = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32" if prec == "f32" else "bfloat16", "--out", str(out), "--max-tokens", "64"],
                       input="\n".join(lines) + "\n", capture_output=True, text=True, timeout=100)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done %d" % i for i in range(len(steps))]
    wa = orc.forward(a)
    orc.reset()
    wb = orc.forward(b)
    for step, want in ((0, wa[[3, 29]]), (2, wa[[32]]), (3, wa[[44, 33]]), (4, wb[[8]]), (5, wb[[3]])):
        got = np.fromfile(str(out / ("%d.f32" % step)), "<f4").reshape(len(want), -1)
        assert off(got, want, prec) < 1, step
