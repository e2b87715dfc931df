"""Nadosun on the GPU against the plain oracle: each mechanism alone, whole prompts against portions and token-by-token
decoding, sequences side by side and reused, window edges that show, layer ranges, greedy generation through the stage
and through the plugin's endpoint, and the trace runner."""
import json
import os
import subprocess
import sys
import urllib.request

import numpy as np
import pytest

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
import nadosun_util as N
from folder_util import Seq, check_greedy, open_stage, run
from oracle.nadosun import NadosunOracle
from util import ROOT, mesh

pytestmark = pytest.mark.gpu

LIMIT = {"bf16": 2e-2, "f32": 3e-5}        # rms of a row's difference over the rms of all rows (nadosun_util.error)
BOTH = pytest.mark.parametrize("prec", ["bf16", "f32"])
_made = {}


def made(tmp, name, seed=11, change=None, key=None):
    """(config, weights, folder, oracle) of a named configuration; `change` rewrites the weights."""
    cfg = N.CONFIGS[name] if isinstance(name, str) else name
    w = N.random_weights(cfg, seed)
    if change:
        w = change(w, cfg)
    return cfg, w, N.write_folder(str(tmp / "model"), cfg, w), NadosunOracle(cfg, w)


# ------------------------------------------------------------------------------------------------ mechanisms
@BOTH
@pytest.mark.parametrize("keep", ["", "mixer", "ff", "side"])
@pytest.mark.parametrize("name", ["mixed", "wide-heads", "odd-shapes", "ones"])
def test_each_mechanism_alone(tmp_path, name, keep, prec):
    """The residual stream after the last layer with every other addition scaled to nothing: the embedding with its position
    vector (""), the mixers, the feed-forwards, the per-token side input; many tokens and one."""
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, name, change=lambda w, c: N.only(w, c, keep))
    t = N.prompt(cfg, 90, 5)
    orc.forward(t)
    want = orc.layers[-1]
    st = open_stage(folder, prec)
    ses = st.session()
    s = Seq(st, ses)
    got = np.concatenate([s.feed(t[:70], out=m.F32)] + [s.feed(t[i:i + 1], out=m.F32) for i in range(70, 90)])
    # (a bf16 row whose vector is small before its output norm is rounded more coarsely than the rest)
    limit, limit_row = (2e-6, 2e-6) if keep == "" else (1e-5, 3e-5) if prec == "f32" else (1e-2, 6e-2)
    assert np.isfinite(got).all()
    # against what the mechanism adds, not against the embedding under it
    base = NadosunOracle(cfg, N.only(w, cfg, ""))
    base.forward(t)
    added = np.sqrt(np.mean((want - base.layers[-1]) ** 2)) if keep else np.sqrt(np.mean(want ** 2))
    err = np.sqrt(np.mean((got - want) ** 2, axis=-1)) / max(added, 1e-3)
    assert np.sqrt(np.mean(err ** 2)) < limit and err.max() < limit_row, (name, keep, prec, err.max())
    ses.close()
    st.close()


@BOTH
@pytest.mark.parametrize("name", sorted(N.CONFIGS))
def test_whole_prompt_portions_and_decoding(tmp_path, name, prec):
    cfg, w, folder, orc = made(tmp_path, name)
    T = 128
    t = N.prompt(cfg, T, 2)
    want = orc.forward(t)
    st = open_stage(folder, prec)
    # (vectors of one element before a norm: bf16 rounding alone moves single rows further)
    limit = LIMIT[prec] * (4 if name == "ones" else 1)
    cuts = {"whole": [T], "halves": [64, 64], "twos": [2] * 20 + [88], "uneven": [17, 2, 33, 3, 64, 2, 5, 1, 1], "one by one": [1] * T, "decoded": [100] + [1] * 28}
    for how, portions in cuts.items():
        e = N.error(run(st, t, portions), want)
        assert e < limit, (name, prec, how, e)
    # the same decoding through the many-token launches, and through replayed graphs
    assert N.error(run(st, t, [100] + [1] * 28, step_fused=0), want) < limit
    ses = st.session(graphs=1)
    assert np.array_equal(run(st, t, [100] + [1] * 28, session=ses), run(st, t, [100] + [1] * 28)) and ses.graph_replays >= 20
    ses.close()
    st.close()


@BOTH
def test_long_prompt_takes_every_kernel(tmp_path, prec):
    """Lengths around the large tile and the chunk kernel's steps, rows at both ends and around window edges."""
    cfg = N.config(300, 192, 24, [N.attention(6, 3, 64, 100, ff=200), N.mingru(160), N.attention(4, 2, 128, 257, scale=0.12), N.mingru(128, ff=264)], scale=0.5)
    cfg, w, folder, orc = made(tmp_path, cfg)
    st = open_stage(folder, prec, n_ctx=1024, batch=1024)
    t = N.prompt(cfg, 900, 8)
    want = orc.forward(t)
    rows = sorted({0, 1, 31, 32, 63, 64, 99, 100, 101, 127, 128, 255, 256, 257, 258, 511, 512, 640, 899})
    for portions in ([900], [128, 129, 643], [895, 5], [127, 33, 740]):
        s = Seq(st, st.session())
        got, at = [], 0
        for p in portions:
            flags = np.isin(np.arange(at, at + p), rows)
            got.append(s.feed(t[at:at + p], want=flags))
            at += p
        s.ses.close()
        e = N.error(np.concatenate(got), want[rows])
        assert e < LIMIT[prec], (portions, prec, e)
    st.close()


@BOTH
def test_layers_wide_enough_for_several_tiles_and_slices(tmp_path, prec):
    """Products whose K spans several batches of a wave, whose rows take more than one per turn, and a side gate cut along K;
    lengths are no multiple of anything."""
    cfg = N.config(4500, 1032, 40, [N.attention(8, 2, 128, 50, ff=4200), N.mingru(1100)], scale=0.6)
    cfg, w, folder, orc = made(tmp_path, cfg)
    st = open_stage(folder, prec, n_ctx=512, batch=512)
    t = N.prompt(cfg, 303, 8)
    want = orc.forward(t)[-20:]
    for portions in ([303], [150, 150, 1, 1, 1], [290] + [1] * 13):
        e = N.error(run(st, t, portions, last=20), want)
        assert e < LIMIT[prec], (portions, prec, e)
    st.close()


@BOTH
def test_far_token_reaches_through_the_state(tmp_path, prec):
    """A recurrence that hardly forgets: changing one token 300 back changes the last logits as the oracle says."""
    def slow(w, cfg):
        for i, l in enumerate(cfg["layers"]):
            if l["type"] == "mingru":
                w["l%d.mix.z.b" % i] = N.bf16(np.full_like(w["l%d.mix.z.b" % i], -6.0))
        w["embed"] = w["embed"].copy()
        w["embed"][5] = N.bf16(w["embed"][5] * 30)
        return w
    cfg, w, folder, orc = made(tmp_path, "recurrent-only", change=slow)
    t = N.prompt(cfg, 330, 3, avoid=(5,))
    u = t.copy()
    u[20] = 5
    a = orc.forward(t)[-4:]
    orc.reset()
    b = orc.forward(u)[-4:]
    assert N.error(a, b) > 3 * LIMIT["bf16"]
    st = open_stage(folder, prec)
    for tok, want in ((t, a), (u, b)):
        for portions in ([165, 165], [256, 70, 1, 1, 1, 1], [21, 2, 200, 100, 7]):
            assert N.error(run(st, tok, portions, last=4), want) < LIMIT[prec]
    st.close()


# ------------------------------------------------------------------------------------------------ windows
@BOTH
@pytest.mark.parametrize("heads,kv,dim,window", [(4, 2, 64, 33), (2, 1, 32, 64), (8, 1, 128, 65), (3, 1, 160, 40), (20, 1, 16, 21), (1, 1, 96, 2), (2, 2, 64, 1)])
def test_keys_just_inside_and_outside_the_window(tmp_path, heads, kv, dim, window, prec):
    """One key stands out for the last token; at distances around the window it is seen or not, whether the asking token ends a
    prompt, ends a portion of two, or is decoded alone, and wherever it lies against the kernels' steps."""
    needle, asker = 7, 9
    cfg = N.config(60, 128, 4, [N.attention(heads, kv, dim, window, scale=24.0 / dim)])
    cfg, w, folder, orc = made(tmp_path, cfg, change=lambda w, c: N.needle_weights(c, 5, needle, asker, 60.0))
    st = open_stage(folder, prec)
    ses = st.session()
    for end in (window + 1, 96, 130, 131):
        for dist in sorted({0, 1, window - 2, window - 1, window, window + 1}):
            if dist < 0 or dist > end - 1 or (dist == 0 and needle == asker):
                continue
            t = N.prompt(cfg, end, 40 + dist, avoid=(needle, asker))
            t[end - 1] = asker
            if dist:
                t[end - 1 - dist] = needle
            orc.reset()
            want = orc.forward(t)[-1:]
            for portions in ([end], [end - 2, 2], [end - 1, 1]):
                if min(portions) < 1:
                    continue
                got = run(st, t, portions, session=ses, last=1)
                e = N.error(got, want)
                assert e < LIMIT[prec], (end, dist, portions, e)
    ses.close()
    st.close()


# ------------------------------------------------------------------------------------------------ sequences
@BOTH
def test_unequal_requests_in_one_call_equal_each_alone(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec, n_seq=4, batch=256)
    lens = [70, 3, 41, 1]
    toks = [N.prompt(cfg, n + 12, 20 + i) for i, n in enumerate(lens)]
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
        assert N.error(got, np.concatenate(rows)) < LIMIT[prec], counts

    call(lens)                       # four prompts at once
    call([1, 1, 1, 1])               # a batch of decode steps
    call([2, 1, 5, 3])               # decode steps beside portions
    call([1, 0, 1, 0])
    call([1, 1, 1, 1])
    ses.close()
    st.close()


@BOTH
def test_a_sequence_given_back_starts_clean(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec, n_seq=2)
    ses = st.session()
    a, b = N.prompt(cfg, 120, 1), N.prompt(cfg, 50, 2)
    want_b = orc.forward(b)
    run(st, a, [100, 1, 1, 18], session=ses, seq=1)
    ses.seq_reset(1)
    assert N.error(run(st, b, [40] + [1] * 10, session=ses, seq=1), want_b) < LIMIT[prec]
    # starting at position 0 again is enough, also with a single token
    assert N.error(run(st, b, [1] * 50, session=ses, seq=1), want_b) < LIMIT[prec]
    # sequence 0 is untouched by all that
    assert N.error(run(st, b, [50], session=ses, seq=0), want_b) < LIMIT[prec]
    # going on where a sequence does not stand is refused, and changes nothing
    with pytest.raises(m.MeshError) as e:
        ses.decode(np.array([3], np.int32), [7], seq=[1], in_fmt=m.TOKENS, out_fmt=m.LOGITS)
    assert e.value.code == m.ERR_INVALID and "stands at 50 tokens" in e.value.message
    for pos, seq in (([50, 52], [1, 1]), ([50, 50, 51], [1, 0, 1])):
        with pytest.raises(m.MeshError) as e:
            ses.decode(np.arange(len(pos), dtype=np.int32), pos, seq=seq, in_fmt=m.TOKENS, out_fmt=m.LOGITS)
        assert e.value.code == m.ERR_INVALID
    with pytest.raises(m.MeshError):
        ses.decode(np.array([cfg["vocab"]], np.int32), [50], seq=[1], in_fmt=m.TOKENS, out_fmt=m.LOGITS)
    more = N.prompt(cfg, 5, 9)
    orc.reset()
    orc.forward(b)
    got = Seq(st, ses, 1)
    got.n = 50
    assert N.error(got.feed(more), orc.forward(more)) < LIMIT[prec]
    ses.close()
    st.close()


def test_wanted_rows_only(tmp_path):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, "bf16")
    t = N.prompt(cfg, 60, 4)
    full = run(st, t, [60])
    s = Seq(st, st.session())
    flags = np.zeros(40, np.uint8)
    flags[[0, 17, 39]] = 1
    assert np.allclose(s.feed(t[:40], want=flags), full[[0, 17, 39]], atol=2e-2)
    assert s.feed(t[40:41], want=[0]).size == 0 and s.feed(t[41:45], want=[0] * 4).size == 0
    assert np.allclose(s.feed(t[45:60], want=[0] * 14 + [1]), full[59:], atol=6e-2)
    s.ses.close()
    st.close()
    # the K-quant models return the same rows
    import models
    g = str(tmp_path / "tiny.gguf")
    lc = models.CONFIGS["tiny-llama"]
    models.write_model(g, lc, range(lc["n_layer"]), seed=3, with_embd=True, with_output=True)
    st = m.Stage(g, 0, -1, n_ctx=64, n_batch_max=32)
    a, b = st.session(), st.session()
    ids = (np.arange(9) % 50).astype(np.int32)
    whole = a.decode(ids, np.arange(9), in_fmt=m.TOKENS, out_fmt=m.LOGITS).view(np.float32).reshape(9, -1)
    some = b.decode(ids, np.arange(9), in_fmt=m.TOKENS, out_fmt=m.LOGITS, want=[0, 1, 0, 0, 0, 0, 0, 0, 1]).view(np.float32).reshape(2, -1)
    assert np.allclose(some, whole[[1, 8]], rtol=1e-4, atol=1e-4)
    assert b.decode(ids[:1], [9], in_fmt=m.TOKENS, out_fmt=m.LOGITS, want=[0]).size == 0
    a.close(), b.close(), st.close()


@BOTH
def test_layer_ranges_joined_at_an_f32_boundary(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    t = N.prompt(cfg, 60, 6)
    want = orc.forward(t)
    first, second = open_stage(folder, prec, 0, 2), open_stage(folder, prec, 2, 4)
    s1, s2 = first.session(), second.session()
    got, at = [], 0
    for n in (40, 1, 1, 2, 16):
        pos, ids = np.arange(at, at + n), t[at:at + n]
        h = s1.decode(ids, pos, in_fmt=m.TOKENS, out_fmt=m.F32)
        with pytest.raises(m.MeshError):
            s2.decode(h, pos, in_fmt=m.F32, out_fmt=m.LOGITS)            # its layers read the token ids
        got.append(s2.decode(h, pos, in_fmt=m.F32, out_fmt=m.LOGITS, token_ids=ids).view(np.float32).reshape(n, -1))
        at += n
    assert N.error(np.concatenate(got), want) < LIMIT[prec]
    for x in (s1, s2, first, second):
        x.close()


@BOTH
def test_long_decoding(tmp_path, prec):
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec, n_ctx=512)
    t = N.prompt(cfg, 420, 12)
    want = orc.forward(t)
    assert N.error(run(st, t, [20] + [1] * 400), want) < LIMIT[prec]
    st.close()


# ------------------------------------------------------------------------------------------------ generation
@BOTH
def test_greedy_generation_through_the_session(tmp_path, prec):
    m = mesh()
    cfg, w, folder, orc = made(tmp_path, "mixed")
    st = open_stage(folder, prec)
    ses = st.session()
    prompts = [N.prompt(cfg, n, 60 + n) for n in (30, 5, 18)]
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
        check_greedy(orc, p, o, 1e-4 if prec == "f32" else 0.15)
    ses.close()
    st.close()


def test_greedy_generation_through_the_plugin_endpoint(tmp_path):
    from plugin_host import PB, PluginHost
    cfg, w, folder, orc = made(tmp_path, "mixed")
    binary = os.path.join(ROOT, "mesh-llm_amd", "mesh-stage-plugin")
    host = PluginHost(binary, ["--model", folder + "/", "--precision", "f32", "-c", "128", "--batch", "64"], tmp_path, name="hybrid")
    info = json.loads(host.initialize().initialize_response.server_info_json)
    assert info["arch"] == "Nadosun" and info["model"] == "model" and info["stage_open"] is True
    env = host.request(initialize_request=PB["InitializeRequest"](host_protocol_version=2, host_version="t", host_info_json="{}", mesh_visibility=1))
    address = env.initialize_response.manifest.endpoints[0].address

    def post(ids, pos0):
        req = urllib.request.Request(address + "/stage/decode", data=np.asarray(ids, np.int32).tobytes(), method="POST",
                                     headers={"X-Mesh-Tokens": str(len(ids)), "X-Mesh-Pos0": str(pos0), "X-Mesh-In-Format": "tokens", "X-Mesh-Out-Format": "logits",
                                              "X-Mesh-Want": str(len(ids) - 1)})
        with urllib.request.urlopen(req, timeout=60) as r:
            return np.frombuffer(r.read(), np.float32)

    p = N.prompt(cfg, 21, 77)
    out = [int(post(p, 0).argmax())]
    for i in range(15):
        lg = post(out[-1:], len(p) + i)
        assert lg.size == cfg["vocab"]
        out.append(int(lg.argmax()))
    check_greedy(orc, p, out, 1e-4)
    with pytest.raises(urllib.error.HTTPError) as err:
        post([1], 90)                # not where the sequence stands
    assert err.value.code == 400
    host.request(shutdown_request=PB["ShutdownRequest"](reason="done"))
    host.close()


@BOTH
def test_trace_runner(tmp_path, prec):
    cfg, w, folder, orc = made(tmp_path, "mixed")
    out = tmp_path / "out"
    out.mkdir()
    a, b = N.prompt(cfg, 45, 1), N.prompt(cfg, 9, 2)
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
        assert N.error(got, want) < LIMIT[prec], step
    assert not (out / "1.f32").exists()
