"""Replays a trace of token ids through a model and writes the logits it asks for: `bin/trace_run`.

Steps come as JSON lines on standard input,
    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}
and run through the library's own stage and session (mesh_stage_decode): a request takes one of the session's sequences,
its tokens go on where it stands, and `end` gives the sequence back.  A step in which something is wanted leaves
<out>/<step>.f32, the logits as little-endian f32 [wanted, vocab] in the order of the entries and of `want`; "done <step>"
is printed after every step.
"""
import argparse
import json
import os
import sys

import numpy as np

BATCH_MAX = 2048        # tokens per library call; a longer portion is fed in several


class Replayer:
    def __init__(self, mesh, model, precision, max_tokens, sequences=8):
        self.mesh = mesh
        n_ctx = max(int(max_tokens), 1)
        self.batch_max = min(BATCH_MAX, n_ctx)
        self.stage = mesh.Stage(model, 0, -1, n_ctx=n_ctx, n_seq_max=sequences, n_batch_max=self.batch_max, precision=precision)
        self.session = self.stage.session()
        self.vocab = int(self.stage.info.n_vocab)
        self.free = list(range(sequences))[::-1]
        self.live = {}          # request id -> [sequence, tokens fed]

    def _portions(self, tokens, want):
        """(begin, end) runs of at most batch_max tokens and as many wanted rows as one call returns."""
        flags = np.zeros(len(tokens), np.uint8)
        flags[want] = 1
        begin = 0
        while begin < len(tokens):
            end = min(begin + self.batch_max, len(tokens))
            over = np.flatnonzero(np.cumsum(flags[begin:end]) > self.mesh.LOGITS_TOKENS_MAX)
            if over.size:
                end = begin + int(over[0])
            yield begin, end, flags[begin:end]
            begin = end

    def feed(self, request, tokens, want):
        """Runs the tokens and returns the logits at the places `want` (in its order) among them."""
        if request not in self.live:
            if not self.free:
                raise RuntimeError("more than %d live requests" % self.stage_sequences)
            self.live[request] = [self.free.pop(), 0]
        entry = self.live[request]
        tokens = np.asarray(tokens, np.int32)
        rows = {}
        for begin, end, flags in self._portions(tokens, want):
            pos = np.arange(entry[1], entry[1] + end - begin, dtype=np.int32)
            out = self.session.decode(tokens[begin:end], pos, seq=np.full(end - begin, entry[0], np.int32), in_fmt=self.mesh.TOKENS, out_fmt=self.mesh.LOGITS, want=flags)
            entry[1] += end - begin
            got = out.view(np.float32).reshape(-1, self.vocab)
            for i, place in enumerate(np.flatnonzero(flags)):
                rows[begin + int(place)] = got[i]
        return [rows[w] for w in want]

    @property
    def stage_sequences(self):
        return len(self.free) + len(self.live)

    def end(self, request):
        if request in self.live:
            seq = self.live.pop(request)[0]
            self.session.seq_reset(seq)
            self.free.append(seq)

    def close(self):
        self.session.close()
        self.stage.close()


def main(argv=None, mesh=None):
    ap = argparse.ArgumentParser(prog="trace_run", description="Feed a trace of token ids through a model and write the logits it asks for.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors, or a GGUF file")
    ap.add_argument("--dtype", required=True, choices=["bfloat16", "float32"], help="the served precision, or everything in 32 bits")
    ap.add_argument("--out", required=True, help="folder for <step>.f32")
    ap.add_argument("--max-tokens", required=True, type=int, help="the most tokens live requests hold at any time")
    a = ap.parse_args(argv)
    replay = Replayer(mesh, a.model, mesh.PRECISION_F32 if a.dtype == "float32" else mesh.PRECISION_DEFAULT, a.max_tokens)
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = []
        for e in step["entries"]:
            rows += replay.feed(e["id"], e["tokens"], e.get("want", []))
        if rows:
            np.stack(rows).astype("<f4").tofile(os.path.join(a.out, "%d.f32" % step["step"]))
        for request in step.get("end", []):
            replay.end(request)
        print("done %d" % step["step"], flush=True)
    replay.close()
    return 0
