"""Replays a trace of token ids through a model, step by step, and writes the logits it asks for.

    bin/trace_run --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

Steps arrive on standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

An entry feeds a request its next tokens through the request's session; the logits at the places in
"want" go to DIR/<step>.f32 (little-endian f32, [wanted, vocab], in the order of the entries), and a
line "done <step>" follows every step.  "end" names requests that are finished: their sessions are
reset and serve the requests that come next.
"""
import argparse
import json
import os
import sys

import numpy as np

DTYPES = {"bfloat16": "bf16", "float32": "f32"}


class SessionPool:
    """Sessions by request; a finished request's session is reset and handed on."""

    def __init__(self, model, max_ctx):
        self.model, self.max_ctx = model, max_ctx
        self.live, self.free = {}, []

    def get(self, request):
        if request not in self.live:
            self.live[request] = self.free.pop() if self.free else self.model.session(batch=1, max_ctx=self.max_ctx)
        return self.live[request]

    def end(self, request):
        s = self.live.pop(request, None)
        if s is not None:
            s.reset()
            self.free.append(s)


def run_entry(session, tokens, want):
    """Logits [len(want), vocab] of one entry: a single token behind a prompt is a decode step, anything
    else a prompt pass over the new tokens."""
    ids = np.asarray(tokens, dtype=np.uint64)
    if ids.size == 1 and session.position > 0:
        out = session.decode(ids)
        return out[[0] * len(want)]
    return session.feed(ids.reshape(1, -1), want)[0]


def run(model, out_dir, max_tokens, lines, echo):
    pool = SessionPool(model, max_tokens)
    for line in lines:
        if not line.strip():
            continue
        step = json.loads(line)
        rows = [run_entry(pool.get(e["id"]), e["tokens"], e.get("want", [])) for e in step["entries"] if e["tokens"]]
        rows = [r for r in rows if r.shape[0]]
        if rows:
            path = os.path.join(out_dir, f"{step['step']}.f32")
            np.concatenate(rows).astype("<f4").tofile(path)
        for request in step.get("end", []):
            pool.end(request)
        echo(f"done {step['step']}")


def main(argv=None):
    ap = argparse.ArgumentParser(description="Replay a trace of token ids and write the wanted logits.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=sorted(DTYPES))
    ap.add_argument("--out", required=True, help="folder that receives <step>.f32 files")
    ap.add_argument("--max-tokens", required=True, type=int, help="most tokens that live requests hold at any time")
    a = ap.parse_args(argv)
    if a.max_tokens < 1:
        ap.error("--max-tokens must be at least 1")

    from .build import ensure_built
    ensure_built()
    from .plugin import load_model
    model = load_model(a.model, weight_dtype=DTYPES[a.dtype], max_seq_len=a.max_tokens)
    run(model, a.out, a.max_tokens, sys.stdin, lambda text: print(text, flush=True))
    return 0


if __name__ == "__main__":
    sys.exit(main())
