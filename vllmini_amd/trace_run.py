"""Replays a trace of token ids through a model, step by step, and writes logits (bin/trace_run).

Steps come from standard input, one JSON object a line:

    {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": ["b"]}

Every entry brings the next tokens of a sequence (a whole prompt, a portion, one token); all entries of a step are one batch
of the decoder's own step().  `want` are the places among the tokens whose logits are written to OUT/<step>.f32 (little-endian
float32, [wanted, vocabulary]); sequences named in `end` give back their pages and state slots after the step.  "done <step>" is
printed after each.  Nothing is sampled.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

MAX_LIVE = 4      # state slots; a trace keeps at most that many sequences alive


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="trace_run", description=__doc__.split("\n\n")[0])
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors")
    ap.add_argument("--dtype", required=True, choices=("bfloat16", "float32"))
    ap.add_argument("--out", required=True, help="folder the logits are written to")
    ap.add_argument("--max-tokens", required=True, type=int,
                    help="the most tokens live sequences hold at any time, each count rounded up to whole pages")
    a = ap.parse_args(argv)

    from . import build
    build.build_hybrid()          # (compiles what is missing or older than its sources; nothing otherwise)
    from .registry import UnsupportedDtype, load_decoder
    try:
        dec = load_decoder(a.model, dtype=a.dtype, max_tokens=a.max_tokens, max_seqs=MAX_LIVE)
    except UnsupportedDtype as e:
        print(e, file=sys.stderr)
        return 3
    if not hasattr(dec, "step"):
        print("this model's decoder takes whole prompts and single tokens only: it cannot replay portions", file=sys.stderr)
        return 2
    live = {}
    fresh = 0
    for line in sys.stdin:
        if not line.strip():
            continue
        s = json.loads(line)
        ids, tokens, want = [], [], []
        for e in s["entries"]:
            if e["id"] not in live:
                live[e["id"]] = fresh
                dec.pool.open(fresh)
                fresh += 1
            ids.append(live[e["id"]])
            tokens.append(e["tokens"])
            want.append(e["want"])
        logits = dec.step(ids, tokens, want) if ids else None
        if logits is not None:
            data = logits.float().cpu().numpy().astype("<f4").tobytes()
            part = os.path.join(a.out, f".{s['step']}.part")
            with open(part, "wb") as f:
                f.write(data)
            os.replace(part, os.path.join(a.out, f"{s['step']}.f32"))
        for name in s.get("end", ()):
            dec.pool.free(live.pop(name))
        print(f"done {s['step']}", flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
