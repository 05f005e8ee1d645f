"""Command line: `python -m vllmini_amd generate --model DIR --prompt-ids 12,7,431 --max-new-tokens 32`.

generate   continuous-batching generation with any registered model (registry.py): every --prompt-ids is a request; prints one
           JSON line per request with its token ids (there is no tokenizer).
models     the architectures config.json may name.
"""
from __future__ import annotations

import argparse
import json
import sys


def _parser() -> argparse.ArgumentParser:
    ap = argparse.ArgumentParser(prog="python -m vllmini_amd", description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    sub = ap.add_subparsers(dest="command", required=True)
    sub.add_parser("models", help="list the architectures config.json may name")
    g = sub.add_parser("generate", help="generate from token-id prompts")
    g.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    g.add_argument("--dtype", default=None, help="element type (default: what the model is served in)")
    g.add_argument("--prompt-ids", action="append", required=True, metavar="ID,ID,...", help="a request; may be repeated")
    g.add_argument("--max-new-tokens", type=int, default=32)
    g.add_argument("--sampler", default="greedy", choices=("greedy", "top_k"))
    g.add_argument("--top-k", type=int, default=50)
    g.add_argument("--temperature", type=float, default=1.0)
    g.add_argument("--seed", type=int, default=0)
    g.add_argument("--max-tokens", type=int, default=0, help="tokens the pool holds (default: what the requests need)")
    g.add_argument("--max-batch", type=int, default=256)
    g.add_argument("--prefill-chunk", type=int, default=0, help="run prompts in portions of this many tokens beside the decode steps")
    g.add_argument("--graph", action="store_true", help="replay decode steps from a hipGraph")
    return ap


def generate(a) -> int:
    import torch

    from .registry import load_decoder
    from .scheduler import BatchScheduler, sample_top_k

    prompts = [[int(t) for t in p.split(",")] for p in a.prompt_ids]
    longest = max(len(p) for p in prompts) + a.max_new_tokens
    batch = min(a.max_batch, len(prompts))
    page = 64                                          # a multiple of every decoder's page
    need = sum(-(-(len(p) + a.max_new_tokens) // page) * page for p in prompts) + page
    dec = load_decoder(a.model, dtype=a.dtype, max_tokens=a.max_tokens or need, max_seqs=batch, max_length=longest)
    gen = torch.Generator(device=dec.device).manual_seed(a.seed)

    def sampler(logits, generator=None):
        return dec.greedy(logits) if a.sampler == "greedy" else sample_top_k(logits, a.top_k, a.temperature, generator=generator)

    eos = getattr(getattr(dec, "model", getattr(dec, "dims", None)), "eos_token_id", -1)
    sch = BatchScheduler(dec, max_length=longest, eos_token_id=eos, max_batch=batch, sampler=sampler, generator=gen,
                         use_graph=a.graph, prefill_chunk=a.prefill_chunk)
    ids = [sch.submit(p, max_new_tokens=a.max_new_tokens) for p in prompts]
    sch.run()
    for i, p in zip(ids, prompts):
        line = {"prompt": p, "generated": sch.sequences[i][len(p):]}
        if i in sch.rejected:
            line["rejected"] = sch.rejected[i]
        print(json.dumps(line))
    return 1 if sch.rejected else 0


def main(argv=None) -> int:
    a = _parser().parse_args(argv)
    if a.command == "models":
        from .registry import architectures
        print("\n".join(architectures()))
        return 0
    return generate(a)


if __name__ == "__main__":
    sys.exit(main())
