"""Command line of the engine.

  python -m zipage_amd.cli generate --model DIR --tokens 5,17,3 [--tokens ...] --max-tokens 32
  python -m zipage_amd.cli trace --model DIR --dtype bfloat16|float32 --out DIR --max-tokens N

`generate` continues token prompts and prints one JSON line per prompt.  `trace` (also
`bin/trace_run`) replays given tokens: it reads steps from standard input, one JSON object a line,

  {"step": 0, "entries": [{"id": "a", "tokens": [5, 17, 3], "want": [0, 2]}], "end": []}

runs each as one batch, writes the fp32 logits at the wanted places to OUT/<step>.f32 and prints
"done <step>".  Both compile the model's kernels first if they are not built.
"""
from __future__ import annotations

import argparse
import json
import os
import sys

DTYPES = ("bfloat16", "float32")


def _engine(folder: str, dtype: str, pages: int, page_size: int, slots: int, **kw):
    from zipage_amd import build
    from zipage_amd.engine.registry import arch_for_shape, read_shape
    shape = read_shape(folder)
    arch = arch_for_shape(shape)
    build.ensure(*(getattr(build, lib) for lib in arch.libs))
    import torch
    from zipage_amd.engine import EngineConfig, ZipageEngine
    # without a limit of its own a model takes what the pool holds
    limit = getattr(shape, "max_positions", None) or getattr(shape, "max_position", pages * page_size)
    return ZipageEngine(EngineConfig(
        shape=shape, model_folder=folder if arch.loads_weights else None, dtype=getattr(torch, dtype),
        num_kvcache_blocks=pages, kvcache_block_size=page_size, max_concurrency=slots,
        max_model_len=limit, **kw))


def generate(args) -> int:
    prompts = [[int(t) for t in p.split(",")] for p in args.tokens]
    from zipage_amd.engine import SamplingParams
    per = max(len(p) for p in prompts) + args.max_tokens
    pages = args.pages or len(prompts) * (-(-per // args.page_size) + 1)
    eng = _engine(args.model, args.dtype, pages, args.page_size, max(1, min(len(prompts), args.slots)),
                  max_num_batched_tokens=args.batch_tokens, eos=args.eos, seed=args.seed,
                  enable_prefix_cache=args.prefix_cache)
    outs = eng.generate(prompts, SamplingParams(temperature=args.temperature, max_tokens=args.max_tokens,
                                                ignore_eos=args.eos < 0))
    for o in outs:
        print(json.dumps({"token_ids": o["token_ids"]}))
    return 0


def trace(args) -> int:
    size = 64
    eng = _engine(args.model, args.dtype, -(-args.max_tokens // size), size, 4)
    os.makedirs(args.out, exist_ok=True)
    live = {}
    for line in sys.stdin:
        if not line.strip():
            continue
        step = json.loads(line)
        entries = []
        for e in step["entries"]:
            if e["id"] not in live:
                live[e["id"]] = eng.open_request()
            entries.append((live[e["id"]], e["tokens"], e["want"]))
        logits = eng.feed(entries) if entries else None
        if logits is not None:
            path = os.path.join(args.out, f"{step['step']}.f32")
            logits.cpu().numpy().astype("<f4").tofile(path + ".part")
            os.replace(path + ".part", path)
        for name in step["end"]:
            eng.close_request(live.pop(name))
        print(f"done {step['step']}", flush=True)
    return 0


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="zipage_amd", description="Run a model of the engine's registry.")
    sub = ap.add_subparsers(dest="command", required=True)
    g = sub.add_parser("generate", help="continue token prompts")
    g.add_argument("--model", required=True, help="folder with config.json and safetensors weights")
    g.add_argument("--dtype", choices=DTYPES, default="bfloat16")
    g.add_argument("--tokens", action="append", required=True, metavar="ID,ID,...", help="one prompt; repeatable")
    g.add_argument("--max-tokens", type=int, default=32)
    g.add_argument("--temperature", type=float, default=0.0)
    g.add_argument("--eos", type=int, default=-1, help="token id that ends a sequence")
    g.add_argument("--seed", type=int, default=0)
    g.add_argument("--page-size", type=int, default=64)
    g.add_argument("--pages", type=int, default=0, help="pages of the cache pool (default: enough for all prompts)")
    g.add_argument("--slots", type=int, default=256, help="sequences resident at once")
    g.add_argument("--batch-tokens", type=int, default=32768, help="most tokens of one step")
    g.add_argument("--prefix-cache", action="store_true")
    g.set_defaults(run=generate)
    t = sub.add_parser("trace", help="replay given tokens and write logits")
    t.add_argument("--model", required=True)
    t.add_argument("--dtype", choices=DTYPES, required=True)
    t.add_argument("--out", required=True)
    t.add_argument("--max-tokens", type=int, required=True,
                   help="tokens of all live requests at once; sizes the cache pool")
    t.set_defaults(run=trace)
    args = ap.parse_args(argv)
    return args.run(args)


if __name__ == "__main__":
    sys.exit(main())
