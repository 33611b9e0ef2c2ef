"""Command line: python3 moondream-zig_amd generate --model PATH --ids 1,2,3 --tokens 16 [--method top_k ...]

PATH is a model folder or a moondream.bin.  Token ids in, token ids out (the tokenizer is not part of this library)."""
import argparse
import importlib
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.dirname(os.path.abspath(__file__))))
moon = importlib.import_module(os.path.basename(os.path.dirname(os.path.abspath(__file__))))


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="moondream-zig_amd")
    sub = ap.add_subparsers(dest="command", required=True)
    sub.add_parser("designs", help="designs that a model folder may name")
    g = sub.add_parser("generate", help="continue a sequence of token ids")
    g.add_argument("--model", required=True, help="model folder or moondream.bin")
    g.add_argument("--dtype", choices=sorted(moon.text_model.DTYPES), help="element type of a model folder's decoder (default: bfloat16)")
    g.add_argument("--ids", required=True, help="prompt as comma-separated token ids")
    g.add_argument("--tokens", type=int, default=16)
    g.add_argument("--eos", type=int, help="end-of-sequence token id")
    g.add_argument("--max-seq", type=int, default=2048)
    g.add_argument("--method", choices=sorted(moon.sampling.METHODS), default="greedy")
    g.add_argument("--temperature", type=float, default=0.5)
    g.add_argument("--top-k", type=int, default=3)
    g.add_argument("--min-p", type=float, default=0.05)
    g.add_argument("--seed", type=int, default=0)
    a = ap.parse_args(argv)
    if a.command == "designs":
        print("\n".join(moon.registry.designs()))
        return 0
    import numpy as np

    model = moon.registry.open_text_model(a.model, a.dtype, a.max_seq)
    model.forward([int(t) for t in a.ids.split(",")])
    cfg = u = None
    if a.method != "greedy":
        cfg = moon.sampling.sampling_config(a.method, temperature=a.temperature, top_k=a.top_k, min_p=a.min_p)
        u = np.random.default_rng(a.seed).random(a.tokens).astype(np.float32)
    if a.eos is not None:
        out = model.generate(a.tokens, a.eos, cfg, u)
    else:
        out = model.greedy(a.tokens) if cfg is None else model.sample(cfg, u)
    print(",".join(str(t) for t in out))
    model.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
