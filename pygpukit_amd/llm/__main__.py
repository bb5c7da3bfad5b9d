"""Command line of the LLM layer:  python -m pygpukit_amd.llm generate --model DIR --tokens 1,2,3 [--tokens 4,5] --max-new-tokens 16

Token ids in, token ids out (one line per prompt): tokenisers are outside this package.  All prompts run as one continuous batch on the
native engine where the model has one, otherwise one after another through the operator surface (GPT-2)."""

from __future__ import annotations

import argparse
import sys


def main(argv: list[str] | None = None) -> int:
    ap = argparse.ArgumentParser(prog="python -m pygpukit_amd.llm")
    sub = ap.add_subparsers(dest="cmd", required=True)
    g = sub.add_parser("generate", help="generate token ids from token ids")
    g.add_argument("--model", required=True, help="folder (or .safetensors file) of the checkpoint")
    g.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    g.add_argument("--tokens", action="append", required=True, help="comma-separated prompt ids; repeat for several prompts")
    g.add_argument("--max-new-tokens", type=int, default=16)
    g.add_argument("--max-batch", type=int, default=16, help="sequences resident at a time")
    g.add_argument("--temperature", type=float, default=0.0)
    g.add_argument("--top-k", type=int, default=0)
    g.add_argument("--top-p", type=float, default=1.0)
    g.add_argument("--eos", type=int, default=None)
    g.add_argument("--seed", type=int, default=None)
    a = ap.parse_args(argv)
    try:
        prompts = [[int(t) for t in p.split(",")] for p in a.tokens]
    except ValueError:
        ap.error("--tokens takes comma-separated integers")

    from pygpukit_amd.llm.loader import load_model_from_safetensors
    from pygpukit_amd.llm.scheduler import BatchScheduler

    model = load_model_from_safetensors(a.model, dtype=a.dtype)
    longest = max(len(p) for p in prompts) + a.max_new_tokens
    try:
        engine = model.build_engine(max_seq_len=longest, max_batch=min(a.max_batch, len(prompts)))
    except NotImplementedError:
        outs = [model.generate(p, a.max_new_tokens, a.temperature, a.top_k, a.top_p, a.eos) for p in prompts]
    else:
        outs = BatchScheduler(engine).generate(prompts, a.max_new_tokens, eos_token_id=a.eos, temperature=a.temperature, top_k=a.top_k,
                                               top_p=a.top_p, seed=a.seed)
    for o in outs:
        print(",".join(str(t) for t in o))
    return 0


if __name__ == "__main__":
    sys.exit(main())
