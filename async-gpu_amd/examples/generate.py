#!/usr/bin/env python3
"""Generates with any model of the registry: a folder with config.json and model.safetensors, or a GPT-2 safetensors file.

    python generate.py MODEL --tokens 5,17,3 [--max-new-tokens 32] [--dtype bfloat16|float32] [--n-positions 1024] [--eos ID]
    python generate.py MODEL --vocab VOCAB --prompt "The capital of France is"
    ... --top-k 40 --temperature 0.8 --seed 42        samples instead of taking the best token

Prints the token ids, prompt included, separated by commas (with --vocab: the decoded text first).
"""
import argparse
import os
import sys

sys.path.insert(0, os.path.dirname(os.path.abspath(__file__)))
from gpt2_inference import load_package  # noqa: E402


def main(argv=None):
    ap = argparse.ArgumentParser(description=__doc__, formatter_class=argparse.RawDescriptionHelpFormatter)
    ap.add_argument("model")
    ap.add_argument("--tokens", help="prompt as token ids")
    ap.add_argument("--prompt", help="prompt as text (needs --vocab)")
    ap.add_argument("--vocab", help="tokenizer table: r50k_base.tiktoken or encoder.json")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--dtype", choices=("bfloat16", "float32"), default="bfloat16")
    ap.add_argument("--n-positions", type=int, default=None)
    ap.add_argument("--eos", type=int, default=None)
    ap.add_argument("--top-k", type=int, default=0)
    ap.add_argument("--temperature", type=float, default=1.0)
    ap.add_argument("--seed", type=int, default=0)
    a = ap.parse_args(argv)
    if (a.tokens is None) == (a.prompt is None) or (a.prompt is not None and a.vocab is None):
        ap.error("give --tokens, or --prompt with --vocab")
    load_package()
    import numpy as np
    from async_gpu_amd import models, ops, tokenizer
    tok = tokenizer.Gpt2Tokenizer.new(a.vocab) if a.vocab else None
    prompt = np.asarray([int(t) for t in a.tokens.split(",")] if a.tokens is not None else tok.encode(a.prompt), np.uint32)
    model = models.load_model(a.model, dtype=a.dtype, n_positions=a.n_positions)
    if a.top_k > 0:
        out = model.generate_cached_sampling(prompt, a.max_new_tokens, a.top_k, a.temperature, ops.SimpleRng(a.seed), eos=a.eos)
    else:
        (out,), (prefill_ms, decode_ms) = model.generate_cached(prompt, a.max_new_tokens, eos=a.eos)
        print(f"prefill {prefill_ms:.2f} ms, decode {decode_ms:.2f} ms", file=sys.stderr)
    if tok:
        print(tok.decode([int(t) for t in out]))
    print(",".join(str(int(t)) for t in out))
    model.close()
    return 0


if __name__ == "__main__":
    sys.exit(main())
