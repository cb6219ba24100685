"""Generate token ids with a layered decoder: python -m pgmi --model DIR --prompt 5,17,3 [--prompt ...]

Prompts are token ids (these checkpoints come without a tokenizer); each is continued in one batch and its new
ids are printed on a line of their own.
"""
from __future__ import annotations

import argparse

import torch

from . import registry


def main() -> None:
    ap = argparse.ArgumentParser(prog="python -m pgmi", description="generate token ids with a layered decoder")
    ap.add_argument("--model", required=True, help="folder with config.json and *.safetensors")
    ap.add_argument("--prompt", action="append", required=True, help="token ids with commas between them")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--do-sample", action="store_true", help="temperature + top-p sampling instead of the argmax")
    ap.add_argument("--temperature", type=float, default=0.8)
    ap.add_argument("--top-p", type=float, default=0.9)
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--eos", type=int, default=None, help="token id that ends a sequence")
    a = ap.parse_args()
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt]
    eng = registry.load_decoder(a.model, dtype=a.dtype, max_batch=max(1, len(prompts)))
    gen = torch.Generator(device=eng.device).manual_seed(a.seed)
    toks, lens = eng.generate(prompts, a.max_new_tokens, do_sample=a.do_sample, temperature=a.temperature, top_p=a.top_p,
                              generator=gen, eos_token_id=a.eos, return_lengths=True)
    for row, n in zip(toks.tolist(), lens.tolist()):
        print(",".join(str(t) for t in row[:n]))


if __name__ == "__main__":
    main()
