"""Generate from the command line with any registered model family.

    python -m llava_mi355x.cli --model DIR --tokens 1,2,3 [--tokens 7,8] --max-new-tokens 32
    python -m llava_mi355x.cli --model DIR --prompt "..." --temperature 0.7 --top-p 0.9

Prompts come as token ids (any checkpoint) or as text (checkpoints with a tokenizer beside the weights).  Several prompts decode together.  One line per prompt: the new
ids, or the new text where there is a tokenizer."""
from __future__ import annotations

import argparse
import os
import sys

import torch


def parse(argv=None):
    ap = argparse.ArgumentParser(prog="llava_mi355x.cli", description="generate with a checkpoint folder")
    ap.add_argument("--model", required=True)
    ap.add_argument("--tokens", action="append", default=[], help="a prompt as comma-separated ids (repeatable)")
    ap.add_argument("--prompt", action="append", default=[], help="a prompt as text (repeatable)")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--dtype", default="bfloat16", choices=["bfloat16", "float16", "float32"])
    ap.add_argument("--temperature", type=float, default=0.0, help="0: greedy")
    ap.add_argument("--top-p", type=float, default=None)
    ap.add_argument("--top-k", type=int, default=None)
    ap.add_argument("--seed", type=int, default=0)
    ap.add_argument("--num-beams", type=int, default=1)
    ap.add_argument("--eos", type=int, default=None)
    ap.add_argument("--max-position", type=int, default=None, help="cache positions per sequence")
    a = ap.parse_args(argv)
    if not a.tokens and not a.prompt:
        ap.error("give --tokens or --prompt")
    return a


def main(argv=None) -> int:
    a = parse(argv)
    from .registry import load_model
    model = load_model(a.model, dtype=getattr(torch, a.dtype), max_position=a.max_position)
    tokenizer = None
    if a.prompt or any(os.path.isfile(os.path.join(a.model, n)) for n in ("tokenizer.json", "tokenizer.model")):
        from transformers import AutoTokenizer
        tokenizer = AutoTokenizer.from_pretrained(a.model, use_fast=False)
    prompts = [[int(t) for t in p.replace(",", " ").split()] for p in a.tokens] + [tokenizer(p).input_ids for p in a.prompt]
    torch.manual_seed(a.seed)
    kw = dict(max_new_tokens=a.max_new_tokens, do_sample=a.temperature > 0, temperature=a.temperature or 1.0, top_p=a.top_p, top_k=a.top_k,
              eos_token_id=a.eos if a.eos is not None else (getattr(model.config, "eos_token_id", None) if getattr(model.config, "eos_token_id", None) is not None else -1))
    if a.num_beams == 1 and len(prompts) > 1:
        outs = model.generate_batch([torch.tensor(p) for p in prompts], **kw)
    else:
        outs = [model.generate(torch.tensor([p]), num_beams=a.num_beams, **kw)[0] for p in prompts]
    for p, o in zip(prompts, outs):
        new = o[len(p):].tolist()
        print(tokenizer.decode(new, skip_special_tokens=True) if tokenizer is not None else ",".join(map(str, new)), flush=True)
    return 0


if __name__ == "__main__":
    sys.exit(main())
