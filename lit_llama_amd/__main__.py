"""Command line: `python -m lit_llama_amd --model PATH --prompt-ids 1,2,3 [--prompt-ids ...]`.

PATH is a folder with config.json and model.safetensors or a lit-llama checkpoint (registry.load_model).  Prompts are token ids, or text
with `--tokenizer` (a SentencePiece model).  Several prompts decode as one batch where the model's engine takes batches."""
from __future__ import annotations

import argparse
import sys
import time

import torch

from .batching import generate_batch
from .registry import load_model


def main(argv=None) -> int:
    ap = argparse.ArgumentParser(prog="lit_llama_amd", description="Generate tokens with a model of the framework.")
    ap.add_argument("--model", required=True, help="folder with config.json and model.safetensors, or a lit-llama .pth")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--quantize", choices=["llm.int8", "gptq.int4", "gptq.int8"], default=None)
    ap.add_argument("--prompt-ids", action="append", default=[], help="comma-separated token ids; repeat for a batch")
    ap.add_argument("--prompt", action="append", default=[], help="text (needs --tokenizer); repeat for a batch")
    ap.add_argument("--tokenizer", help="SentencePiece model")
    ap.add_argument("--max-new-tokens", type=int, default=50)
    ap.add_argument("--temperature", type=float, default=0.8)
    ap.add_argument("--top-k", type=int, default=200, help="1: greedy")
    ap.add_argument("--eos-id", type=int)
    ap.add_argument("--seed", type=int, default=1234)
    ap.add_argument("--max-batch", type=int, default=16)
    ap.add_argument("--portion", type=int, help="prompt tokens of a request per step")
    a = ap.parse_args(argv)
    prompts = [[int(t) for t in p.split(",")] for p in a.prompt_ids]
    sp = None
    if a.prompt:
        if not a.tokenizer:
            ap.error("--prompt needs --tokenizer")
        import sentencepiece

        sp = sentencepiece.SentencePieceProcessor(model_file=a.tokenizer)
        prompts += [[sp.bos_id(), *sp.encode(p)] for p in a.prompt]
    if not prompts:
        ap.error("nothing to continue: give --prompt-ids or --prompt")
    model = load_model(a.model, getattr(torch, a.dtype), quantize=a.quantize)
    t0 = time.perf_counter()
    outs = generate_batch(model, prompts, a.max_new_tokens, temperature=a.temperature, top_k=a.top_k, eos_id=a.eos_id, seed=a.seed,
                          max_batch=a.max_batch, portion=a.portion)
    torch.cuda.synchronize()
    dt = time.perf_counter() - t0
    for p, o in zip(prompts, outs):
        print(sp.decode(p + o) if sp is not None else ",".join(map(str, p + o)))
    n = sum(map(len, outs))
    print(f"{n} new tokens in {dt:.2f} s ({n / dt:.1f} tokens/s, prompts included)", file=sys.stderr)
    return 0


if __name__ == "__main__":
    sys.exit(main())
