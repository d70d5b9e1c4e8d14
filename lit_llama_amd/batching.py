"""Requests that decode together.

`BatchScheduler` keeps up to `max_batch` requests live on an engine that takes packed batches (hybrid_engine.HybridEngine): every round
admits waiting requests as prompt portions of at most `portion` tokens, then lets every request that has its whole prompt in decode one
token.  Finished requests give their slot back at once.  Models whose engine holds one sequence are served one request after another by
`generate_batch`.
"""
from __future__ import annotations

from collections import deque
from dataclasses import dataclass, field
from typing import Deque, List, Optional, Sequence

import torch

from . import ops
from .generate import generate


@dataclass
class Request:
    prompt: List[int]
    max_new_tokens: int
    temperature: float = 1.0
    top_k: Optional[int] = None      # 1: greedy
    eos_id: Optional[int] = None
    seed: Optional[int] = None       # of this request's draws
    out: List[int] = field(default_factory=list)
    slot: int = -1
    done: int = 0                    # tokens fed so far
    uniforms: Optional[torch.Tensor] = None

    def finished(self) -> bool:
        return len(self.out) >= self.max_new_tokens or (self.eos_id is not None and bool(self.out) and self.out[-1] == self.eos_id)


class BatchScheduler:
    def __init__(self, engine, *, max_batch: int = 16, portion: Optional[int] = None, max_len: int = 4096):
        self.engine, self.max_batch = engine, max_batch
        self.portion = portion or engine.max_rows
        engine.ensure(engine.slots.live + max_batch, max(max_len, engine.max_len))
        self.waiting: Deque[Request] = deque()
        self.live: List[Request] = []
        dev = engine.device
        self._pos = torch.zeros(1, dtype=torch.int32, device=dev)
        self._next = torch.zeros(1, dtype=torch.int32, device=dev)

    def submit(self, request: Request) -> Request:
        if not request.prompt or request.max_new_tokens < 1:
            raise ValueError("a request has a prompt and at least one new token")
        if len(request.prompt) + request.max_new_tokens > self.engine.max_len:
            raise ValueError(f"request of {len(request.prompt)} + {request.max_new_tokens} tokens in a cache of {self.engine.max_len}")
        self.waiting.append(request)
        return request

    def _admit(self) -> None:
        while self.waiting and len(self.live) < self.max_batch:
            r = self.waiting.popleft()
            r.slot = self.engine.acquire()
            self.live.append(r)

    def _draw(self, r: Request, row: torch.Tensor) -> int:
        if r.uniforms is None:
            gen = torch.Generator(device=row.device)
            gen.manual_seed(r.seed if r.seed is not None else torch.seed() & 0x7FFFFFFF)
            r.uniforms = torch.rand(r.max_new_tokens, generator=gen, device=row.device)
        self._pos.fill_(len(r.out))
        ops.sample(row, r.temperature, r.top_k, r.uniforms, self._pos, self._next)
        return int(self._next)

    def round(self) -> bool:
        """One step of the batch; False once nothing is left."""
        from .hybrid_engine import Entry

        self._admit()
        if not self.live:
            return False
        entries, asks = [], []
        for r in self.live:
            seq = r.prompt if r.done < len(r.prompt) else r.out[-1:]
            lo = r.done if r.done < len(r.prompt) else 0
            toks = seq[lo:lo + self.portion]
            last = r.done + len(toks) >= len(r.prompt)
            entries.append(Entry(r.slot, r.done, toks, [len(toks) - 1] if last else []))
            r.done += len(toks)
            if last:
                asks.append(r)
        logits = self.engine.step(entries)
        if asks:
            greedy = torch.argmax(logits, -1).tolist() if any(r.top_k == 1 for r in asks) else None
            for i, r in enumerate(asks):
                r.out.append(greedy[i] if r.top_k == 1 else self._draw(r, logits[i].contiguous()))
        for r in [r for r in self.live if r.finished()]:
            self.engine.release(r.slot)
            r.slot = -1
            self.live.remove(r)
        return bool(self.live or self.waiting)

    def run(self) -> None:
        while self.round():
            pass


@torch.no_grad()
def generate_batch(model, prompts: Sequence[Sequence[int]], max_new_tokens, *, temperature: float = 1.0, top_k: Optional[int] = None,
                   eos_id: Optional[int] = None, seed: Optional[int] = None, max_batch: int = 16,
                   portion: Optional[int] = None) -> List[List[int]]:
    """New tokens of every prompt (`max_new_tokens`: one number or one per prompt), in the order of the prompts."""
    new = list(max_new_tokens) if not isinstance(max_new_tokens, int) else [max_new_tokens] * len(prompts)
    engine = model.engine()
    if getattr(engine, "supports_batches", False):
        need = max(len(p) + n for p, n in zip(prompts, new))
        sched = BatchScheduler(engine, max_batch=min(max_batch, len(prompts)), portion=portion, max_len=need)
        reqs = [sched.submit(Request(list(p), n, temperature, top_k, eos_id, None if seed is None else seed + i))
                for i, (p, n) in enumerate(zip(prompts, new))]
        sched.run()
        return [[t for t in r.out if t != eos_id] if eos_id is not None else r.out for r in reqs]
    dev = next(model.parameters()).device
    out = []
    for i, (p, n) in enumerate(zip(prompts, new)):
        if seed is not None:
            torch.manual_seed(seed + i)
        model.reset_cache()
        y = generate(model, torch.tensor(list(p), device=dev), n, temperature=temperature, top_k=top_k, eos_id=eos_id)
        out.append(y[len(p):].tolist())
    return out
