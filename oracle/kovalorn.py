"""Plain CPU restatement of the Kovalorn design: one function per mechanism.

Test infrastructure: slow, no batching, no cache, nothing shared with lit_llama_amd.  A whole sequence is computed from its first token;
`dtype` picks the arithmetic (float64 by default: the reference of the product's rounding).

    cfg      the parsed config.json
    tensors  name -> tensor, the names of model.safetensors
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional, Tuple

import torch

Tensors = Dict[str, torch.Tensor]


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square (eps inside the root), along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """The weight is stored as its distance from one."""
    return unit_rms(x, eps) * (1 + weight)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1 + torch.exp(-z))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3)))


def visible(i: int, window: int, keep: int) -> List[int]:
    """Positions that position i sees: the window that ends at i, and the first `keep` of the sequence."""
    return [j for j in range(i + 1) if i - j < window or j < keep]


def sink_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: int, keep: int,
                   sink: Optional[torch.Tensor]) -> torch.Tensor:
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; sink [H]: one more term of every softmax sum, without a value."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        see = visible(i, window, keep)
        for h in range(H):
            s = (k[see, h // per] @ q[i, h]) * scale
            top = s.max() if sink is None else torch.maximum(s.max(), sink[h])
            p = torch.exp(s - top)
            total = p.sum() if sink is None else p.sum() + torch.exp(sink[h] - top)
            out[i, h] = (p / total) @ v[see, h // per]
    return out


def attention_mixer(w: Tensors, i: int, m: dict, h: torch.Tensor, eps: float, kept: Dict[int, tuple]) -> torch.Tensor:
    """`kept`: layer -> (keys, values) of the layers that projected them, for the layers that borrow."""
    T, p = h.shape[0], f"l{i}.mix."
    q = unit_rms((h @ w[p + "q"].T).view(T, m["heads"], m["dim"]), eps)
    if m.get("kv_from") is None:
        k = unit_rms((h @ w[p + "k"].T).view(T, m["kv_heads"], m["dim"]), eps)
        kept[i] = k, (h @ w[p + "v"].T).view(T, m["kv_heads"], m["vdim"])
    k, v = kept[i if m.get("kv_from") is None else m["kv_from"]]
    mask = m.get("mask") or {}
    o = sink_attention(q, k, v, m["scale"], mask.get("size", T), mask.get("keep_first", 0), w[p + "sink"])
    return (o.reshape(T, -1) * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


def gated_ff(w: Tensors, p: str, h: torch.Tensor, act) -> torch.Tensor:
    return (act(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(h: torch.Tensor, router: torch.Tensor, top: int, scale: float) -> Tuple[torch.Tensor, torch.Tensor]:
    """(experts [T, top], their weights [T, top]): the largest sigmoid scores, scaled to sum to `scale`."""
    s = torch.sigmoid(h @ router.T)
    chosen = torch.argsort(s, dim=-1, descending=True, stable=True)[:, :top]
    picked = torch.gather(s, 1, chosen)
    return chosen, picked / (picked.sum(-1, keepdim=True) + 1e-20) * scale


def experts_ff(w: Tensors, p: str, spec: dict, h: torch.Tensor) -> torch.Tensor:
    r = spec["router"]
    chosen, weight = route(h, w[p + "router"], r["top"], r["scale"])
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(chosen[t].tolist(), weight[t]):
            out[t] += a * gated_ff(w, f"{p}e{e}.", h[t:t + 1], silu)[0]
    if spec.get("shared"):
        out = out + gated_ff(w, p + "shared.", h, silu)
    return out


def forward(cfg: dict, tensors: Tensors, tokens: List[int], dtype: torch.dtype = torch.float64) -> Tuple[torch.Tensor, torch.Tensor]:
    """(logits [T, vocab], residual after every layer [layers, T, width]) of one sequence from its first token."""
    w = {n: t.to(dtype) for n, t in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    trail, kept = [], {}
    for i, spec in enumerate(cfg["layers"]):
        x = x + attention_mixer(w, i, spec["mixer"], rms_norm(x, w[f"l{i}.norm1"], eps), eps, kept)
        mlp = spec["mlp"]
        if mlp is not None:
            h = rms_norm(x, w[f"l{i}.norm2"], eps)
            x = x + (gated_ff(w, f"l{i}.mlp.", h, gelu_tanh) if mlp["kind"] == "dense" else experts_ff(w, f"l{i}.mlp.", mlp, h))
        trail.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["embed"].T * cfg["logit_scale"], torch.stack(trail)
