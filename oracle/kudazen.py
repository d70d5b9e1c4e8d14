"""Plain CPU restatement of the Kudazen design: one function per mechanism.

Test infrastructure: slow, no batching, no cache, nothing shared with lit_llama_amd.  A whole sequence is computed from its first token;
`dtype` picks the arithmetic (float64 by default: the reference of the product's rounding).

    cfg      the parsed config.json
    tensors  name -> tensor, the names of model.safetensors
"""
from __future__ import annotations

from typing import Dict, List, Optional, Tuple

import torch

Tensors = Dict[str, torch.Tensor]


def unit_rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    """x over its root mean square (eps inside the root), along the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """Every one of `groups` equal parts of a vector over its own root mean square, then the weight."""
    parts = x.view(*x.shape[:-1], groups, x.shape[-1] // groups)
    return unit_rms(parts, eps).reshape(x.shape) * weight


def rotate_pairs(x: torch.Tensor, base: float) -> torch.Tensor:
    """x [T, ..., n], row t at position t: the pair (2i, 2i + 1) turns by t base^(-2i / n)."""
    T, n = x.shape[0], x.shape[-1]
    f = torch.tensor([base ** (-2 * i / n) for i in range(n // 2)], dtype=torch.float64)
    a = (torch.arange(T, dtype=torch.float64)[:, None] * f).view(T, *[1] * (x.dim() - 2), n // 2)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    u, v = x[..., 0::2], x[..., 1::2]
    return torch.stack([u * c - v * s, v * c + u * s], -1).reshape(x.shape)


def softmax_rows(scores: torch.Tensor, sink: Optional[float] = None) -> torch.Tensor:
    """Weights of a row of scores; a sink is one more term of the sum."""
    m = scores.max() if sink is None else torch.maximum(scores.max(), sink)
    e = torch.exp(scores - m)
    return e / (e.sum() if sink is None else e.sum() + torch.exp(sink - m))


# ---------------------------------------------------------------------------------------- chunked attention with a distance bias
def slopes(heads: int) -> List[float]:
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def chunk_visible(i: int, size: Optional[int]) -> range:
    """Positions that position i sees: from the first of its chunk on."""
    return range(0 if size is None else i - i % size, i + 1)


def chunk_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, factor: torch.Tensor, slope: List[float], size: Optional[int]) -> torch.Tensor:
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; factor [H] of the scores, slope [H] of the distance taken off."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        see = chunk_visible(i, size)
        a, b = see.start, see.stop
        dist = i - torch.arange(a, b, dtype=q.dtype)
        for h in range(H):
            s = k[a:b, h // per] @ q[i, h] * factor[h] - slope[h] * dist
            out[i, h] = softmax_rows(s) @ v[a:b, h // per]
    return out


def attention_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ w[p + "q"].T).view(T, H, m["dim"])
    k = (h @ w[p + "k"].T).view(T, G, m["dim"])
    v = unit_rms((h @ w[p + "v"].T).view(T, G, m["vdim"]), eps)
    o = chunk_attention(q, k, v, m["scale"] * w[p + "temp"], slopes(H), (m.get("mask") or {}).get("size"))
    return o.reshape(T, -1) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------- latent attention
def sink_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sink: torch.Tensor) -> torch.Tensor:
    """Causal; q, k [T, H, n], v [T, H, vdim], sink [H]."""
    T, H, _ = q.shape
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        for h in range(H):
            out[i, h] = softmax_rows(k[:i + 1, h] @ q[i, h] * scale, sink[h]) @ v[:i + 1, h]
    return out


def latent_parts(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> Tuple[torch.Tensor, torch.Tensor, torch.Tensor]:
    """Rotated queries [T, H, dim + rot_dim], latents [T, kv_rank] and the shared rotated key part [T, rot_dim]."""
    T, H, n, r = h.shape[0], m["heads"], m["dim"], m["kv_rank"]
    q = unit_rms(h @ w[p + "dq"].T, eps) * w[p + "dq.norm"] @ w[p + "uq"].T
    q = q.view(T, H, n + m["rot_dim"])
    q = torch.cat([q[..., :n], rotate_pairs(q[..., n:], m["rot"]["base"])], -1)
    d = h @ w[p + "dkv"].T
    return q, unit_rms(d[:, :r], eps) * w[p + "dkv.norm"], rotate_pairs(d[:, r:], m["rot"]["base"])


def latent_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H = h.shape[0], m["heads"]
    q, c, kr = latent_parts(w, p, m, h, eps)
    k = (c @ w[p + "uk"].T).view(T, H, m["dim"])
    k = torch.cat([k, kr[:, None].expand(T, H, m["rot_dim"])], -1)
    v = (c @ w[p + "uv"].T).view(T, H, m["vdim"])
    return sink_attention(q, k, v, m["scale"], w[p + "sink"]).reshape(T, -1) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------- time mixing with a matrix state
def shifted(h: torch.Tensor) -> torch.Tensor:
    """Every row's predecessor, zeros in front of the first."""
    return torch.cat([torch.zeros_like(h[:1]), h[:-1]])


def token_mix(h: torch.Tensor, mu: torch.Tensor) -> torch.Tensor:
    return h + (shifted(h) - h) * mu


def channel_decay(z: torch.Tensor) -> torch.Tensor:
    return torch.exp(-torch.exp(z))


def wkv(r: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: torch.Tensor, u: torch.Tensor) -> torch.Tensor:
    """r, k, v, decay [T, H, dim], u [H, dim] -> o [T, H, dim]: the state in front of a token, and the token itself with the bonus u."""
    T, H, n = r.shape
    S = torch.zeros((H, n, n), dtype=r.dtype)
    out = torch.zeros_like(r)
    for t in range(T):
        new = k[t][:, :, None] * v[t][:, None, :]
        out[t] = ((S + u[:, :, None] * new) * r[t][:, :, None]).sum(1)
        S = decay[t][:, :, None] * S + new
    return out


def wkv_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, n = h.shape[0], m["heads"], m["dim"]
    x = {s: token_mix(h, w[f"{p}mu.{s}"]) for s in "rkvgw"}
    r, k, v = ((x[s] @ w[p + s].T).view(T, H, n) for s in "rkv")
    g = x["g"] @ w[p + "g"].T
    z = torch.tanh(x["w"] @ w[p + "w1"].T) @ w[p + "w2"].T + w[p + "w0"]
    o = unit_rms(wkv(r, k, v, channel_decay(z).view(T, H, n), w[p + "u"]), eps).reshape(T, -1) * w[p + "norm"]
    return (o * (g / (1 + torch.exp(-g)))) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------- feed-forward, layers
def clamped_gate(gate: torch.Tensor, up: torch.Tensor, limit: float) -> torch.Tensor:
    g, u = gate.clamp(max=limit), up.clamp(-limit, limit)
    return g / (1 + torch.exp(-1.702 * g)) * (u + 1)


def clamped_ff(w: Tensors, p: str, f: dict, h: torch.Tensor) -> torch.Tensor:
    return clamped_gate(h @ w[p + "gate"].T, h @ w[p + "up"].T, f["limit"]) @ w[p + "down"].T


MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer, "wkv": wkv_mixer}


def forward(cfg: dict, tensors: Tensors, tokens: List[int], dtype: torch.dtype = torch.float64) -> Tuple[torch.Tensor, torch.Tensor]:
    """Logits [T, vocab], and the residual stream behind every layer [layers, T, width]."""
    w = {n: t.to(dtype) for n, t in tensors.items()}
    eps, groups = cfg["norm"]["eps"], cfg["norm"]["groups"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    trail = []
    for i, spec in enumerate(cfg["layers"]):
        src = spec.get("weights_of")
        p = f"l{i if src is None else src}."
        h = group_norm(x, w[p + "norm1"], groups, eps)
        y = MIXERS[spec["type"]](w, p + "mix.", spec["mixer"], h, eps)
        if spec.get("mlp") is not None:
            y = y + clamped_ff(w, p + "mlp.", spec["mlp"], h)
        x = x + y
        trail.append(x)
    return group_norm(x, w["final.norm"], groups, eps) @ w["embed"].T, torch.stack(trail)
