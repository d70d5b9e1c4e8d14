"""Plain CPU restatement of the Sekulorn design: one function per mechanism, one token at a time where there is a recurrence.

Test infrastructure: slow, no batching, no cache, nothing shared with lit_llama_amd.  A whole sequence is computed from its first token;
`dtype` picks the arithmetic (float64 by default: the reference of the product's rounding).

    cfg      the parsed config.json
    tensors  name -> tensor, the names of model.safetensors
"""
from __future__ import annotations

from typing import Dict, List, Tuple

import torch

Tensors = Dict[str, torch.Tensor]


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * weight over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def unit_vector(x: torch.Tensor, eps: float = 1e-6) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + eps)


def silu(x: torch.Tensor) -> torch.Tensor:
    return x / (1 + torch.exp(-x))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def squared_relu(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0) ** 2


def rotate_pairs(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """x [T, heads, dim], row t at position t: dimensions (2i, 2i + 1), 2i + 1 < dims, turn by t * base^(-2i / dims)."""
    T = x.shape[0]
    out = x.clone()
    for i in range(dims // 2):
        a = torch.arange(T, dtype=torch.float64) * base ** (-2.0 * i / dims)
        c, s = torch.cos(a).to(x.dtype)[:, None], torch.sin(a).to(x.dtype)[:, None]
        u, v = x[..., 2 * i], x[..., 2 * i + 1]
        out[..., 2 * i], out[..., 2 * i + 1] = u * c - v * s, v * c + u * s
    return out


def window_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, window: int) -> torch.Tensor:
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]; row i sees rows j with 0 <= i - j < window."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    for i in range(T):
        lo = max(0, i - window + 1)
        for h in range(H):
            s = (k[lo:i + 1, h // per] @ q[i, h]) * scale
            p = torch.exp(s - s.max())
            out[i, h] = (p / p.sum()) @ v[lo:i + 1, h // per]
    return out


def short_conv(x: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """y[t, c] = sum_j taps[c, n - 1 - j] x[t - j, c], zeros before the first row (x [T, channels], taps [channels, n])."""
    n = taps.shape[1]
    out = torch.zeros_like(x)
    for j in range(n):
        shifted = torch.zeros_like(x)
        if j < x.shape[0]:
            shifted[j:] = x[:x.shape[0] - j]
        out = out + shifted * taps[:, n - 1 - j]
    return out


def delta_rule(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor) -> torch.Tensor:
    """q, k [T, G, dim], v [T, H, vdim], g, beta [T, H] -> [T, H, vdim]: decay, correct the stored value of k, read with q."""
    T, H, vd = v.shape
    per = H // k.shape[1]
    S = torch.zeros((H, k.shape[2], vd), dtype=v.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        kt, qt = k[t].repeat_interleave(per, 0), q[t].repeat_interleave(per, 0)
        S = S * g[t][:, None, None]
        u = beta[t][:, None] * (v[t] - (S * kt[:, :, None]).sum(1))
        S = S + kt[:, :, None] * u[:, None, :]
        out[t] = (S * qt[:, :, None]).sum(1)
    return out


def gated_linear_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, alpha: torch.Tensor) -> torch.Tensor:
    """q, k, alpha [T, H, dim], v [T, H, vdim] -> [T, H, vdim]: every key channel's row of the state decays by its own alpha."""
    T, H, vd = v.shape
    S = torch.zeros((H, k.shape[2], vd), dtype=v.dtype)
    out = torch.zeros_like(v)
    for t in range(T):
        S = S * alpha[t][:, :, None] + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out


# ---------------------------------------------------------------------------------------- mixers
def attention_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T = h.shape[0]
    q = (h @ w[p + "q"].T).view(T, m["heads"], m["dim"])
    k = (h @ w[p + "k"].T).view(T, m["kv_heads"], m["dim"])
    v = (h @ w[p + "v"].T).view(T, m["kv_heads"], m["vdim"])
    if m.get("rot"):
        q, k = (rotate_pairs(t, m["rot"]["dims"], m["rot"]["base"]) for t in (q, k))
    o = window_attention(q, k, v, m["scale"], m["mask"]["size"] if m.get("mask") else T)
    o = o * torch.sigmoid(h @ w[p + "g"].T)[:, :, None]
    return o.reshape(T, -1) @ w[p + "o"].T


def delta_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T = h.shape[0]
    q, k, v = (silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit_vector(q.view(T, m["kv_heads"], m["dim"])) * m["dim"] ** -0.5
    k = unit_vector(k.view(T, m["kv_heads"], m["dim"]))
    v = v.view(T, m["heads"], m["vdim"])
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o = rms_norm(delta_rule(q, k, v, g, beta), w[p + "norm"], eps).reshape(T, -1)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def gla_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, d = h.shape[0], m["heads"], m["dim"]
    q = (h @ w[p + "q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, d)
    v = (h @ w[p + "v"].T).view(T, H, m["vdim"])
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    alpha = torch.exp(-softplus(-z) / m["tau"]).view(T, H, d)
    o = rms_norm(gated_linear_attention(q, k, v, alpha), w[p + "norm"], eps).reshape(T, -1)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


MIXERS = {"attention": attention_mixer, "delta": delta_mixer, "gla": gla_mixer}


def layer_order(cfg: dict) -> List[int]:
    """Layer index of every run: layers loop.start .. loop.stop - 1 are run loop.times times in a row."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return list(range(n))
    return (list(range(loop["start"])) + list(range(loop["start"], loop["stop"])) * loop["times"] + list(range(loop["stop"], n)))


def forward(cfg: dict, tensors: Tensors, tokens: List[int], dtype: torch.dtype = torch.float64) -> Tuple[torch.Tensor, torch.Tensor]:
    """(logits [T, vocab], residual after every layer run [runs, T, width]) of one sequence from its first token."""
    w = {n: t.to(dtype) for n, t in tensors.items()}
    eps, mult = cfg["norm"]["eps"], cfg["residual_mult"]
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    trail = []
    for i in layer_order(cfg):
        spec, p = cfg["layers"][i], f"l{i}."
        x = x + mult * MIXERS[spec["type"]](w, p + "mix.", spec["mixer"], rms_norm(x, w[p + "norm1"], eps), eps)
        if spec["mlp"] is not None:
            x = x + mult * (squared_relu(rms_norm(x, w[p + "norm2"], eps) @ w[p + "mlp.up"].T) @ w[p + "mlp.down"].T)
        trail.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(trail)
