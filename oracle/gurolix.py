"""Plain CPU restatement of the Gurolix design: one function per mechanism, one token at a time where there is a recurrence.

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


def sigmoid(z: torch.Tensor) -> torch.Tensor:
    return 1 / (1 + torch.exp(-z))


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * sigmoid(z)


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


# ---------------------------------------------------------------------------------------- around a sublayer
def gated_result(y: torch.Tensor, h: torch.Tensor, weight: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """A sublayer's result behind a gate per element that reads what the sublayer read."""
    return y * sigmoid(h @ weight.T + bias)


def depth_average(weights: torch.Tensor, stream: List[torch.Tensor]) -> torch.Tensor:
    """What goes on to the next layer: a weighted sum of the embedding output and every layer's result so far."""
    out = torch.zeros_like(stream[0])
    for w, x in zip(weights, stream):
        out = out + w * x
    return out


# ---------------------------------------------------------------------------------------- state-space recurrence
def short_conv(x: torch.Tensor, taps: torch.Tensor, bias: torch.Tensor) -> torch.Tensor:
    """y[t, c] = bias[c] + sum_j taps[c, n - 1 - j] x[t - j, c], zeros in front of the first row (x [T, channels], taps [channels, n])."""
    T, n = x.shape[0], taps.shape[1]
    out = bias.expand(T, -1).clone()
    for t in range(T):
        for j in range(min(n, t + 1)):
            out[t] += taps[:, n - 1 - j] * x[t - j]
    return out


def state_space(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, a_log: torch.Tensor, D: torch.Tensor) -> torch.Tensor:
    """x [T, H, vdim], B, C [T, G, N], dt [T, H] -> [T, H, vdim]: every head's state decays by exp(-exp(a_log) dt) and takes dt B x^T."""
    T, H, vd = x.shape
    per = H // B.shape[1]
    S = torch.zeros((H, B.shape[2], vd), dtype=x.dtype)
    out = torch.zeros_like(x)
    for t in range(T):
        b, c = B[t].repeat_interleave(per, 0), C[t].repeat_interleave(per, 0)
        S = S * torch.exp(-torch.exp(a_log) * dt[t])[:, None, None] + dt[t][:, None, None] * b[:, :, None] * x[t][:, None, :]
        out[t] = (S * c[:, :, None]).sum(1) + D[:, None] * x[t]
    return out


def gated_group_norm(y: torch.Tensor, z: torch.Tensor, weight: torch.Tensor, groups: int, eps: float) -> torch.Tensor:
    """silu(z) y, every one of `groups` equal parts over its own root mean square, then the weight."""
    g = y * silu(z)
    return unit_rms(g.view(g.shape[0], groups, -1), eps).reshape(g.shape) * weight


def mamba2_mixer(w: Tensors, p: str, m: dict, h: torch.Tensor, eps: float) -> torch.Tensor:
    T, H, G, N = h.shape[0], m["heads"], m["groups"], m["state"]
    inner = H * m["vdim"]
    z, xbc, dt = (h @ w[p + "in"].T).split([inner, inner + 2 * G * N, H], -1)
    x, B, C = silu(short_conv(xbc, w[p + "conv"], w[p + "conv.b"])).split([inner, G * N, G * N], -1)
    y = state_space(x.reshape(T, H, -1), B.reshape(T, G, N), C.reshape(T, G, N), softplus(dt + w[p + "dt_bias"]), w[p + "A_log"], w[p + "D"])
    return gated_group_norm(y.reshape(T, inner), z, w[p + "norm"], m["norm_groups"], eps) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------- attention
def frequencies(rot: dict) -> torch.Tensor:
    """Turns per position of every pair; with `scaling` slow ones are divided by its factor, those between two wavelengths partly."""
    n = rot["dims"]
    f = [float(rot["base"]) ** (-2 * i / n) for i in range(n // 2)]
    s = rot.get("scaling")
    if s:
        out = []
        for v in f:
            wave = 2 * math.pi / v
            if wave < s["original"] / s["high"]:
                out.append(v)
            elif wave > s["original"] / s["low"]:
                out.append(v / s["factor"])
            else:
                t = (s["original"] / wave - s["low"]) / (s["high"] - s["low"])
                out.append((1 - t) * v / s["factor"] + t * v)
        f = out
    return torch.tensor(f, dtype=torch.float64)


def rotate_halves(x: torch.Tensor, rot: dict) -> torch.Tensor:
    """x [T, heads, dim], row t at position t: dimensions (i, i + dims / 2), i < dims / 2, turn by t times their frequency."""
    T, half = x.shape[0], rot["dims"] // 2
    a = torch.arange(T, dtype=torch.float64)[:, None, None] * frequencies(rot)
    c, s = torch.cos(a).to(x.dtype), torch.sin(a).to(x.dtype)
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * c - v * s, v * c + u * s, x[..., 2 * half:]], -1)


def attend(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, softcap: Optional[float]) -> torch.Tensor:
    """q [T, H, dim], k [T, G, dim], v [T, G, vdim] -> [T, H, vdim]: every earlier row and the row itself; softcap bounds the scores."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    out = torch.zeros((T, H, v.shape[2]), dtype=q.dtype)
    seen = torch.ones((T, T), dtype=torch.bool).tril()
    for h in range(H):
        s = q[:, h] @ k[:, h // per].T * scale
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        s = torch.where(seen, s, torch.full_like(s, -math.inf))
        e = torch.exp(s - s.max(-1, keepdim=True).values)
        out[:, h] = e / e.sum(-1, keepdim=True) @ v[:, h // per]
    return out


def mix_values(v: torch.Tensor, first: torch.Tensor, lam: torch.Tensor) -> torch.Tensor:
    return (1 - lam) * v + lam * first


def attention_mixer(w: Tensors, p: str, kind: str, m: dict, h: torch.Tensor, eps: float, first: dict) -> torch.Tensor:
    """`first`: holds the values of the first layer that mixes them, once that has run."""
    T, H, G = h.shape[0], m["heads"], m["kv_heads"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, -1)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, -1)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, -1)
    if kind == "attention":
        q, k = unit_rms(q, eps) * w[p + "q.norm"], unit_rms(k, eps) * w[p + "k.norm"]
    q, k = rotate_halves(q, m["rot"]), rotate_halves(k, m["rot"])
    if m.get("v_mix"):
        if "v" in first:
            v = mix_values(v, first["v"], w[p + "vmix"])
        else:
            first["v"] = v
    return attend(q, k, v, m["scale"], m.get("softcap") if kind == "attention_2" else None).reshape(T, -1) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------- experts
def route(z: torch.Tensor, correction: torch.Tensor, top: int, groups: int, keep: int) -> Tuple[List[int], torch.Tensor]:
    """One token's logits -> (chosen experts, their weights): softmax scores; the choice adds the correction and looks into the `keep` best of
    `groups` equal runs of experts only."""
    e = torch.exp(z - z.max())
    s = e / e.sum()
    choice = s + correction
    size = len(z) // groups
    best = sorted(range(groups), key=lambda g: -float(choice[g * size:(g + 1) * size].max()))[:keep]
    allowed = [i for g in best for i in range(g * size, (g + 1) * size)]
    chosen = sorted(allowed, key=lambda i: -float(choice[i]))[:top]
    return chosen, s[chosen]


def expert(up: torch.Tensor, down: torch.Tensor, h: torch.Tensor) -> torch.Tensor:
    return torch.clamp(h @ up.T, min=0) ** 2 @ down.T


def experts_ff(w: Tensors, p: str, spec: dict, h: torch.Tensor) -> torch.Tensor:
    """Router outputs from `experts` on stand for the input itself."""
    r = spec["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(*route(h[t] @ w[p + "router"].T, w[p + "correction"], r["top"], g["count"], g["keep"])):
            out[t] += a * (h[t] if e >= r["experts"] else expert(w[f"{p}e{e}.up"], w[f"{p}e{e}.down"], h[t]))
    return out


def forward(cfg: dict, tensors: Tensors, tokens: List[int], dtype: torch.dtype = torch.float64) -> Tuple[torch.Tensor, torch.Tensor]:
    """(logits [T, vocab], residual after every layer [layers, T, width]) of one sequence from its first token."""
    w = {n: t.to(dtype) for n, t in tensors.items()}
    eps = cfg["norm"]["eps"]
    x = rms_norm(w["embed"][torch.as_tensor(tokens, dtype=torch.long)], w["embed.norm"], eps)
    stream, trail, first = [x], [], {}
    for i, spec in enumerate(cfg["layers"]):
        p = f"l{i}."
        h = rms_norm(x, w[p + "norm1"], eps)
        if spec["type"] == "mamba2":
            y = mamba2_mixer(w, p + "mix.", spec["mixer"], h, eps)
        else:
            y = attention_mixer(w, p + "mix.", spec["type"], spec["mixer"], h, eps, first)
        x = x + rms_norm(gated_result(y, h, w[p + "rg1"], w[p + "rg1.b"]), w[p + "norm1b"], eps)
        if spec.get("mlp") is not None:
            h = rms_norm(x, w[p + "norm2"], eps)
            y = experts_ff(w, p + "mlp.", spec["mlp"], h)
            x = x + rms_norm(gated_result(y, h, w[p + "rg2"], w[p + "rg2.b"]), w[p + "norm2b"], eps)
        stream.append(x)
        x = depth_average(w[p + "dwa"], stream)
        trail.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T, torch.stack(trail)
