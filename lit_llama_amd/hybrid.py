"""Layered hybrid decoders: a list of layers, each with its own mixer (window attention, gated delta rule, gated linear attention) and an
optional feed-forward, some of them run several times in a row.

`HybridConfig` reads a parsed config.json; `HybridLM` holds the weights under their checkpoint names and hands the arithmetic to
`hybrid_engine.HybridEngine` (csrc/hybrid.hip and the kernels it calls).  The Sekulorn design is the family registered here; a mixer or a
feed-forward of another design is an entry in MIXERS / MLPS and a kernel.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from . import _native as nat


@dataclass
class MixerSpec:
    """Sizes and constants of one layer's mixer; which fields count depends on `type`."""

    type: str                      # attention | delta | gla
    heads: int
    kv_heads: int
    dim: int                       # query / key size of a head
    vdim: int                      # value size of a head
    scale: float = 1.0             # attention
    window: int = 0
    rot_dims: int = 0
    rot_base: float = 10000.0
    taps: int = 0                  # delta: convolution taps
    tau: float = 1.0               # gla


@dataclass
class LayerSpec:
    mixer: MixerSpec
    ff: int = 0                    # width of the squared-ReLU feed-forward, 0: none


def _only(d: dict, known: Tuple[str, ...], what: str) -> None:
    extra = sorted(set(d) - set(known))
    if extra:
        raise ValueError(f"{what}: unknown configuration {extra}")


def _attention(m: dict) -> MixerSpec:
    """No `rot`: no rotation; no `mask`: every earlier row is seen."""
    _only(m, ("heads", "kv_heads", "dim", "vdim", "rot", "scale", "mask"), "attention mixer")
    rot, mask = m.get("rot") or {"base": 1.0, "dims": 0}, m.get("mask") or {"size": 1 << 30}
    _only(rot, ("base", "dims"), "rotation")
    _only(mask, ("size",), "mask")
    return MixerSpec("attention", m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale=float(m["scale"]), window=int(mask["size"]),
                     rot_dims=int(rot["dims"]), rot_base=float(rot["base"]))


def _delta(m: dict) -> MixerSpec:
    _only(m, ("heads", "kv_heads", "dim", "vdim", "conv"), "delta mixer")
    return MixerSpec("delta", m["heads"], m["kv_heads"], m["dim"], m["vdim"], taps=int(m["conv"]))


def _gla(m: dict) -> MixerSpec:
    _only(m, ("heads", "dim", "vdim", "tau"), "gla mixer")
    return MixerSpec("gla", m["heads"], m["heads"], m["dim"], m["vdim"], tau=float(m["tau"]))


MIXERS = {"attention": _attention, "delta": _delta, "gla": _gla}
MLPS = ("dense",)


@dataclass
class HybridConfig:
    vocab_size: int
    width: int
    layers: List[LayerSpec]
    eps: float
    residual_mult: float = 1.0
    loop: Tuple[int, int, int] = (0, 0, 1)  # layers start .. stop - 1 run `times` times in a row
    architecture: str = "Sekulorn"
    block_size: int = 1 << 24               # (positions are not tabulated: nothing limits a sequence but its cache)
    raw: dict = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, d: dict) -> "HybridConfig":
        _only(d["norm"], ("eps",), "norm")
        layers = []
        for e in d["layers"]:
            _only(e, ("type", "mixer", "mlp"), "layer")
            if e["type"] not in MIXERS:
                raise ValueError(f"unknown mixer {e['type']!r} (known: {sorted(MIXERS)})")
            mlp = e.get("mlp")
            if mlp is not None:
                _only(mlp, ("kind", "ff"), "feed-forward")
                if mlp["kind"] not in MLPS:
                    raise ValueError(f"unknown feed-forward {mlp['kind']!r} (known: {list(MLPS)})")
            spec = MIXERS[e["type"]](e["mixer"])
            if spec.heads % spec.kv_heads:
                raise ValueError(f"{spec.heads} heads over {spec.kv_heads} key / value heads")
            layers.append(LayerSpec(spec, int(mlp["ff"]) if mlp is not None else 0))
        loop = d.get("loop")
        if loop is not None:
            _only(loop, ("start", "stop", "times"), "loop")
            span = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            if not (0 <= span[0] <= span[1] <= len(layers) and span[2] >= 1):
                raise ValueError(f"bad loop {span} over {len(layers)} layers")
        return cls(int(d["vocab"]), int(d["width"]), layers, float(d["norm"]["eps"]), float(d.get("residual_mult", 1.0)),
                   span if loop is not None else (0, 0, 1), d.get("architecture", "Sekulorn"), raw=d)

    @property
    def padded_vocab_size(self) -> int:
        return self.vocab_size

    def runs(self) -> List[int]:
        """The layer of every run, in order: a looped layer appears once per pass."""
        a, b, times = self.loop
        return [*range(a), *(list(range(a, b)) * times), *range(b, len(self.layers))]


# the pieces of a mixer's stacked input projection, in the order of their columns
PROJECTIONS = {"attention": ("q", "k", "v", "g"), "delta": ("q", "k", "v", "g", "a", "b"), "gla": ("q", "k", "v", "g", "a1")}


def tensor_shapes(cfg: HybridConfig, rank: Dict[int, int]) -> Dict[str, Tuple[int, ...]]:
    """name -> shape of every tensor of a checkpoint; rank[i]: the low-rank size of gla layer i (only its tensors know it)."""
    W = cfg.width
    out = {"embed": (cfg.vocab_size, W)}
    for i, l in enumerate(cfg.layers):
        p, m = f"l{i}.", l.mixer
        hv, gk = m.heads * m.vdim, m.kv_heads * m.dim
        out[p + "norm1"] = (W,)
        x = p + "mix."
        if m.type == "attention":
            out.update({x + "q": (m.heads * m.dim, W), x + "k": (gk, W), x + "v": (m.kv_heads * m.vdim, W), x + "g": (m.heads, W)})
        else:
            out.update({x + "q": (gk, W), x + "k": (gk, W), x + "v": (hv, W), x + "g": (hv, W), x + "norm": (m.vdim,)})
        if m.type == "delta":
            out.update({x + "q.conv": (gk, m.taps), x + "k.conv": (gk, m.taps), x + "v.conv": (hv, m.taps), x + "b": (m.heads, W),
                        x + "a": (m.heads, W), x + "A_log": (m.heads,), x + "dt_bias": (m.heads,)})
        if m.type == "gla":
            out.update({x + "a1": (rank[i], W), x + "a2": (gk, rank[i]), x + "a2.b": (gk,)})
        out[x + "o"] = (W, hv)
        if l.ff:
            out.update({p + "norm2": (W,), p + "mlp.up": (l.ff, W), p + "mlp.down": (W, l.ff)})
    out.update({"final.norm": (W,), "head": (cfg.vocab_size, W)})
    return out


class HybridLM(nn.Module):
    """Weights by checkpoint name (`model.tensors["l0.mix.q"]`), forward through the native engine.

    `forward(idx, max_seq_length, input_pos)` is LLaMA.forward's interface for one sequence with a cache; batches go through
    `engine().step` (batching.BatchScheduler)."""

    def __init__(self, config: HybridConfig, dtype: torch.dtype = torch.bfloat16, device="cuda"):
        super().__init__()
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError("a hybrid model runs in bfloat16 or float32")
        self.config = config
        self.dtype = dtype
        self.device = torch.device(device)
        self.tensors: Dict[str, torch.Tensor] = {}
        self._engine = None
        self.use_engine = True

    def load_state_dict(self, sd, strict: bool = True):
        """`sd`: name -> tensor (lazy tensors of checkpoint.lazy_load included).  Names and shapes must be the configuration's."""
        rank = {i: sd[f"l{i}.mix.a1"].shape[0] for i, l in enumerate(self.config.layers) if l.mixer.type == "gla" and f"l{i}.mix.a1" in sd}
        shapes = tensor_shapes(self.config, {**{i: 0 for i in range(len(self.config.layers))}, **rank})
        missing, extra = sorted(set(shapes) - set(sd)), sorted(set(sd) - set(shapes))
        if missing or (strict and extra):
            raise ValueError(f"checkpoint and configuration differ: missing {missing[:5]}, unexpected {extra[:5]}")
        self._engine = None
        self.tensors = {}
        for name, shape in shapes.items():
            t = sd[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name}: shape {tuple(t.shape)}, the configuration says {tuple(shape)}")
            self.tensors[name] = t.to(device=self.device, dtype=self.dtype)

    def state_dict(self, *args, **kwargs):
        return dict(self.tensors)

    def engine(self, check: bool = True):
        from .hybrid_engine import HybridEngine

        if self._engine is None:
            if self.device.type != "cuda":
                raise nat.NativeError(f"HybridLM: the weights are on {self.device}; the model runs on the GPU only")
            if not self.tensors:
                raise nat.NativeError("HybridLM: no weights loaded")
            self._engine = HybridEngine(self)
        return self._engine

    def reset_cache(self) -> None:
        if self._engine is not None:
            self._engine.reset_cache()

    def forward(self, idx: torch.Tensor, max_seq_length: Optional[int] = None, input_pos: Optional[torch.Tensor] = None) -> torch.Tensor:
        nat.require_gpu(idx, "HybridLM.forward")
        B, T = idx.shape
        eng = self.engine()
        if input_pos is None:  # no cache: every row of idx is a sequence of its own
            return eng.forward_no_cache(idx)
        if B != 1:
            raise nat.NativeError("HybridLM.forward with a cache takes one sequence (batches: batching.BatchScheduler)")
        return eng.forward(idx, max_seq_length or self.config.block_size, input_pos)
