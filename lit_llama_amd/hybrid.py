"""Layered hybrid decoders: a list of layers, each with its own mixer (window or chunk attention, latent attention, gated delta rule, gated
linear attention, WKV time mixing, state-space duality) and an optional feed-forward (squared ReLU, gated GELU, clamped gate, mixture of
experts), behind or beside the mixer, or between norms of its own; some layers run several times in a row, some use another layer's weights.

`HybridConfig` reads a parsed config.json; `HybridLM` holds the weights under their checkpoint names and hands the arithmetic to
`hybrid_engine.HybridEngine` (csrc/hybrid.hip and the kernels it calls).  A design is an entry in DESIGNS: which mixers and feed-forwards it
has, how it reads them from its configuration, and what it does around them; a mixer or a feed-forward that none has yet is a spec and a
kernel.
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Callable, Dict, List, Optional, Tuple

import torch
import torch.nn as nn

from . import _native as nat


@dataclass
class MixerSpec:
    """Sizes and constants of one layer's mixer; which fields count depends on `type`."""

    type: str                      # attention | latent | delta | gla | wkv | ssd
    heads: int
    kv_heads: int
    dim: int                       # query / key size of a head
    vdim: int                      # value size of a head
    scale: float = 1.0             # attention
    window: int = 0
    keep: int = 0                  # first tokens that stay visible
    rot_dims: int = 0
    rot_base: float = 10000.0
    unit_qk: bool = False          # q and k over their root mean square
    sink: bool = False             # a learned term in every softmax sum
    gate_values: bool = False      # a gate per value, not per head
    kv_from: Optional[int] = None  # the layer whose keys and values are read
    taps: int = 0                  # delta, ssd: convolution taps
    tau: float = 1.0               # gla
    chunked: bool = False          # `window` counts chunks from position 0
    temp: bool = False             # a learned factor per head of the scores
    bias: bool = False             # a distance bias, its slopes from the number of heads
    unit_v: bool = False           # v over its root mean square
    gated: bool = True             # attention with a sigmoid gate
    rot_dim: int = 0               # latent: rotated query / key size of a head, next to dim
    q_rank: int = 0
    kv_rank: int = 0
    rot_halves: bool = False       # dimension i turns with i + rot_dims / 2, not with its neighbour
    rot_scaling: Optional[Tuple[float, float, float, float]] = None  # factor, low, high, original length: slow turns are slowed down further
    qk_norm: bool = False          # factors per dimension behind unit_qk
    biased: bool = False           # q, k and v have biases
    softcap: float = 0.0           # bound of the scores, 0: none
    v_mix: bool = False            # v is mixed with that of the first such layer
    norm_groups: int = 1           # ssd: parts of the output that are normalised by themselves


@dataclass
class MlpSpec:
    kind: str                      # relu2 | geglu | experts | clampglu
    ff: int                        # hidden size (of one expert)
    experts: int = 0
    top: int = 0
    scale: float = 1.0             # the chosen experts' weights sum to this
    ff_shared: int = 0             # of the expert that every token runs, 0: none
    limit: float = 0.0             # clampglu: bound of both halves
    act: str = "silu_gate"         # experts: silu_gate | relu2
    score: str = "sigmoid"         # experts: sigmoid (renormalised) | softmax (with a correction of the choice)
    groups: int = 0                # experts are chosen from the best `keep_groups` of `groups` equal runs, 0: from all
    keep_groups: int = 0
    identity: int = 0              # router outputs behind the experts' that stand for the row itself


@dataclass
class LayerSpec:
    mixer: MixerSpec
    mlp: Optional[MlpSpec] = None
    weights_of: Optional[int] = None  # the layer whose tensors it uses

    @property
    def ff(self) -> int:
        return self.mlp.ff if self.mlp is not None else 0


def _only(d: dict, known: Tuple[str, ...], what: str) -> None:
    extra = sorted(k for k in set(d) - set(known) if d[k] is not None)
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


def _sink_attention(m: dict) -> MixerSpec:
    """Attention without rotation: unit queries and keys, first tokens kept, sinks, a gate per value, keys and values of another layer."""
    _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask", "kv_from"), "attention mixer")
    mask = m.get("mask") or {}
    _only(mask, ("size", "keep_first"), "mask")
    lender = m.get("kv_from")
    return MixerSpec("attention", m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale=float(m["scale"]), window=int(mask.get("size") or 1 << 30),
                     keep=int(mask.get("keep_first") or 0), unit_qk=True, sink=True, gate_values=True,
                     kv_from=None if lender is None else int(lender))


def _delta(m: dict) -> MixerSpec:
    _only(m, ("heads", "kv_heads", "dim", "vdim", "conv"), "delta mixer")
    return MixerSpec("delta", m["heads"], m["kv_heads"], m["dim"], m["vdim"], taps=int(m["conv"]))


def _gla(m: dict) -> MixerSpec:
    _only(m, ("heads", "dim", "vdim", "tau"), "gla mixer")
    return MixerSpec("gla", m["heads"], m["heads"], m["dim"], m["vdim"], tau=float(m["tau"]))


def _chunk_attention(m: dict) -> MixerSpec:
    """Attention inside chunks of the sequence: no rotation, a distance bias and a learned factor per head, unit values, no gate."""
    _only(m, ("heads", "kv_heads", "dim", "vdim", "scale", "mask"), "attention mixer")
    mask = m.get("mask") or {}
    _only(mask, ("size",), "mask")
    size = mask.get("size")
    return MixerSpec("attention", m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale=float(m["scale"]), window=int(size or 1 << 30),
                     chunked=size is not None, temp=True, bias=True, unit_v=True, gated=False)


def _latent_attention(m: dict) -> MixerSpec:
    """Queries, keys and values through latents; a rotated part of every query and one rotated key part that the heads share; sinks."""
    _only(m, ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "rot", "scale"), "latent attention mixer")
    rot = m["rot"]
    _only(rot, ("base", "dims"), "rotation")
    if int(rot["dims"]) != int(m["rot_dim"]) or int(m["rot_dim"]) % 2:
        raise ValueError(f"latent attention rotates its {m['rot_dim']} rotated dimensions, not {rot['dims']}")
    return MixerSpec("latent", m["heads"], m["heads"], m["dim"], m["vdim"], scale=float(m["scale"]), window=1 << 30, rot_dims=int(rot["dims"]),
                     rot_base=float(rot["base"]), sink=True, gated=False, rot_dim=int(m["rot_dim"]), q_rank=int(m["q_rank"]), kv_rank=int(m["kv_rank"]))


def _wkv(m: dict) -> MixerSpec:
    _only(m, ("heads", "dim"), "wkv mixer")
    return MixerSpec("wkv", m["heads"], m["heads"], m["dim"], m["dim"])


def _halves(m: dict, extra: Tuple[str, ...], scaled: bool, **kw) -> MixerSpec:
    """Attention over every earlier row: biased projections, rotation by halves, values mixed with the first such layer's, no gate."""
    _only(m, ("heads", "kv_heads", "dim", "vdim", "rot", "scale", "v_mix", *extra), "attention mixer")
    rot = m.get("rot") or {"base": 1.0, "dims": 0}
    _only(rot, ("base", "dims", "scaling") if scaled else ("base", "dims"), "rotation")
    if int(rot["dims"]) % 2 or int(rot["dims"]) > int(m["dim"]):
        raise ValueError(f"rotation of {rot['dims']} of {m['dim']} dimensions")
    scaling = rot.get("scaling")
    if scaling is not None:
        _only(scaling, ("factor", "low", "high", "original"), "rotation scaling")
        scaling = tuple(float(scaling[n]) for n in ("factor", "low", "high", "original"))
    return MixerSpec("attention", m["heads"], m["kv_heads"], m["dim"], m["vdim"], scale=float(m["scale"]), window=1 << 30, rot_dims=int(rot["dims"]),
                     rot_base=float(rot["base"]), rot_halves=True, rot_scaling=scaling, biased=True, gated=False, v_mix=bool(m.get("v_mix")), **kw)


def _normed_attention(m: dict) -> MixerSpec:
    """Queries and keys over their root mean square, times a factor per dimension."""
    return _halves(m, (), False, unit_qk=True, qk_norm=True)


def _capped_attention(m: dict) -> MixerSpec:
    """Bounded scores, slow rotations slowed down."""
    return _halves(m, ("softcap",), True, softcap=float(m.get("softcap") or 0.0))


def _ssd(m: dict) -> MixerSpec:
    _only(m, ("heads", "groups", "state", "vdim", "conv", "norm_groups"), "state-space mixer")
    spec = MixerSpec("ssd", m["heads"], m["groups"], m["state"], m["vdim"], taps=int(m["conv"]), norm_groups=int(m["norm_groups"]))
    if spec.norm_groups < 1 or spec.heads * spec.vdim % spec.norm_groups:
        raise ValueError(f"state-space mixer: {spec.norm_groups} groups of {spec.heads * spec.vdim} outputs")
    return spec


def _grouped_experts(d: dict) -> MlpSpec:
    """Softmax scores with corrected choices inside the best groups, squared-ReLU experts, the last router outputs the row itself."""
    _only(d, ("kind", "expert", "router"), "feed-forward")
    _only(d["expert"], ("ff",), "expert")
    r = d["router"]
    _only(r, ("experts", "top", "groups", "identity"), "router")
    g = r.get("groups") or {"count": 1, "keep": 1}
    _only(g, ("count", "keep"), "router groups")
    spec = MlpSpec("experts", int(d["expert"]["ff"]), int(r["experts"]), int(r["top"]), act="relu2", score="softmax", groups=int(g["count"]),
                   keep_groups=int(g["keep"]), identity=int(r.get("identity") or 0))
    total = spec.experts + spec.identity
    if not (spec.groups >= 1 and total % spec.groups == 0 and 1 <= spec.keep_groups <= spec.groups and 1 <= spec.top <= spec.keep_groups * (total // spec.groups)):
        raise ValueError(f"router: {spec.top} of {total} outputs in {spec.keep_groups} of {spec.groups} groups")
    return spec


def _clamped(d: dict) -> MlpSpec:
    _only(d, ("kind", "ff", "limit"), "feed-forward")
    return MlpSpec("clampglu", int(d["ff"]), limit=float(d["limit"]))


def _plain(kind: str) -> Callable[[dict], MlpSpec]:
    def read(d: dict) -> MlpSpec:
        _only(d, ("kind", "ff"), "feed-forward")
        return MlpSpec(kind, int(d["ff"]))

    return read


def _experts(d: dict) -> MlpSpec:
    _only(d, ("kind", "expert", "router", "shared"), "feed-forward")
    _only(d["expert"], ("ff",), "expert")
    _only(d["router"], ("experts", "top", "scale"), "router")
    shared = d.get("shared") or {"ff": 0}
    _only(shared, ("ff",), "shared expert")
    r = d["router"]
    spec = MlpSpec("experts", int(d["expert"]["ff"]), int(r["experts"]), int(r["top"]), float(r.get("scale", 1.0)), int(shared["ff"]))
    if not 1 <= spec.top <= spec.experts:
        raise ValueError(f"router: {spec.top} of {spec.experts} experts")
    return spec


@dataclass(frozen=True)
class Design:
    mixers: Dict[str, Callable[[dict], MixerSpec]]
    mlps: Dict[str, Callable[[dict], MlpSpec]]
    keys: Tuple[str, ...]          # of the configuration, next to the common ones
    norm_add: float = 0.0          # an RMSNorm's scale is norm_add + its weight
    tied: bool = False             # the logits are products with the embedding table
    parallel: bool = False         # mixer and feed-forward read one norm, x += mixer(h) + ff(h); norms in groups
    sandwich: bool = False         # x += post(gate(h) * sublayer(h)), then x becomes an average over depth; the embedding has a norm


DESIGNS = {
    "Sekulorn": Design({"attention": _attention, "delta": _delta, "gla": _gla}, {"dense": _plain("relu2")}, ("loop", "residual_mult")),
    "Kovalorn": Design({"attention": _sink_attention}, {"dense": _plain("geglu"), "moe": _experts}, ("logit_scale",), norm_add=1.0, tied=True),
    "Kudazen": Design({"attention": _chunk_attention, "latent_attention": _latent_attention, "wkv": _wkv}, {"dense": _clamped}, (), tied=True, parallel=True),
    "Gurolix": Design({"mamba2": _ssd, "attention": _normed_attention, "attention_2": _capped_attention}, {"moe": _grouped_experts}, (), norm_add=1.0,
                      sandwich=True),
}


@dataclass
class HybridConfig:
    vocab_size: int
    width: int
    layers: List[LayerSpec]
    eps: float
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    norm_groups: int = 0                    # equal parts of a row that are normalised by themselves (parallel layers)
    loop: Tuple[int, int, int] = (0, 0, 1)  # layers start .. stop - 1 run `times` times in a row
    architecture: str = "Sekulorn"
    block_size: int = 1 << 24               # (positions are not tabulated: nothing limits a sequence but its cache)
    raw: dict = field(default_factory=dict, repr=False)

    @classmethod
    def from_dict(cls, d: dict) -> "HybridConfig":
        name = d.get("architecture", "Sekulorn")
        if name not in DESIGNS:
            raise ValueError(f"unknown design {name!r} (known: {sorted(DESIGNS)})")
        design = DESIGNS[name]
        _only(d, ("architecture", "vocab", "width", "layers", "norm", *design.keys), "configuration")
        _only(d["norm"], ("eps", "groups") if design.parallel else ("eps",), "norm")
        groups = int(d["norm"].get("groups") or 1) if design.parallel else 0
        if groups and (groups < 0 or int(d["width"]) % groups):
            raise ValueError(f"norm: {groups} groups of a row of {d['width']}")
        layers: List[LayerSpec] = []
        for e in d["layers"]:
            _only(e, ("type", "mixer", "mlp", "weights_of") if design.parallel else ("type", "mixer", "mlp"), "layer")
            if e["type"] not in design.mixers:
                raise ValueError(f"unknown mixer {e['type']!r} (known: {sorted(design.mixers)})")
            mlp = e.get("mlp")
            if mlp is not None and mlp["kind"] not in design.mlps:
                raise ValueError(f"unknown feed-forward {mlp['kind']!r} (known: {sorted(design.mlps)})")
            spec = design.mixers[e["type"]](e["mixer"])
            if spec.heads % spec.kv_heads:
                raise ValueError(f"{spec.heads} heads over {spec.kv_heads} key / value heads")
            if spec.kv_from is not None:
                own = layers[spec.kv_from].mixer if 0 <= spec.kv_from < len(layers) else None
                if own is None or own.type != "attention" or own.kv_from is not None:
                    raise ValueError(f"layer {len(layers)}: layer {spec.kv_from} in front of it has no keys of its own")
                if (own.kv_heads, own.dim, own.vdim) != (spec.kv_heads, spec.dim, spec.vdim):
                    raise ValueError(f"layer {len(layers)}: the keys and values of layer {spec.kv_from} have other sizes")
            layers.append(LayerSpec(spec, design.mlps[mlp["kind"]](mlp) if mlp is not None else None, e.get("weights_of")))
        for i, l in enumerate(layers):
            if l.weights_of is not None:
                own = layers[l.weights_of] if 0 <= l.weights_of < len(layers) else None
                if own is None or own.weights_of is not None:
                    raise ValueError(f"layer {i}: layer {l.weights_of} has no tensors of its own")
                if (own.mixer, own.mlp) != (l.mixer, l.mlp):
                    raise ValueError(f"layer {i} differs from layer {l.weights_of}, whose weights it uses")
        mixed = [(i, l.mixer) for i, l in enumerate(layers) if l.mixer.v_mix]
        for i, m in mixed:
            if (m.kv_heads, m.vdim) != (mixed[0][1].kv_heads, mixed[0][1].vdim):
                raise ValueError(f"layer {i} mixes values of other sizes than layer {mixed[0][0]}'s")
        loop = d.get("loop")
        if loop is not None:
            _only(loop, ("start", "stop", "times"), "loop")
            span = (int(loop["start"]), int(loop["stop"]), int(loop["times"]))
            if not (0 <= span[0] <= span[1] <= len(layers) and span[2] >= 1):
                raise ValueError(f"bad loop {span} over {len(layers)} layers")
        return cls(int(d["vocab"]), int(d["width"]), layers, float(d["norm"]["eps"]), float(d.get("residual_mult", 1.0)),
                   float(d.get("logit_scale", 1.0)), groups, span if loop is not None else (0, 0, 1), name, raw=d)

    @property
    def design(self) -> Design:
        return DESIGNS[self.architecture]

    @property
    def padded_vocab_size(self) -> int:
        return self.vocab_size

    def runs(self) -> List[int]:
        """The layer of every run, in order: a looped layer appears once per pass."""
        a, b, times = self.loop
        return [*range(a), *(list(range(a, b)) * times), *range(b, len(self.layers))]

    def first_values(self) -> Optional[int]:
        """The layer whose values the others that mix them read."""
        return next((i for i, l in enumerate(self.layers) if l.mixer.v_mix), None)

    def lenders(self) -> List[Optional[int]]:
        """Per run, the run whose keys and values it reads (the last one of its lender so far), None: its own."""
        last: Dict[int, int] = {}
        out: List[Optional[int]] = []
        for r, i in enumerate(self.runs()):
            j = self.layers[i].mixer.kv_from
            out.append(None if j is None else last[j])
            last[i] = r
        return out


def projections(m: MixerSpec) -> Tuple[str, ...]:
    """The pieces of a mixer's stacked input projection, in the order of their columns."""
    if m.type == "attention":
        return ("q", *(("k", "v") if m.kv_from is None else ()), *(("g",) if m.gated else ()))
    if m.type == "latent":
        return ("dq", "dkv")
    if m.type == "wkv":
        return ("r", "k", "v", "g", "w1")  # (each reads a mix of its own)
    if m.type == "ssd":
        return ("z", "x", "B", "C", "dt")  # (the rows of one tensor, `in`)
    return ("q", "k", "v", "g", "a", "b") if m.type == "delta" else ("q", "k", "v", "g", "a1")


def tensor_shapes(cfg: HybridConfig, rank: Dict[int, int]) -> Dict[str, Tuple[int, ...]]:
    """name -> shape of every tensor of a checkpoint; rank[i]: the low-rank size of gla or wkv layer i (only its tensors know it)."""
    W = cfg.width
    out = {"embed": (cfg.vocab_size, W)}
    sandwich = cfg.design.sandwich
    if sandwich:
        out["embed.norm"] = (W,)

    def gated(p: str, ff: int) -> None:
        out.update({p + "gate": (ff, W), p + "up": (ff, W), p + "down": (W, ff)})

    for i, l in enumerate(cfg.layers):
        if l.weights_of is not None:
            continue
        p, m = f"l{i}.", l.mixer
        hv, gk = m.heads * m.vdim, m.kv_heads * m.dim
        out[p + "norm1"] = (W,)
        x = p + "mix."
        if m.type == "attention":
            out[x + "q"] = (m.heads * m.dim, W)
            if m.kv_from is None:
                out.update({x + "k": (gk, W), x + "v": (m.kv_heads * m.vdim, W)})
            if m.sink:
                out[x + "sink"] = (m.heads,)
            if m.gated:
                out[x + "g"] = (hv if m.gate_values else m.heads, W)
            if m.temp:
                out[x + "temp"] = (m.heads,)
            if m.biased:
                out.update({x + "q.b": (m.heads * m.dim,), x + "k.b": (gk,), x + "v.b": (m.kv_heads * m.vdim,)})
            if m.qk_norm:
                out.update({x + "q.norm": (m.dim,), x + "k.norm": (m.dim,)})
            if m.v_mix:
                out[x + "vmix"] = ()
        elif m.type == "ssd":
            n = hv + 2 * gk
            out.update({x + "in": (hv + n + m.heads, W), x + "conv": (n, m.taps), x + "conv.b": (n,), x + "dt_bias": (m.heads,), x + "A_log": (m.heads,),
                        x + "D": (m.heads,), x + "norm": (hv,)})
        elif m.type == "latent":
            out.update({x + "dq": (m.q_rank, W), x + "dq.norm": (m.q_rank,), x + "uq": (m.heads * (m.dim + m.rot_dim), m.q_rank),
                        x + "dkv": (m.kv_rank + m.rot_dim, W), x + "dkv.norm": (m.kv_rank,), x + "uk": (gk, m.kv_rank), x + "uv": (hv, m.kv_rank),
                        x + "sink": (m.heads,)})
        elif m.type == "wkv":
            out.update({x + f"mu.{s}": (W,) for s in "rkvgw"})
            out.update({x + s: (hv, W) for s in "rkvg"})
            out.update({x + "w1": (rank[i], W), x + "w2": (hv, rank[i]), x + "w0": (hv,), x + "u": (m.heads, m.dim), x + "norm": (hv,)})
        else:
            out.update({x + "q": (gk, W), x + "k": (gk, W), x + "v": (hv, W), x + "g": (hv, W), x + "norm": (m.vdim,)})
        if m.type == "delta":
            out.update({x + "q.conv": (gk, m.taps), x + "k.conv": (gk, m.taps), x + "v.conv": (hv, m.taps), x + "b": (m.heads, W),
                        x + "a": (m.heads, W), x + "A_log": (m.heads,), x + "dt_bias": (m.heads,)})
        if m.type == "gla":
            out.update({x + "a1": (rank[i], W), x + "a2": (gk, rank[i]), x + "a2.b": (gk,)})
        out[x + "o"] = (W, hv)
        f = l.mlp
        if sandwich:
            out.update({p + "norm1b": (W,), p + "rg1": (W, W), p + "rg1.b": (W,), p + "dwa": (i + 2,)})
            if f is not None:
                out.update({p + "norm2b": (W,), p + "rg2": (W, W), p + "rg2.b": (W,)})
        if f is not None:
            if not cfg.design.parallel:
                out[p + "norm2"] = (W,)
            if f.kind == "relu2":
                out.update({p + "mlp.up": (f.ff, W), p + "mlp.down": (W, f.ff)})
            elif f.kind in ("geglu", "clampglu"):
                gated(p + "mlp.", f.ff)
            else:
                out[p + "mlp.router"] = (f.experts + f.identity, W)
                if f.score == "softmax":
                    out[p + "mlp.correction"] = (f.experts + f.identity,)
                for e in range(f.experts):
                    if f.act == "relu2":
                        out.update({f"{p}mlp.e{e}.up": (f.ff, W), f"{p}mlp.e{e}.down": (W, f.ff)})
                    else:
                        gated(f"{p}mlp.e{e}.", f.ff)
                if f.ff_shared:
                    gated(p + "mlp.shared.", f.ff_shared)
    out["final.norm"] = (W,)
    if not cfg.design.tied:
        out["head"] = (cfg.vocab_size, W)
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
        low = {"gla": "a1", "wkv": "w1"}
        rank = {i: sd[n].shape[0] for i, l in enumerate(self.config.layers) for n in (f"l{i}.mix.{low.get(l.mixer.type)}",) if n in sd}
        shapes = tensor_shapes(self.config, {**{i: 0 for i in range(len(self.config.layers))}, **rank})
        first = self.config.first_values()
        idle = {f"l{i}.mix.vmix" for i, l in enumerate(self.config.layers) if l.mixer.type == "attention" and (not l.mixer.v_mix or i == first)}
        shapes = {n: s for n, s in shapes.items() if n not in idle or n in sd}  # (nobody reads these factors: they may be there or not)
        missing, extra = sorted(set(shapes) - set(sd)), sorted(set(sd) - set(shapes) - idle)
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
