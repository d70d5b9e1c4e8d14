"""Native engine of a layered hybrid model: descriptors, slots of state, steps over packed batches.

`step(entries)` is the one way tokens get in: every entry is a slot, the position its first new token has and the tokens; rows of all
entries are packed without padding and run through `mi355_hybrid_forward` once (a step with more rows than the scratch holds is cut).
A decode step (one token per entry) is replayed as a hipGraph per batch size.  `generate()` drives the engine through the same
attributes and methods as `engine.DecodeEngine` (`_ensure_cache`, `prefill`, `set_step`, `run_step`, ...).
"""
from __future__ import annotations

import ctypes as C
import gc
import math
import os
import weakref
from typing import Dict, List, NamedTuple, Optional, Sequence, Tuple

import torch

from . import _native as nat
from . import ops
from ._native import ExpertsArgs, HybridLayer, HybridModel, Proj, SeqBatch, check, lib, ptr
from .hybrid import HybridLM, LayerSpec, MixerSpec, MlpSpec, projections
from .state import SlotManager, grown

MIX = {"attention": 0, "delta": 1, "gla": 2, "wkv": 3, "latent": 4, "ssd": 5}
MLP = {"relu2": 1, "geglu": 2, "experts": 3, "clampglu": 4}
KV_OWN, KV_LENDS, KV_BORROWS = 0, 1, 2
REC_DELTA, REC_GLA, REC_WKV, REC_SSD = 0, 1, 2, 3
REC = {MIX["delta"]: REC_DELTA, MIX["gla"]: REC_GLA, MIX["wkv"]: REC_WKV, MIX["ssd"]: REC_SSD}
SCORE = {"sigmoid": 0, "softmax": 1}
ACT = {"silu_gate": 0, "relu2": 1}
LATENT_RECORDS = 64 << 20  # bytes of softmax records of a latent attention's key splits


class Entry(NamedTuple):
    """New tokens of one sequence: `want` = the places among them whose logits are asked for."""

    slot: int
    pos: int
    tokens: Sequence[int]
    want: Sequence[int]


def _pad16(n: int) -> int:
    return (n + 15) // 16 * 16


def _pad128(n: int) -> int:
    return (n + 127) // 128 * 128


def _slowed(f: float, factor: float, low: float, high: float, original: float) -> float:
    """A rotation's turns per position for longer contexts: those with more than `high` full turns in the original length stay, those with fewer
    than `low` are divided by `factor`, in between the two are mixed."""
    turns = original * f / (2 * math.pi)
    if turns > high:
        return f
    if turns < low:
        return f / factor
    keep = (turns - low) / (high - low)
    return (1 - keep) * f / factor + keep * f


class HybridEngine:
    supports_batches = True

    def __init__(self, model: HybridLM, *, max_rows: Optional[int] = None):
        # (the weights, not the model: the model owns its engine, and a cycle would leave both to the garbage collector)
        self.weights, self.cfg, self.device = model.tensors, model.config, model.device
        self.dtype = model.dtype
        self.max_rows = max_rows or int(os.environ.get("MI355_HYBRID_ROWS", "4096"))
        self.use_graph = os.environ.get("MI355_HYBRID_GRAPH", "1") != "0"
        self.stream = torch.cuda.Stream(self.device)
        self._keep: List[torch.Tensor] = []
        self._graphs: Dict[tuple, C.c_void_p] = {}
        self._warm: set = set()
        self.max_len = 0            # longest sequence the rings are sized for
        with torch.cuda.device(self.device), torch.cuda.stream(self.stream):
            self.stream.wait_stream(torch.cuda.default_stream(self.device))
            self._pack()
            self._scratch()
        grow = weakref.WeakMethod(self._grow)
        self.slots = SlotManager(lambda n: grow()(n))
        self._single: Optional[int] = None  # generate()'s slot
        self.stream.synchronize()

    # ---- weights ---------------------------------------------------------------------------------------
    def _own(self, w: torch.Tensor) -> int:
        self._keep.append(w)
        self.weight_bytes += w.numel() * w.element_size()
        return ptr(w)

    def _stream(self, w: torch.Tensor, pair: Optional[torch.Tensor] = None) -> torch.Tensor:
        """What the products read of a weight [N, K] or of a pair of them."""
        if self.dtype == torch.bfloat16:
            return ops.repack_bf16(w, pair, 1 if pair is None else 2)
        return (w if pair is None else torch.cat([w, pair])).contiguous()

    def _proj(self, w: torch.Tensor, pair: Optional[torch.Tensor] = None, bias: Optional[torch.Tensor] = None) -> Proj:
        """A weight [N, K] with its rows padded to a multiple of 16 (zero rows: the padding columns of every buffer stay zero)."""
        N, K = w.shape
        if bias is not None:
            bias = torch.nn.functional.pad(bias.float(), (0, _pad16(N) - N))
        n = _pad16(N)
        if n != N:
            w, pair = (t if t is None else torch.cat([t, t.new_zeros((n - N, K))]) for t in (w, pair))
        return Proj(self._own(self._stream(w, pair)), n, K, None if bias is None else self._f32(bias))

    def _norm(self, name: str) -> int:
        """A norm's weight; f32 models hold what is multiplied by, bf16 models the stored weight (their kernels add norm_add)."""
        w = self.weights[name]
        return ptr(w) if self.dtype == torch.bfloat16 or not self.cfg.design.norm_add else self._f32(w.float() + self.cfg.design.norm_add)

    def _experts(self, i: int, f: MlpSpec) -> ExpertsArgs:
        p = f"l{i}.mlp."
        T, a = self.weights, ExpertsArgs()
        a.dtype, a.width, a.experts, a.top = nat.dtype_code(self.dtype), self.cfg.width, f.experts, f.top
        a.ff, a.ff_shared, a.scale = f.ff, f.ff_shared, f.scale
        a.score, a.act, a.identity, a.groups, a.keep_groups = SCORE[f.score], ACT[f.act], f.identity, f.groups, f.keep_groups
        if f.score == "softmax":
            a.correction = self._f32(T[p + "correction"])
        if not self.cfg.design.sandwich:
            a.router = self._own(self._stream(T[p + "router"]))
        if f.act == "relu2":
            up = [self._stream(T[f"{p}e{e}.up"]) for e in range(f.experts)]
        else:
            up = [self._stream(T[f"{p}e{e}.gate"], T[f"{p}e{e}.up"]) for e in range(f.experts)]
        before = self.weight_bytes
        a.up = self._own(torch.stack(up))
        a.down = self._own(torch.stack([self._stream(T[f"{p}e{e}.down"]) for e in range(f.experts)]))
        self._expert_bytes[i] = (self.weight_bytes - before) / f.experts
        if f.ff_shared:
            a.shared_up = self._own(self._stream(T[p + "shared.gate"], T[p + "shared.up"]))
            a.shared_down = self._own(self._stream(T[p + "shared.down"]))
        return a

    def _f32(self, t: torch.Tensor) -> int:
        t = t.detach().float().contiguous()
        self._keep.append(t)
        return ptr(t)

    def _pack(self) -> None:
        cfg, T = self.cfg, self.weights
        self.weight_bytes = 0
        self._expert_bytes: Dict[int, float] = {}
        self.norm_dtype = nat.dtype_code(self.dtype)
        layers: List[Optional[HybridLayer]] = []
        self._cats: Dict[tuple, int] = {}
        for i, spec in enumerate(cfg.layers):
            if spec.weights_of is not None:
                layers.append(None)
                continue
            m, p = spec.mixer, f"l{i}."
            x = p + "mix."
            L = HybridLayer()
            L.mixer, L.mlp = MIX[m.type], MLP[spec.mlp.kind] if spec.mlp is not None else 0
            L.norm1 = self._norm(p + "norm1")
            # one stacked projection, every piece padded to 16 columns
            off, parts = {}, []
            weights, biases = self._pieces(x, m)
            for name, w in zip(projections(m), weights):
                off[name] = sum(q.shape[0] for q in parts)
                pad = _pad16(w.shape[0]) - w.shape[0]
                parts.append(torch.cat([w, w.new_zeros((pad, w.shape[1]))]) if pad else w)
            if m.type == "wkv":
                self._token_shift(L, x, parts, off)
            elif cfg.design.sandwich:
                self._sandwich(L, p, spec, parts, biases)
            else:
                setattr(L, "in", self._proj(torch.cat(parts)))
            if cfg.design.parallel:
                self._parallel(L, p, spec)
            elif not cfg.design.sandwich:
                L.out = self._proj(T[x + "o"])
            if spec.mlp is not None and not cfg.design.parallel:
                L.norm2 = self._norm(p + "norm2")
                if spec.mlp.kind == "experts":
                    L.moe = self._experts(i, spec.mlp)
                else:
                    L.up = self._proj(T[p + "mlp.gate"], T[p + "mlp.up"]) if spec.mlp.kind == "geglu" else self._proj(T[p + "mlp.up"])
                    L.down = self._proj(T[p + "mlp.down"])
            if m.type == "attention":
                a = L.attn
                a.heads, a.kv_heads, a.dim, a.vdim = m.heads, m.kv_heads, m.dim, m.vdim
                a.off_q, a.off_k, a.off_v, a.off_g = off["q"], off.get("k", 0), off.get("v", 0), off.get("g", -1)
                a.scale, a.window, a.rot_dims, a.keep = m.scale, m.window, m.rot_dims, m.keep
                a.gate_values, a.unit_qk, a.unit_eps = int(m.gate_values), int(m.unit_qk), cfg.eps
                a.chunked, a.unit_v = int(m.chunked), int(m.unit_v)
                if m.sink:
                    a.sink = self._f32(T[x + "sink"])
                if m.temp:
                    a.head_scale = self._f32(T[x + "temp"])
                if m.bias:
                    a.slope = self._f32(torch.tensor([2.0 ** (-8.0 * (h + 1) / m.heads) for h in range(m.heads)], dtype=torch.float64, device=self.device))
                if m.rot_dims:
                    a.inv_freq = self._inv_freq(m)
                a.softcap = m.softcap
                if m.qk_norm:
                    turn = self._turned(m)
                    a.q_norm, a.k_norm = (self._f32(T[x + n][turn]) for n in ("q.norm", "k.norm"))
                if m.v_mix and i != cfg.first_values():
                    a.v_mix = float(T[x + "vmix"])
            elif m.type == "latent":
                self._latent(L, x, m, off)
            else:
                r = L.rec
                r.kind = REC[L.mixer]
                r.heads, r.kv_heads, r.dim, r.vdim = m.heads, m.kv_heads, m.dim, m.vdim
                names = {"wkv": "rkvg", "ssd": "CBxz"}.get(m.type, "qkvg")
                r.off_q, r.off_k, r.off_v, r.off_g = (off[n] for n in names)
                r.q_scale, r.eps, r.unit_eps = m.dim ** -0.5, cfg.eps, 1e-6
                if m.type != "ssd":
                    r.head_norm = self._f32(T[x + "norm"])
                if m.type == "ssd":
                    self._state_space(r, x, m, off)
                elif m.type == "wkv":
                    r.q_scale, r.norm_ld, r.bonus = 1.0, m.vdim, self._f32(T[x + "u"])
                    r.off_a, r.rank = off["w1"], T[x + "w1"].shape[0]
                    r.a2, r.a2_bias = self._f32(T[x + "w2"]), self._f32(T[x + "w0"])
                elif m.type == "delta":
                    r.off_a, r.off_b, r.taps = off["a"], off["b"], m.taps
                    r.conv_q, r.conv_k, r.conv_v = (self._f32(T[x + n + ".conv"]) for n in "qkv")
                    r.a_log, r.dt_bias = self._f32(T[x + "A_log"]), self._f32(T[x + "dt_bias"])
                else:
                    r.off_a, r.rank, r.inv_tau = off["a1"], T[x + "a1"].shape[0], 1.0 / m.tau
                    r.a2, r.a2_bias = self._f32(T[x + "a2"]), self._f32(T[x + "a2.b"])
            layers.append(L)
        layers = [layers[spec.weights_of if l is None else i] for i, (l, spec) in enumerate(zip(layers, cfg.layers))]
        runs = cfg.runs()
        self.run_layers = runs
        self.layers = (HybridLayer * max(1, len(runs)))()
        for r, i in enumerate(runs):
            C.memmove(C.byref(self.layers[r]), C.byref(layers[i]), C.sizeof(HybridLayer))
            self.layers[r].kv_lender = self.layers[r].kv_last = -1
        # a lender's cache covers the windows and the first tokens of all that read it
        self.lenders = cfg.lenders()
        self.spans = [(1 << 30, 0) if l.mixer == MIX["latent"] else (l.attn.window, l.attn.keep) for l in self.layers[: len(runs)]]
        for r, j in enumerate(self.lenders):
            if j is not None:
                self.layers[r].kv_lender, self.layers[j].kv_last = j, r
                self.layers[r].attn.role, self.layers[j].attn.role = KV_BORROWS, KV_LENDS
                self.spans[j] = tuple(map(max, self.spans[j], self.spans[r]))
        first = cfg.first_values()
        if first is not None and first in runs:  # (its projections outlive the layer: the others read its values from them)
            lender, own = self.layers[runs.index(first)], getattr(layers[first], "in")
            self._first_rows = self._buf(self.max_rows * own.N, self.dtype)
            lender.proj_rows = ptr(self._first_rows)
            for r, i in enumerate(runs):
                if cfg.layers[i].mixer.v_mix and i != first:
                    a = self.layers[r].attn
                    a.v_first = lender.proj_rows + lender.attn.off_v * self._first_rows.element_size()
                    a.ld_v_first = own.N
        M = self.m = HybridModel()
        M.n_runs, M.dtype, M.norm_dtype = len(runs), nat.dtype_code(self.dtype), self.norm_dtype
        M.width, M.ldx, M.vocab, M.max_rows = cfg.width, _pad16(cfg.width), cfg.vocab_size, self.max_rows
        M.eps, M.residual_mult, M.logit_scale = cfg.eps, cfg.residual_mult, cfg.logit_scale
        M.norm_groups, M.ld_n = cfg.norm_groups, _pad128(cfg.width)
        M.norm_add = cfg.design.norm_add if self.dtype == torch.bfloat16 else 0.0
        M.embed, M.final_norm = ptr(T["embed"]), self._norm("final.norm")
        M.head = self._proj(T["embed" if cfg.design.tied else "head"])
        M.ld_logits = M.head.N
        M.layers = self.layers
        if cfg.design.sandwich:
            M.embed_norm = self._norm("embed.norm")
        self.n_logits = cfg.vocab_size

    def _inv_freq(self, m: MixerSpec) -> int:
        f = [m.rot_base ** (-2.0 * j / m.rot_dims) for j in range(m.rot_dims // 2)]
        if m.rot_scaling is not None:
            f = [_slowed(v, *m.rot_scaling) for v in f]
        t = torch.tensor(f, dtype=torch.float64, device=self.device)
        self._keep.append(t)
        return ptr(t)

    def _turned(self, m: MixerSpec) -> torch.Tensor:
        """Dimensions of a head in the kernels' order: the kernels turn neighbours, so the two halves are dealt out in turn.  Products of
        queries and keys do not see the order."""
        half = torch.arange(m.rot_dims // 2, device=self.device)
        return torch.cat([torch.stack([half, half + m.rot_dims // 2], 1).flatten(), torch.arange(m.rot_dims, m.dim, device=self.device)])

    def _pieces(self, x: str, m: MixerSpec) -> Tuple[List[torch.Tensor], Optional[List[torch.Tensor]]]:
        """Weights and biases of a mixer's input projections, in the order of `projections`."""
        T = self.weights
        if m.type == "ssd":
            hv, gk = m.heads * m.vdim, m.kv_heads * m.dim
            return list(T[x + "in"].split([hv, hv, gk, gk, m.heads])), None
        ws = [T[x + n] for n in projections(m)]
        bs = [T[x + n + ".b"] for n in projections(m)] if m.biased else None
        if m.type == "attention" and m.rot_halves and m.rot_dims:
            turn = self._turned(m)
            for j, n in enumerate(projections(m)):
                if n in ("q", "k"):
                    ws[j] = ws[j].view(-1, m.dim, ws[j].shape[1])[:, turn].reshape(ws[j].shape)
                    if bs is not None:
                        bs[j] = bs[j].view(-1, m.dim)[:, turn].reshape(-1)
        return ws, bs

    def _state_space(self, r, x: str, m: MixerSpec, off: Dict[str, int]) -> None:
        T = self.weights
        hv, gk = m.heads * m.vdim, m.kv_heads * m.dim
        r.q_scale, r.off_a, r.taps = 1.0, off["dt"], m.taps
        r.conv_v, r.conv_k, r.conv_q = (self._f32(t) for t in T[x + "conv"].split([hv, gk, gk]))
        r.conv_bv, r.conv_bk, r.conv_bq = (self._f32(t) for t in T[x + "conv.b"].split([hv, gk, gk]))
        r.a_log, r.dt_bias, r.skip = (self._f32(T[x + n]) for n in ("A_log", "dt_bias", "D"))

    def _sandwich(self, L: HybridLayer, p: str, spec: LayerSpec, parts: List[torch.Tensor], biases: Optional[List[torch.Tensor]]) -> None:
        """Sublayers between norms: the mixer's gate is one more piece of its input projection; the feed-forward's stands in a product with the router."""
        T, W = self.weights, self.cfg.width
        n = sum(w.shape[0] for w in parts)
        bias = torch.zeros(n, device=self.device)
        at = 0
        for w, b in zip(parts, biases or ()):
            bias[at:at + b.shape[0]] = b.float()
            at += w.shape[0]
        L.sandwich, L.gate_at = 1, n
        setattr(L, "in", self._proj(torch.cat([*parts, T[p + "rg1"]]), bias=torch.cat([bias, T[p + "rg1.b"].float()])))
        L.out = self._proj(T[p + "mix.o"])
        L.ld_cat = _pad128(L.out.K)
        key = (L.out.K, L.out.K)  # rows of one length share their buffer: the padding behind them stays zero
        if key not in self._cats:
            self._cats[key] = ptr(self._buf(self.max_rows * L.ld_cat, self.dtype))
        L.cat = self._cats[key]
        L.post1, L.average = self._norm(p + "norm1b"), self._f32(T[p + "dwa"])
        if spec.mixer.type == "ssd":
            L.out_norm, L.out_groups = ptr(T[p + "mix.norm"]), spec.mixer.norm_groups
        if spec.mlp is not None:
            pad = _pad16(W) - W
            gate = torch.nn.functional.pad(T[p + "rg2"], (0, 0, 0, pad))
            L.side = self._proj(torch.cat([gate, T[p + "mlp.router"]]),
                                bias=torch.cat([T[p + "rg2.b"].float(), torch.zeros(pad + T[p + "mlp.router"].shape[0], device=self.device)]))
            L.logits_at, L.post2 = W + pad, self._norm(p + "norm2b")

    def _token_shift(self, L: HybridLayer, x: str, parts: List[torch.Tensor], off: Dict[str, int]) -> None:
        """Input projections that read a mix of their own each; bf16: those of one size as one stream, where its parts are whole tiles."""
        T, names = self.weights, projections(MixerSpec("wkv", 1, 1, 1, 1))
        L.n_mix = len(names)
        L.mu = self._f32(torch.stack([T[f"{x}mu.{s[0]}"] for s in names]))
        n = sum(1 for w in parts if w.shape == parts[0].shape)
        stack = self.dtype == torch.bfloat16 and all(w.shape == parts[0].shape for w in parts[:n]) and n > 1
        if stack:
            L.mix_w[0] = self._proj(torch.cat(parts[:n]))
            L.mix_stacked = n
        for i, (s, w) in enumerate(zip(names, parts)):
            L.mix_at[i] = off[s]
            if not stack or i >= n:
                L.mix_w[i] = self._proj(w)
        setattr(L, "in", Proj(None, sum(w.shape[0] for w in parts), self.cfg.width))

    def _parallel(self, L: HybridLayer, p: str, spec: LayerSpec) -> None:
        """Feed-forward beside the mixer: its gate / up pair, and one output weight over the row [mixer | hidden]."""
        T = self.weights
        o = T[p + "mix.o"]
        pad = lambda w: torch.nn.functional.pad(w, (0, _pad16(w.shape[1]) - w.shape[1]))
        L.parallel, L.hid_at = 1, _pad16(o.shape[1])
        if spec.mlp is not None:
            L.up = self._proj(T[p + "mlp.gate"], T[p + "mlp.up"])
            L.limit = spec.mlp.limit
            o = torch.cat([pad(o), pad(T[p + "mlp.down"])], 1)
        L.out = self._proj(o)
        L.ld_cat = _pad128(L.out.K)
        key = (T[p + "mix.o"].shape[1], L.out.K)  # layers of one layout share their rows: what no layer writes stays zero
        if key not in self._cats:
            self._cats[key] = ptr(self._buf(self.max_rows * L.ld_cat, self.dtype))
        L.cat = self._cats[key]

    def _latent(self, L: HybridLayer, x: str, m: MixerSpec, off: Dict[str, int]) -> None:
        T, a = self.weights, L.latent
        a.heads, a.dim, a.rot_dim, a.vdim, a.q_rank, a.kv_rank = m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank
        a.off_q, a.off_c, a.scale, a.eps = off["dq"], off["dkv"], m.scale, self.cfg.eps
        a.q_norm, a.c_norm, a.sink = (self._f32(T[x + n]) for n in ("dq.norm", "dkv.norm", "sink"))
        a.inv_freq = self._inv_freq(m)
        a.uq = self._proj(T[x + "uq"])
        uk, uv = T[x + "uk"], T[x + "uv"]
        a.uk_t = self._own(uk.view(m.heads, m.dim, m.kv_rank).transpose(1, 2).contiguous())
        a.uv = self._own(uv.contiguous())
        if self.dtype == torch.bfloat16:
            before = self.weight_bytes  # (a second form of the same weights, for prompts)
            rows = lambda w: torch.nn.functional.pad(w, (0, 0, 0, _pad16(w.shape[0]) - w.shape[0]))
            a.expand = self._proj(torch.cat([rows(uk), rows(uv)]))
            self.weight_bytes = before

    def _latent_scratch(self) -> None:
        """Rows of a step and of a sequence's expanded keys and values, shared by the latent attentions of all runs."""
        ls = [l.latent for l in list(self.layers)[: self.m.n_runs] if l.mixer == MIX["latent"]]
        if not ls:
            return
        R, f32 = self.max_rows, self.dtype == torch.float32
        cq = self._buf(R * max(_pad128(a.q_rank) for a in ls), self.dtype)
        q = self._buf(R * max(a.uq.N for a in ls), self.dtype)
        qa = self._buf(R * max(a.heads * (a.kv_rank + a.rot_dim) for a in ls), self.dtype)
        n = max(LATENT_RECORDS, max(a.heads * (a.kv_rank + 4) * 4 for a in ls))
        rec = self._buf(n // 4, torch.float32)
        for r in range(self.m.n_runs):
            a = self.layers[r].latent
            if self.layers[r].mixer == MIX["latent"]:
                a.cq, a.q, a.qa, a.partials, a.partials_bytes = ptr(cq), ptr(q), ptr(qa), ptr(rec), n

    def _expand_scratch(self) -> None:
        """bf16: room for the keys and values of every position of a sequence (grows with the longest one)."""
        ls = [l.latent for l in list(self.layers)[: self.m.n_runs] if l.mixer == MIX["latent"]]
        rows = max(self.max_rows, self.max_len)
        if not ls or self.dtype == torch.float32 or rows <= getattr(self, "_expand_rows", 0):
            return
        new = lambda n, dtype=self.dtype: torch.zeros(n, dtype=dtype, device=self.device)
        ws = int(lib().mi355_linear_gemm_workspace_bytes(rows, max(_pad128(a.kv_rank) for a in ls)))
        self._expand = [new(rows * max(_pad128(a.kv_rank) for a in ls)), new(rows * max(a.expand.N for a in ls))]
        if ws > self.m.gemm_ws_bytes:
            self._expand.append(new(ws, torch.uint8))
            self.m.gemm_ws, self.m.gemm_ws_bytes = ptr(self._expand[2]), ws
        for r in range(self.m.n_runs):
            if self.layers[r].mixer == MIX["latent"]:
                a = self.layers[r].latent
                a.rows_c, a.kv_rows, a.expand_rows = ptr(self._expand[0]), ptr(self._expand[1]), rows
        self._expand_rows = rows

    def _buf(self, n: int, dtype: torch.dtype) -> torch.Tensor:
        t = torch.zeros(max(1, n), dtype=dtype, device=self.device)
        self._keep.append(t)
        return t

    def _scratch(self) -> None:
        M, R, cfg = self.m, self.max_rows, self.cfg
        ls = list(self.layers)[: M.n_runs]
        self.x = self._buf(R * M.ldx, torch.float32)
        M.x, M.xw = ptr(self.x), ptr(self._buf(R * M.ldx, torch.float32))
        M.ld_att = max([_pad16(l.out.K) for l in ls], default=16)
        M.proj = ptr(self._buf(R * max([getattr(l, "in").N for l in ls], default=16), self.dtype))
        M.att = ptr(self._buf(R * M.ld_att, self.dtype))
        f32 = self.dtype == torch.float32
        M.hid = ptr(self._buf(R * max([l.up.N * (3 if f32 and l.mlp in (MLP["geglu"], MLP["clampglu"]) else 1) for l in ls], default=16), self.dtype))
        sandwich = cfg.design.sandwich
        if f32 or sandwich:
            M.tmp = ptr(self._buf(R * M.ldx, torch.float32))
        if sandwich:
            M.stream = ptr(self._buf((M.n_runs + 1) * R * M.ldx, torch.float32))
            M.ld_side = max([l.side.N for l in ls], default=16)
            M.side = ptr(self._buf(R * M.ld_side, torch.float32))
            M.ld_mixed = max([_pad16(l.out.K) for l in ls if l.mixer == MIX["ssd"]], default=16)
            M.mixed = ptr(self._buf(R * M.ld_mixed if any(l.mixer == MIX["ssd"] for l in ls) else 1, torch.float32))
        if f32:
            M.xn = ptr(self._buf(R * M.ld_n, torch.float32))
        else:
            K = max([M.head.K] + [q.K for l in ls for q in (getattr(l, "in"), l.out, l.up, l.down, l.latent.uq, l.side)])  # (K = 0: not there)
            n = int(lib().mi355_linear_gemm_workspace_bytes(R, _pad128(K)))
            M.gemm_ws, M.gemm_ws_bytes = ptr(self._buf(n, torch.uint8)), n
            M.xb = ptr(self._buf(R * M.ld_n, torch.bfloat16))
        M.mix = ptr(self._buf((R * M.ld_n + 1152) * max([l.n_mix for l in ls], default=0), self.dtype))
        self._latent_scratch()
        # a split attention step keeps one record per (row, head, split); one split takes none
        n = max([512 * (l.attn.vdim + 2) * max(8, l.attn.heads // l.attn.kv_heads) for l in ls if l.mixer == 0], default=0)
        M.partials, M.partials_bytes = ptr(self._buf(n, torch.float32)), n * 4
        n = max([int(lib().mi355_recurrent_scratch_bytes(l.rec.kind, R, 64, l.rec.heads, l.rec.kv_heads, l.rec.dim, l.rec.vdim))
                 for l in ls if l.mixer in REC], default=0)
        M.rec_scratch, M.rec_scratch_bytes = ptr(self._buf(n, torch.uint8)), n
        n = 0
        for l in ls:
            if l.mlp == MLP["experts"]:
                a = ExpertsArgs.from_buffer_copy(l.moe)
                a.rows = R
                n = max(n, int(lib().mi355_experts_scratch_bytes(C.byref(a))))
        M.moe_scratch, M.moe_scratch_bytes = ptr(self._buf(n, torch.uint8)), n
        # prepared keys and values of a step's rows, one buffer per lender
        for r, l in enumerate(ls):
            if l.mixer == MIX["attention"] and l.attn.role == KV_LENDS:
                self.layers[r].attn.kv_rows = ptr(self._buf(R * l.attn.kv_heads * (l.attn.dim + l.attn.vdim), self.dtype))
        for r, j in enumerate(self.lenders):
            if j is not None:
                self.layers[r].attn.kv_rows = self.layers[j].attn.kv_rows
        self.logits_buf = self._buf(self.max_logits_rows * M.ld_logits, torch.float32).view(self.max_logits_rows, M.ld_logits)
        # the step's integers: tokens | row0 | count | slot | pos | want, one upload
        self.meta = torch.zeros((6, R), dtype=torch.int32, device=self.device)
        self.meta_host = torch.zeros((6, R), dtype=torch.int32, pin_memory=True)
        self._meta_sent = torch.cuda.Event()
        self._meta_sent.record(self.stream)

    @property
    def max_logits_rows(self) -> int:
        return min(self.max_rows, max(256, (1 << 28) // max(1, self.m.ld_logits)))

    # ---- slots -----------------------------------------------------------------------------------------
    def ensure(self, n_slots: int, max_len: int) -> None:
        """Room for `n_slots` live sequences of at most `max_len` tokens."""
        if max_len > self.max_len:
            self._set_len(max_len)
        with torch.cuda.stream(self.stream):
            self.slots.reserve(n_slots)

    def _set_len(self, n: int) -> None:
        """Rings hold min(window, longest sequence) rows (behind the first tokens').  Growing them re-lays the rings, so no sequence may be live unless every ring
        already spans its window."""
        need = any(l.mixer in (MIX["attention"], MIX["latent"]) and self._ring(r, n) != self._ring(r, self.max_len) for r, l in enumerate(list(self.layers)[: self.m.n_runs]))
        if need and self.slots.live == 1 and self._single is not None:
            self.reset_cache()  # (what is live is a sequence that generate() or forward() left behind)
        if need and self.max_len and self.slots.live:
            raise nat.NativeError(f"hybrid engine: sequences are live at cache length {self.max_len}; {n} needs a larger one")
        self.max_len = n
        with torch.cuda.device(self.device), torch.cuda.stream(self.stream):
            self._destroy_graphs()  # (captured launches hold the scratch)
            self._expand_scratch()
        if need and self.slots.capacity:
            self.pools = [None] * self.m.n_runs
            with torch.cuda.stream(self.stream):
                self._grow(self.slots.capacity)

    def _ring(self, r: int, max_len: int) -> int:
        return min(self.spans[r][0], max(1, max_len))

    def _grow(self, n: int) -> None:
        self._destroy_graphs()  # captured launches hold the old addresses
        if not hasattr(self, "pools"):
            self.pools = [None] * self.m.n_runs
        dev = self.device
        for r in range(self.m.n_runs):
            l, old = self.layers[r], self.pools[r] or (None, None)
            if l.mixer == 0:
                a, j = l.attn, self.lenders[r]
                if j is not None:
                    b = self.layers[j].attn
                    a.ring, a.kept, a.kring, a.vring = b.ring, b.kept, b.kring, b.vring
                    self.pools[r] = (None, None)
                    continue
                a.ring, a.kept = self._ring(r, self.max_len or 1), self.spans[r][1]
                k = grown(old[0], (n, a.kv_heads, a.kept + a.ring, a.dim), self.dtype, dev)
                v = grown(old[1], (n, a.kv_heads, a.kept + a.ring, a.vdim), self.dtype, dev)
                a.kring, a.vring = ptr(k), ptr(v)
                self.pools[r] = (k, v)
            elif l.mixer == MIX["latent"]:
                a = l.latent
                a.cache_rows = self._ring(r, self.max_len or 1)
                c = grown(old[0], (n, a.cache_rows, a.kv_rank + a.rot_dim), self.dtype, dev)
                a.cache = ptr(c)
                self.pools[r] = (c, None)
            else:
                e = l.rec
                st = grown(old[0], (n, e.heads, e.dim, e.vdim), torch.float32, dev)
                cv = None
                if e.kind in (REC_DELTA, REC_SSD):
                    cv = grown(old[1], (n, e.taps, 2 * e.kv_heads * e.dim + e.heads * e.vdim), self.dtype, dev)
                    e.conv_ring = ptr(cv)
                if l.n_mix:
                    cv = grown(old[1], (n, self.cfg.width), torch.float32, dev)
                    l.shift = ptr(cv)
                e.state = ptr(st)
                self.pools[r] = (st, cv)

    def state_bytes(self) -> int:
        """Bytes of cache and state per slot."""
        return sum(t.numel() * t.element_size() for p in self.pools for t in p if t is not None) // max(1, self.slots.capacity)

    def weight_bytes_of(self, rows: int) -> float:
        """Bytes of weights that a step of `rows` rows reads, rows choosing their experts independently."""
        total = float(self.weight_bytes)
        for i, l in enumerate(self.cfg.layers):
            f = l.mlp
            if f is not None and f.kind == "experts":
                used = f.experts * (1 - (1 - f.top / f.experts) ** rows)
                total -= (f.experts - used) * self._expert_bytes[i]
        return total

    def acquire(self) -> int:
        """A slot for a new sequence, its recurrent state zeroed."""
        with torch.cuda.stream(self.stream):
            slot = self.slots.acquire()
            self._reset([slot])
        return slot

    def release(self, slot: int) -> None:
        self.slots.release(slot)

    def _reset(self, slots: List[int]) -> None:
        t = torch.tensor(slots, dtype=torch.int32).to(self.device)
        check(lib().mi355_hybrid_reset_slots(C.byref(self.m), ptr(t), len(slots), self.stream.cuda_stream), "mi355_hybrid_reset_slots")
        self.stream.synchronize()  # (`t` may go)

    # ---- steps -----------------------------------------------------------------------------------------
    def _batch(self, rows: int, seqs: int, max_count: int, max_end: int = 0) -> SeqBatch:
        b = SeqBatch()
        b.rows, b.seqs, b.max_count, b.max_end = rows, seqs, max_count, max_end
        b.row0, b.count, b.slot, b.pos = (ptr(self.meta[i]) for i in (1, 2, 3, 4))
        return b

    def _upload(self, entries: Sequence[Entry]) -> tuple:
        """Packs a step's integers and sends them; returns (batch, wanted rows)."""
        h = self.meta_host
        self._meta_sent.synchronize()  # the previous upload has left the pinned buffer
        rows, n_want, most = 0, 0, 0
        for s, e in enumerate(entries):
            n = len(e.tokens)
            h[0, rows:rows + n] = torch.as_tensor(e.tokens, dtype=torch.int32)
            h[1, s], h[2, s], h[3, s], h[4, s] = rows, n, e.slot, e.pos
            if len(e.want):
                h[5, n_want:n_want + len(e.want)] = torch.as_tensor(e.want, dtype=torch.int32) + rows
                n_want += len(e.want)
            rows += n
            most = max(most, n)
        self.meta.copy_(h, non_blocking=True)
        self._meta_sent.record(self.stream)
        return self._batch(rows, len(entries), most, max(e.pos + len(e.tokens) for e in entries)), n_want

    def _cut(self, entries: Sequence[Entry]) -> List[List[Entry]]:
        """Sub-steps of at most max_rows rows and max_logits_rows wanted rows; a long portion continues in the next one."""
        subs, cur, room, wants = [], [], self.max_rows, self.max_logits_rows
        for e in entries:
            if e.pos + len(e.tokens) > self.max_len:
                raise nat.NativeError(f"hybrid engine: position {e.pos + len(e.tokens) - 1} is outside the cache of {self.max_len}")
            if min(e.tokens, default=0) < 0 or max(e.tokens, default=0) >= self.cfg.vocab_size:
                raise nat.NativeError(f"hybrid engine: token outside the vocabulary of {self.cfg.vocab_size}")
            at, want = 0, sorted(e.want)
            if list(e.want) != want:
                raise nat.NativeError("hybrid engine: wanted places must ascend")
            while at < len(e.tokens):
                if room == 0 or wants == 0:
                    subs.append(cur)
                    cur, room, wants = [], self.max_rows, self.max_logits_rows
                n = min(room, len(e.tokens) - at)
                inside = [k for k in want if at <= k < at + n]
                if len(inside) > wants:  # stop behind the last row whose logits still fit
                    inside = inside[:wants]
                    n = inside[-1] + 1 - at
                cur.append(Entry(e.slot, e.pos + at, e.tokens[at:at + n], [k - at for k in inside]))
                at, room, wants = at + n, room - n, wants - len(inside)
                if at < len(e.tokens):  # one sequence has one entry per sub-step
                    subs.append(cur)
                    cur, room, wants = [], self.max_rows, self.max_logits_rows
        if cur:
            subs.append(cur)
        return subs

    def step(self, entries: Sequence[Entry]) -> torch.Tensor:
        """Runs the new tokens of every entry; returns the wanted logits [n, vocab] f32 in the order of entries and places (a buffer of
        this engine when one sub-step was enough: valid until the next step).  Work is queued on the current stream's behalf."""
        entries = [e for e in entries if len(e.tokens)]
        cur = torch.cuda.current_stream(self.device)
        self.stream.wait_stream(cur)
        outs = []
        with torch.cuda.device(self.device), torch.cuda.stream(self.stream):
            subs = self._cut(entries)
            for sub in subs:
                b, n_want = self._upload(sub)
                self._run(b, n_want)
                if n_want:
                    out = self.logits_buf[:n_want, : self.n_logits]
                    outs.append(out if len(subs) == 1 else out.clone())
            res = outs[0] if len(outs) == 1 else torch.cat(outs) if outs else self.logits_buf[:0, : self.n_logits]
        cur.wait_stream(self.stream)
        return res

    def _launch(self, b: SeqBatch, n_want: int, all_rows: bool, run_end: int = 1 << 30) -> None:
        check(lib().mi355_hybrid_forward(C.byref(self.m), C.byref(b), ptr(self.meta[0]), None if all_rows else ptr(self.meta[5]), n_want,
                                         ptr(self.logits_buf), min(run_end, self.m.n_runs), self.stream.cuda_stream), "mi355_hybrid_forward")

    def _run(self, b: SeqBatch, n_want: int) -> None:
        decode = b.max_count == 1 and (n_want == b.rows or n_want == 0)
        if not decode:
            self._launch(b, n_want, False)
        else:
            self._replay(("step", b.rows, n_want), lambda: self._launch(b, n_want, n_want > 0))

    def _replay(self, key: tuple, enqueue) -> None:
        """The launches of `enqueue` as a graph of their own per key.  The first time they run as they are (launchers set kernel attributes
        lazily, which a capture must not see; a recurrent step cannot be repeated), the second time they are captured, then replayed."""
        s = self.stream.cuda_stream
        if not self.use_graph or key not in self._warm:
            enqueue()
            self._warm.add(key)
            return
        g = self._graphs.get(key)
        if g is None:
            # a collection inside the capture may free another engine or a tensor: synchronizing calls, which end the capture
            collecting = gc.isenabled()
            gc.disable()
            try:
                check(lib().mi355_graph_begin(s), "mi355_graph_begin")
                handle = C.c_void_p()
                try:
                    enqueue()
                finally:
                    rc = lib().mi355_graph_end(s, C.byref(handle))
            finally:
                if collecting:
                    gc.enable()
            check(rc, "mi355_graph_end")
            g = self._graphs[key] = handle
        check(lib().mi355_graph_launch(g, s), "mi355_graph_launch")

    def _destroy_graphs(self) -> None:
        if self._graphs:
            self.stream.synchronize()
        for g in self._graphs.values():
            lib().mi355_graph_destroy(g)
        self._graphs = {}

    def __del__(self):
        try:
            self._destroy_graphs()
        except Exception:
            pass

    def residual_after(self, entries: Sequence[Entry], run_end: int) -> torch.Tensor:
        """The residual stream [rows, width] behind the first `run_end` layer runs of a step (it advances the state like a step)."""
        with torch.cuda.device(self.device), torch.cuda.stream(self.stream):
            b, _ = self._upload(entries)
            self._launch(b, 0, False, run_end)
        self.stream.synchronize()
        return self.x.view(self.max_rows, self.m.ldx)[: b.rows, : self.cfg.width].clone()

    # ---- model(idx, max_seq_length, input_pos) ---------------------------------------------------------
    def forward_no_cache(self, idx: torch.Tensor) -> torch.Tensor:
        B, T = idx.shape
        self.ensure(self.slots.live + B, max(self.max_len, T))
        slots = [self.acquire() for _ in range(B)]
        rows = idx.tolist()
        out = self.step([Entry(s, 0, r, range(T)) for s, r in zip(slots, rows)]).clone().view(B, T, -1)
        for s in slots:
            self.release(s)
        return out

    def forward(self, idx: torch.Tensor, max_seq_length: int, input_pos: torch.Tensor) -> torch.Tensor:
        T = idx.shape[1]
        pos0 = getattr(input_pos, "_mi355_pos0", None)
        if pos0 is None:
            pos0 = int(input_pos[0])
        if pos0 == 0 or self._single is None:
            self._ensure_cache(max_seq_length)
        if pos0 != self._next:
            raise nat.NativeError(f"a recurrent model continues its sequence at position {self._next}, not {pos0} (reset_cache() starts over)")
        out = self.step([Entry(self._single, pos0, idx.reshape(-1).tolist(), range(T))]).clone()
        self._next = pos0 + T
        return out.view(1, T, -1)

    # ---- generate()'s interface (engine.DecodeEngine's) ------------------------------------------------
    def reset_cache(self) -> None:
        if self._single is not None:
            self.release(self._single)
            self._single = None

    def _ensure_cache(self, S: int) -> None:
        """A fresh sequence of at most S tokens in the slot that generate() owns."""
        self.reset_cache()
        self.ensure(self.slots.live + 1, max(S, self.max_len))
        self._single, self._next = self.acquire(), 0
        if getattr(self, "out_tokens", None) is None or self.out_tokens.numel() < S + 1:
            self.out_tokens = torch.zeros(S + 1, dtype=torch.int32, device=self.device)
            self._destroy_graphs()
        self.next_token = getattr(self, "next_token", None)
        if self.next_token is None:
            self.next_token = torch.zeros(1, dtype=torch.int32, device=self.device)

    @property
    def tokens(self) -> torch.Tensor:
        return self.meta[0]

    @property
    def pos(self) -> torch.Tensor:
        return self.meta[4]

    @property
    def logits(self) -> torch.Tensor:
        return self.logits_buf

    def clear_status(self) -> None:
        pass

    def status_due(self) -> bool:
        return False  # (no step of this engine leaves a state to be read back)

    def check_status(self) -> Optional[int]:
        return None

    def _advance(self) -> None:
        check(lib().mi355_argmax_advance_rows(ptr(self.logits_buf), self.m.ld_logits, self.n_logits, 1, ptr(self.next_token),
                                              ptr(self.meta[0]), ptr(self.meta[4]), ptr(self.out_tokens), self.out_tokens.numel(),
                                              self.stream.cuda_stream), "mi355_argmax_advance_rows")

    def prefill(self, idx: torch.Tensor, pos0: int, *, all_logits: bool, argmax: bool = False) -> Optional[torch.Tensor]:
        toks = idx.reshape(-1).tolist()
        T = len(toks)
        subs = self._cut([Entry(self._single, pos0, toks, range(T) if all_logits else [T - 1])])
        out = []
        for sub in subs:
            b, n = self._upload(sub)
            self._launch(b, n, False)
            if all_logits and n:
                out.append(self.logits_buf[:n, : self.n_logits].clone())
        self._next = pos0 + T
        if argmax:  # the draw of position T - 1: out_tokens[T]
            self.set_step(idx.reshape(-1)[-1:], 1, pos0 + T - 1)
            self._advance()
        return torch.cat(out) if all_logits else None

    def set_step(self, idx: Optional[torch.Tensor], T: int, pos0: int, from_next: bool = False) -> None:
        """One-token entry state of generate()'s slot (host-known token or the last draw)."""
        self.meta[0, :1].copy_((self.next_token if from_next else idx.reshape(-1)[:1]).to(torch.int32))
        h = torch.tensor([[0], [1], [self._single], [pos0]], dtype=torch.int32)
        self.meta[1:5, :1].copy_(h.to(self.device))

    def embed_step(self) -> None:
        pass  # (the step starts at its token)

    def run_step(self, argmax) -> None:
        """One decode step at the token / position on the device; argmax 3: the greedy draw becomes the next step's token."""
        b = self._batch(1, 1, 1)

        def enqueue():
            self._launch(b, 1, True)
            if int(argmax) & 1:
                self._advance()

        self._replay(("single", int(argmax)), enqueue)
        self._next += 1
