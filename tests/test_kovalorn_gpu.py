"""The Kovalorn design on the GPU against the plain restatement in oracle/kovalorn.py: each mechanism's kernels alone, then the model through
its engine, scheduler and generate().  Inputs are made so that a fault shows: keys that stand out just inside and just outside a window or
the first tokens, loud sinks, sizes that differ from each other."""
import json

import pytest
import torch

from oracle import kovalorn as O

pytestmark = pytest.mark.gpu


def rel(got, ref):
    """Largest deviation over the reference's root mean square; a bf16 result has its last rounding (2^-8 of the value) for free."""
    free = 2.0 ** -8 if got.dtype == torch.bfloat16 else 0.0
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    assert got.shape == ref.shape
    return float(((got - ref).abs() - free * ref.abs()).max() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


TOL = {torch.float32: 2e-5, torch.bfloat16: 4e-2}
EPS = 2e-3


# ---------------------------------------------------------------------------------------- attention
class Case:
    """Packed projections of one sequence.  Keys around the window's and the first tokens' edges stand out for the queries at both sides."""

    def __init__(self, T, H, G, dim, vdim, window, keep, dtype, seed=0, sinks=True):
        gen = torch.Generator().manual_seed(seed)
        pad = lambda n: (n + 15) // 16 * 16
        self.T, self.H, self.G, self.dim, self.vdim, self.window, self.keep, self.dtype = T, H, G, dim, vdim, window, keep, dtype
        self.off_k = pad(H * dim)
        self.off_v = self.off_k + pad(G * dim)
        self.off_g = self.off_v + pad(G * vdim)
        p = torch.randn((T, self.off_g + pad(H * vdim)), generator=gen)
        q, k, v = p[:, :H * dim].view(T, H, dim), p[:, self.off_k:self.off_k + G * dim].view(T, G, dim), p[:, self.off_v:self.off_v + G * vdim].view(T, G, vdim)
        k *= 3.0 ** torch.randint(-2, 3, (T, 1, 1), generator=gen)      # (their size must not count)
        for j in [*range(2, T - 1, max(1, T // 7)), 0, keep - 1, keep]:
            if not 0 <= j < T:
                continue
            loud = torch.randn((G, dim), generator=gen)
            k[j] = 2 * loud
            v[j] += 4
            for i in (j + window - 1, j + window, j + 2 * window + 5, T - 1 - j):
                if j <= i < T:
                    q[i] = 0.5 * loud.repeat_interleave(H // G, 0)
        self.p = p.to(dtype)
        self.scale = 6.0 / dim
        self.sink = (torch.randn(H, generator=gen) * 2 + 3).float() if sinks else None

    def parts(self):
        d, T = self.p.double(), self.T
        cut = lambda off, n, s: d[:, off:off + n * s].view(T, n, s)
        return cut(0, self.H, self.dim), cut(self.off_k, self.G, self.dim), cut(self.off_v, self.G, self.vdim), cut(self.off_g, self.H, self.vdim)

    def reference(self, k=None, v=None):
        q, k0, v0, g = self.parts()
        k, v = (k0, v0) if k is None else (k, v)
        o = O.sink_attention(O.unit_rms(q, EPS), O.unit_rms(k, EPS), v, self.scale, self.window, self.keep,
                             None if self.sink is None else self.sink.double())
        return (o * torch.sigmoid(g)).reshape(self.T, -1)

    def kw(self, dev, **kw):
        return dict(heads=self.H, scale=self.scale, window=self.window, keep=self.keep, off_q=0, off_k=self.off_k, off_v=self.off_v, off_g=self.off_g,
                    gate_values=True, unit_eps=EPS, sink=None if self.sink is None else self.sink.to(dev), **kw)

    def rings(self, dev, kept, ring):
        shape = (3, self.G, kept + ring)
        return (torch.full((*shape, self.dim), 7.0, dtype=self.dtype, device=dev), torch.full((*shape, self.vdim), 9.0, dtype=self.dtype, device=dev))


def run_portions(dev, case, cuts, kept, ring, path=0, split=False):
    from lit_llama_amd import ops

    kr, vr = case.rings(dev, kept, ring)
    part = torch.zeros(1 << 20, device=dev) if split else None
    out, at = [], 0
    for n in cuts:
        b = ops.PackedBatch([n], [1], [at], dev)
        out.append(ops.window_attention(case.p[at:at + n].contiguous().to(dev), b, kr, vr, path=path, partials=part, kept=kept, **case.kw(dev)))
        at += n
    assert at == case.T
    assert (kr[0] == 7).all() and (kr[2] == 7).all() and (vr[0] == 9).all() and (vr[2] == 9).all()
    return torch.cat(out)


SHAPES = [(4, 2, 40, 24, 37, 3), (6, 1, 64, 64, 64, 64), (3, 3, 18, 10, 20, 1), (8, 2, 128, 128, 130, 70), (10, 1, 72, 200, 1, 5), (2, 1, 32, 16, 500, 4),
          (5, 5, 24, 56, 3, 9), (16, 1, 96, 80, 48, 0)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,dim,vdim,window,keep", SHAPES)
def test_attention(dev, dtype, H, G, dim, vdim, window, keep):
    T = 210
    case = Case(T, H, G, dim, vdim, window, keep, dtype)
    ref = case.reference()
    ring = min(window, T)
    assert rel(run_portions(dev, case, [T], keep, ring), ref) < TOL[dtype]
    for cuts in ([2] * 3 + [T - 6], [100, 1, 64, T - 165], [1, 1, 1, T - 3], [T - 70] + [1] * 70):
        assert rel(run_portions(dev, case, cuts, keep, ring), ref) < TOL[dtype], cuts
    assert rel(run_portions(dev, case, [90, T - 90], keep, ring, path=1), ref) < TOL[dtype]
    assert rel(run_portions(dev, case, [90, T - 140] + [1] * 50, keep + 6, ring + 3), ref) < TOL[dtype]  # (a lender's cache spans more)


def test_attention_token_by_token_from_the_first(dev):
    case = Case(90, 4, 2, 32, 16, 21, 6, torch.float32, seed=3)
    assert rel(run_portions(dev, case, [1] * 90, 6, 21), case.reference()) < TOL[torch.float32]


@pytest.mark.parametrize("sinks", [False, True])
def test_attention_split_decode(dev, sinks):
    T = 700
    case = Case(T, 4, 1, 64, 32, 560, 40, torch.float32, sinks=sinks)
    assert rel(run_portions(dev, case, [T - 60] + [1] * 60, 44, 560, split=True), case.reference()) < TOL[torch.float32]


def test_a_sink_far_above_and_far_below_the_scores(dev):
    case = Case(150, 2, 1, 64, 64, 40, 4, torch.bfloat16)
    for level in (-60.0, 25.0):
        case.sink = torch.full((2,), level)
        for cuts in ([150], [100] + [1] * 50):
            got, ref = run_portions(dev, case, cuts, 4, 40), case.reference()
            assert torch.isfinite(got).all() and rel(got, ref) < TOL[torch.bfloat16]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_lent_keys_and_values(dev, dtype):
    """A lender with a short window and two borrowers with other windows and first tokens, in portions that wrap the cache and in decoding."""
    from lit_llama_amd import ops

    T, H, G, dim, vdim = 230, 4, 2, 32, 48
    lender = Case(T, H, G, dim, vdim, 20, 2, dtype, seed=1)
    borrowers = [Case(T, H, G, dim, vdim, 70, 0, dtype, seed=2), Case(T, H, G, dim, vdim, 9, 11, dtype, seed=3)]
    _, k, v, _ = lender.parts()
    for b in borrowers:  # a borrower's queries look for keys at the edges of its own window and first tokens
        q = b.p[:, :H * dim].view(T, H, dim)
        for j in (0, 1, b.keep - 1, b.keep, 60, 100, 130):
            for i in (j + b.window - 1, j + b.window, j + 150):
                if 0 <= j <= i < T:
                    q[i] = k[j].to(dtype).repeat_interleave(H // G, 0)
    refs = [lender.reference()] + [b.reference(k, v) for b in borrowers]
    kept, ring = 11, 70
    for cuts in ([T], [2, 90, 3, T - 95], [150] + [1] * 80, [40, 1, 1, 60, T - 102]):
        kr, vr = lender.rings(dev, kept, ring)
        out, at = [[], [], []], 0
        for n in cuts:
            b = ops.PackedBatch([n], [1], [at], dev)
            rows = torch.full((n, G * (dim + vdim)), float("nan"), dtype=dtype, device=dev)
            for x, (case, role) in enumerate(((lender, "lends"), (borrowers[0], "borrows"), (borrowers[1], "borrows"))):
                out[x].append(ops.window_attention(case.p[at:at + n].contiguous().to(dev), b, kr, vr, kept=kept, role=role, kv_rows=rows, **case.kw(dev)))
            ops.window_cache_write(b, kr, vr, rows, kept)
            at += n
        for got, ref in zip(out, refs):
            assert rel(torch.cat(got), ref) < TOL[dtype], cuts
        assert (kr[0] == 7).all() and (vr[2] == 9).all()


# ---------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,W,E,top,ff,shared", [(1, 72, 5, 2, 24, 40), (3, 200, 9, 9, 17, 0), (8, 384, 70, 4, 130, 7), (9, 130, 19, 5, 33, 0),
                                                    (40, 104, 6, 1, 50, 150), (333, 72, 4, 2, 24, 40), (700, 256, 7, 3, 140, 300), (65, 98, 150, 8, 16, 16)])
def test_experts(dev, dtype, rows, W, E, top, ff, shared):
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(rows)
    rnd = lambda *s, gain=1.0: (torch.randn(s, generator=gen) * gain * s[-1] ** -0.5).to(dtype)
    x = torch.randn((rows, W), generator=gen) * 3
    norm, router = (0.3 * torch.randn(W, generator=gen)).to(dtype), rnd(E, W, gain=2)
    ws = [(rnd(ff, W, gain=2), rnd(ff, W, gain=2), rnd(W, ff, gain=2)) for _ in range(E)]
    sh = (rnd(shared, W), rnd(shared, W), rnd(W, shared)) if shared else None
    w = {"router": router, **{f"e{e}.{n}": t for e, ts in enumerate(ws) for n, t in zip(("gate", "up", "down"), ts)}}
    w.update({f"shared.{n}": t for n, t in zip(("gate", "up", "down"), sh or ())})
    w = {n: t.double() for n, t in w.items()}
    h = O.rms_norm(x.double(), norm.double(), 1e-4)
    spec = {"router": {"top": top, "scale": 1.7}, "shared": sh}
    ref = x.double() + 0.6 * O.experts_ff(w, "", spec, h)
    if top < E:  # rows whose last chosen and first left-out expert are a rounding apart may differ
        z = (h @ w["router"].T).sort(-1, descending=True).values
        clear = (z[:, top - 1] - z[:, top]) > (0.02 if dtype == torch.bfloat16 else 1e-5)
    else:
        clear = torch.ones(rows, dtype=torch.bool)
    assert clear.float().mean() > 0.5
    to = lambda ts: tuple(t.to(dev) for t in ts)
    for path in ((0, 1, 2) if dtype == torch.bfloat16 else (0,)):
        got = ops.experts(x.to(dev), norm.to(dev), router.to(dev), [to(t) for t in ws], to(sh) if sh else None, top=top, scale=1.7, eps=1e-4,
                          norm_add=1.0, alpha=0.6, path=path).cpu()
        assert torch.isfinite(got).all()
        d, r = (got - x)[clear], (ref - x.double())[clear]
        assert rel(d, r) < (5e-5 if dtype == torch.float32 else 0.06), path
        if rows > 1 and path != 1:  # a row's result does not depend on its batch
            one = ops.experts(x[1:2].to(dev), norm.to(dev), router.to(dev), [to(t) for t in ws], to(sh) if sh else None, top=top, scale=1.7, eps=1e-4,
                              norm_add=1.0, alpha=0.6, path=path).cpu()
            assert rel(one - x[1:2], got[1:2] - x[1:2]) < (2e-5 if dtype == torch.float32 else 0.02)


def test_all_rows_choose_the_same_expert(dev):
    """One expert takes every row (full tiles and a rest), the others none; and two experts of equal score: the lower index."""
    from lit_llama_amd import ops

    W, E, rows = 64, 6, 300
    gen = torch.Generator().manual_seed(1)
    x = torch.randn((rows, W), generator=gen).abs() + 0.1
    ws = [tuple(torch.randn(s, generator=gen).to(torch.bfloat16) * 0.2 for s in ((32, W), (32, W), (W, 32))) for _ in range(E)]
    router = torch.full((E, W), -0.01).to(torch.bfloat16)
    router[3] = router[5] = 0.01
    h = O.rms_norm(x.double(), torch.zeros(W).double(), 1e-5)
    got = ops.experts(x.to(dev), torch.zeros(W, dtype=torch.bfloat16, device=dev), router.to(dev), [tuple(t.to(dev) for t in w) for w in ws],
                      top=1, scale=2.0, eps=1e-5, norm_add=1.0).cpu()
    g, u, d = (t.double() for t in ws[3])
    ref = 2.0 * (O.silu(h @ g.T) * (h @ u.T)) @ d.T
    assert rel(got - x, ref) < 0.03


# ---------------------------------------------------------------------------------------- gated GELU, norm around one, logit scale
@pytest.mark.parametrize("M", [1, 5, 40, 300])
@pytest.mark.parametrize("N,K", [(80, 96), (272, 256)])
def test_gated_gelu_product(dev, M, N, K):
    import ctypes as C

    from lit_llama_amd import _native as nat
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(M)
    x = (torch.randn((M, K), generator=gen) * 2).to(dev)
    norm = (0.3 * torch.randn(K, generator=gen)).to(torch.bfloat16).to(dev)
    g, u = ((torch.randn((N, K), generator=gen) * 2 * K ** -0.5).to(torch.bfloat16).to(dev) for _ in range(2))
    y = torch.zeros((M, N), dtype=torch.bfloat16, device=dev)
    a = nat.LinearArgs()
    w = ops.repack_bf16(g, u, 2)
    a.fmt, a.R, a.w, a.N, a.K, a.x, a.x_dtype, a.M, a.ldx = nat.W_BF16, 2, nat.ptr(w), N, K, nat.ptr(x), nat.F32, M, K
    a.norm_scale, a.norm_dtype, a.eps, a.epi, a.y, a.y_dtype, a.ldy = nat.ptr(norm), nat.BF16, 1e-4, nat.EPI_GEGLU, nat.ptr(y), nat.BF16, N
    a.flags = nat.LF_NORM_ONE
    h = O.rms_norm(x.cpu().double(), norm.cpu().double(), 1e-4)
    ref = O.gelu_tanh(h @ g.cpu().double().T) * (h @ u.cpu().double().T)
    ws = torch.empty(nat.lib().mi355_linear_gemm_workspace_bytes(M, K), dtype=torch.uint8, device=dev)
    if M <= 5:
        nat.check(nat.lib().mi355_linear_fast(C.byref(a), nat.stream_ptr()))
        assert rel(y, ref) < 0.05
        y.zero_()
    nat.check(nat.lib().mi355_linear_gemm(C.byref(a), nat.ptr(ws), ws.numel(), nat.stream_ptr()))
    assert rel(y, ref) < 0.05


# ---------------------------------------------------------------------------------------- the model
def small_config(**kw):
    def att(**m):
        return {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 40, "scale": 0.3, "mask": {"size": 19, "keep_first": 3}, **m}

    moe = {"kind": "moe", "expert": {"ff": 36}, "router": {"experts": 5, "scale": 1.4, "top": 2}, "shared": {"ff": 52}}
    layers = [
        {"type": "attention", "mixer": att(), "mlp": moe},
        {"type": "attention", "mixer": att(kv_heads=1, heads=6, dim=40, vdim=16, mask={"size": 33, "keep_first": 0}), "mlp": {"kind": "dense", "ff": 72}},
        {"type": "attention", "mixer": att(kv_from=0, mask={"size": 47, "keep_first": 6}, scale=0.2), "mlp": None},
        {"type": "attention", "mixer": att(kv_from=1, kv_heads=1, heads=6, dim=40, vdim=16, mask={"size": 11, "keep_first": 1}), "mlp": {**moe, "shared": None}},
        {"type": "attention", "mixer": att(kv_from=0, mask={"size": 7, "keep_first": 2}), "mlp": {**moe, "router": {"experts": 3, "scale": 0.8, "top": 1}}},
    ]
    return {"architecture": "Kovalorn", "vocab": 211, "width": 104, "norm": {"eps": 3e-5}, "logit_scale": 0.6, "layers": layers, **kw}


def build(config, dtype, dev, seed=1):
    from lit_llama_amd import synth
    from lit_llama_amd.registry import build_model

    sd = synth.make_hybrid_state_dict(config, seed=seed)
    m = build_model(config, dtype, dev)
    m.load_state_dict(sd)
    return m, sd


def tokens_of(n, vocab=211, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


ONE = {"type": "attention", "mixer": {"heads": 3, "kv_heads": 3, "dim": 18, "vdim": 10, "scale": 0.25}, "mlp": {"kind": "dense", "ff": 30}}
CONFIGS = {
    "mixed": small_config(),
    "no window, odd sizes": small_config(layers=[ONE, {**ONE, "mixer": {**ONE["mixer"], "kv_from": 0, "mask": {"size": 5, "keep_first": 1}}}], width=61, vocab=130,
                                         logit_scale=1.0),
    "every expert, one head": small_config(layers=[{"type": "attention", "mixer": {"heads": 1, "kv_heads": 1, "dim": 64, "vdim": 32, "scale": 0.125,
                                                                                   "mask": {"size": 16, "keep_first": 1}},
                                                    "mlp": {"kind": "moe", "expert": {"ff": 16}, "router": {"experts": 2, "scale": 1.0, "top": 2},
                                                            "shared": {"ff": 16}}}] * 2, width=128, logit_scale=2.0),
}


@pytest.mark.parametrize("name", CONFIGS)
def test_model_layer_by_layer_and_logits(dev, name):
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS[name]
    m, sd = build(config, torch.float32, dev)
    eng = m.engine()
    eng.ensure(2, 128)
    toks = tokens_of(61, config["vocab"])
    logits, trail = O.forward(config, sd, toks)
    for r in range(1, len(trail) + 1):
        s = eng.acquire()
        assert rel(eng.residual_after([Entry(s, 0, toks, [])], r), trail[r - 1]) < 5e-5, r
        eng.release(s)
    s = eng.acquire()
    assert rel(eng.step([Entry(s, 0, toks, range(61))]), logits) < 5e-5
    eng.release(s)


def reference(config, sd, toks, monkeypatch):
    """The oracle's logits, and the positions where no router's last choice was close to the next expert (rounding may take the other one)."""
    route, gaps = O.route, [torch.full((len(toks),), 1.0, dtype=torch.float64)]

    def watched(h, router, top, scale):
        if top < router.shape[0]:
            z = (h @ router.T).sort(-1, descending=True).values
            gaps.append(z[:, top - 1] - z[:, top])
        return route(h, router, top, scale)

    with monkeypatch.context() as mp:
        mp.setattr(O, "route", watched)
        logits = O.forward(config, sd, toks)[0]
    return logits, torch.stack(gaps).min(0).values > 0.05


def close(got, ref, dtype):
    """float32: every logit; bfloat16: the positions with clear choices (a few may see a token that went elsewhere)."""
    logits, clear = ref
    if dtype == torch.float32:
        return rel(got, logits) < 1e-4
    err = (got.double().cpu() - logits).pow(2).mean(-1).sqrt() / logits.pow(2).mean().sqrt()
    return float(torch.quantile(err[clear], 0.95)) < 0.03


@pytest.mark.parametrize("name,dtype", [("mixed", torch.float32), ("mixed", torch.bfloat16), ("every expert, one head", torch.bfloat16),
                                        ("no window, odd sizes", torch.float32)])
def test_portions_batches_slots_and_decoding(dev, name, dtype, monkeypatch):
    """Unequal requests in one batch, cut differently, decoded together, their slots used again: the logits of each alone."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS[name]
    m, sd = build(config, dtype, dev)
    eng = m.engine()
    eng.ensure(4, 200)
    seqs = [tokens_of(n, config["vocab"], seed=n) for n in (150, 9, 64, 33)]
    refs = [reference(config, sd, s, monkeypatch) for s in seqs]
    assert sum(float(c.sum()) for _, c in refs) > 200
    for first in ((100, 2, 31, 32), (64, 8, 1, 3), (1, 1, 1, 1)):  # (the second and third time in the slots of the first)
        slots = [eng.acquire() for _ in seqs]
        at = [0] * 4
        got = [[] for _ in seqs]

        def feed(counts):
            es = []
            for i, n in enumerate(counts):
                n = min(n, len(seqs[i]) - at[i])
                if n:
                    es.append((i, Entry(slots[i], at[i], seqs[i][at[i]:at[i] + n], range(n))))
            lg = eng.step([e for _, e in es]).clone().split([len(e.tokens) for _, e in es])
            for (i, e), x in zip(es, lg):
                got[i].append(x)
                at[i] += len(e.tokens)

        feed(first)
        feed((2, 1, 2, 30))      # a mixed batch: two-row portions and single rows
        while any(a < len(s) for a, s in zip(at, seqs)):
            feed((1, 1, 1, 1))
        for i in range(4):
            assert close(torch.cat(got[i]), refs[i], dtype), (i, first)
        for s in slots:
            eng.release(s)
    assert eng.slots.live == 0


def test_a_large_batch_decodes_like_each_alone(dev, monkeypatch):
    """Enough sequences that the experts are sorted by expert in a decode step."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS["mixed"]
    m, sd = build(config, torch.bfloat16, dev)
    eng = m.engine()
    eng.ensure(24, 64)
    seqs = [tokens_of(30 + i, seed=i) for i in range(24)]
    slots = [eng.acquire() for _ in seqs]
    eng.step([Entry(s, 0, t[:20], []) for s, t in zip(slots, seqs)])
    rows = torch.stack([eng.step([Entry(s, 20 + k, t[20 + k:21 + k], [0]) for s, t in zip(slots, seqs)]).clone() for k in range(8)], 1)
    for i in (0, 11, 23):
        logits, clear = reference(config, sd, seqs[i][:28], monkeypatch)
        assert clear[20:].any() and close(rows[i], (logits[20:], clear[20:]), torch.bfloat16)


def test_a_step_larger_than_the_scratch_is_cut(dev):
    from lit_llama_amd.hybrid_engine import Entry, HybridEngine

    config = CONFIGS["mixed"]
    m, sd = build(config, torch.float32, dev)
    eng = HybridEngine(m, max_rows=48)
    eng.ensure(3, 200)
    seqs = [tokens_of(n, seed=n) for n in (130, 17, 60)]
    slots = [eng.acquire() for _ in seqs]
    out = eng.step([Entry(s, 0, t, [0, len(t) - 1]) for s, t in zip(slots, seqs)])
    ref = torch.cat([O.forward(config, sd, t)[0][[0, len(t) - 1]] for t in seqs])
    assert rel(out, ref) < 1e-4


def greedy_reference(config, sd, prompt, n, margin):
    """Greedy continuation by the oracle, up to the first near tie."""
    seq = list(prompt)
    for _ in range(n):
        top = torch.topk(O.forward(config, sd, seq)[0][-1], 2)
        if float(top.values[0] - top.values[1]) < margin:
            break
        seq.append(int(top.indices[0]))
    return seq[len(prompt):]


def test_greedy_generation_through_generate_and_the_scheduler(dev):
    import lit_llama_amd
    from lit_llama_amd.batching import generate_batch

    config = CONFIGS["mixed"]
    m, sd = build(config, torch.float32, dev)
    prompts = [tokens_of(n, seed=n) for n in (23, 3, 40, 1, 18)]
    refs = [greedy_reference(config, sd, p, 10, 1e-3) for p in prompts]
    assert sum(map(len, refs)) > 25
    outs = generate_batch(m, prompts, 10, top_k=1, max_batch=3, portion=16)  # (requests wait, enter late, are cut)
    for o, r in zip(outs, refs):
        assert len(o) == 10 and o[:len(r)] == r
    assert m.engine().slots.live == 0
    for p, r in zip(prompts[:2], refs):
        y = lit_llama_amd.generate(m, torch.tensor(p, device=dev), 10, top_k=1).tolist()
        assert y[:len(p)] == p and len(y) == len(p) + 10 and y[len(p):len(p) + len(r)] == r
    # a batch behind generate() that needs a longer cache than its sequence
    fresh, _ = build(config, torch.float32, dev)
    lit_llama_amd.generate(fresh, torch.tensor([1, 2, 3], device=dev), 2, top_k=1)
    assert generate_batch(fresh, prompts[:2], 10, top_k=1) == outs[:2]
    x = generate_batch(m, [prompts[0], prompts[2]], 8, temperature=0.9, top_k=50, seed=3)
    assert x == generate_batch(m, [prompts[0], prompts[2]], 8, temperature=0.9, top_k=50, seed=3)


def test_long_decoding_matches_the_prompt_pass(dev):
    """Hundreds of decoded tokens (windows pass over them, graphs replayed, eager work in between) against one prompt pass."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS["mixed"]
    m, sd = build(config, torch.float32, dev)
    eng = m.engine()
    eng.ensure(2, 400)
    toks = tokens_of(380)
    s, t = eng.acquire(), eng.acquire()
    whole = eng.step([Entry(s, 0, toks, range(380))]).clone()
    rows = [eng.step([Entry(t, 0, toks[:5], range(5))]).clone()]
    for i in range(5, 380):
        rows.append(eng.step([Entry(t, i, toks[i:i + 1], [0])]).clone())
        if i % 50 == 0:
            torch.randn(1000, device=dev).sum().item()
    assert rel(torch.cat(rows), whole) < 2e-4
    assert rel(whole[-1:], O.forward(config, sd, toks)[0][-1:]) < 1e-4


def test_trace_replay_and_command_line(dev, tmp_path, capsys, monkeypatch):
    import io

    import numpy as np
    from safetensors.torch import save_file

    from lit_llama_amd import __main__ as cli
    from lit_llama_amd import synth, trace

    config = CONFIGS["mixed"]
    sd = synth.make_hybrid_state_dict(config, seed=9)
    (tmp_path / "config.json").write_text(json.dumps(config))
    save_file(sd, str(tmp_path / "model.safetensors"))
    a, b = tokens_of(25, seed=1), tokens_of(11, seed=2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:21], "want": [0]}, {"id": "b", "tokens": b[8:9], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[21:22], "want": []}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    ra, rb = O.forward(config, sd, a)[0], O.forward(config, sd, b)[0]
    got = [torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, 211)) for i in (0, 1)]
    assert rel(got[0], ra[[0, 19]]) < 1e-4 and rel(got[1], torch.stack([ra[20], rb[8]])) < 1e-4
    assert not (tmp_path / "2.f32").exists()
    assert cli.main(["--model", str(tmp_path), "--dtype", "float32", "--prompt-ids", ",".join(map(str, a)), "--prompt-ids", "1,2", "--top-k", "1",
                     "--max-new-tokens", "5"]) == 0
    lines = capsys.readouterr().out.strip().split("\n")
    assert len(lines) == 2 and lines[0].startswith(",".join(map(str, a))) and len(lines[0].split(",")) == 30
