"""The Gurolix design on the GPU against the plain restatement in oracle/gurolix.py: each mechanism's kernels alone, then the model through its
engine, scheduler and generate().  Inputs are made so that a fault shows: far keys that stand out among hundreds, scores beyond their bound,
states that decay slowly and at once, corrections that change the choice, sizes that differ from each other."""
import ctypes as C
import json
import math

import pytest
import torch

from oracle import gurolix as O

pytestmark = pytest.mark.gpu


def rel(got, ref):
    """Largest deviation over the reference's root mean square; a bf16 result has its last rounding (2^-8 of the value) for free."""
    free = 2.0 ** -8 if got.dtype == torch.bfloat16 else 0.0
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    assert got.shape == ref.shape
    return float(((got - ref).abs() - free * ref.abs()).max() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


def rows_off(got, ref):
    """The largest error of a row over the row's own size, root mean squares."""
    e = got.detach().double().cpu() - ref
    return float((e.pow(2).mean(-1) / ref.pow(2).mean(-1)).sqrt().max())


TOL = {torch.float32: 2e-5, torch.bfloat16: 4e-2}
EPS = 2e-3
pad16 = lambda n: (n + 15) // 16 * 16


# ---------------------------------------------------------------------------------------- attention
class Case:
    """Packed projections of one sequence, heads in the checkpoint's order of dimensions; a few keys stand out for queries near and far."""

    def __init__(self, T, H, G, dim, vdim, rot, dtype, norm=False, cap=0.0, mix=None, seed=0, gain=4.0, loud=2.0):
        gen = torch.Generator().manual_seed(seed)
        self.T, self.H, self.G, self.dim, self.vdim, self.rot, self.dtype = T, H, G, dim, vdim, rot, dtype
        self.cap, self.mix, self.scale = cap, mix, gain / dim
        self.off_k = pad16(H * dim)
        self.off_v = self.off_k + pad16(G * dim)
        p = torch.randn((T, self.off_v + pad16(G * vdim)), generator=gen)
        q, k, v = p[:, :H * dim].view(T, H, dim), p[:, self.off_k:self.off_k + G * dim].view(T, G, dim), p[:, self.off_v:self.off_v + G * vdim].view(T, G, vdim)
        if norm:
            q *= 3.0 ** torch.randint(-2, 3, (T, 1, 1), generator=gen)  # (their size must not count)
            k *= 3.0 ** torch.randint(-2, 3, (T, 1, 1), generator=gen)
        turned = rot["dims"]
        for j in {0, 1, 63, 64, T // 2, T - 2}:  # (where rotation leaves dimensions alone, or the same place: exact matches at any distance)
            if not 0 <= j < T:
                continue
            ray = torch.randn((G, dim), generator=gen)
            if turned < dim:
                ray[:, :turned] *= 0.1
            k[j] = loud * ray
            v[j] += 4
            for i in {j, j + 1, j + 7, T - 1 - j, T - 1}:
                if j <= i < T:
                    q[i] = loud * ray.repeat_interleave(H // G, 0)
        self.p = p.to(dtype)
        self.first = torch.randn((T, G * vdim), generator=gen).to(dtype) if mix is not None else None
        self.q_norm, self.k_norm = ((1 + 0.3 * torch.randn(dim, generator=gen)) for _ in range(2)) if norm else (None, None)

    def reference(self):
        d, T = self.p.double(), self.T
        q, k, v = (d[:, off:off + n * s].view(T, n, s) for off, n, s in ((0, self.H, self.dim), (self.off_k, self.G, self.dim), (self.off_v, self.G, self.vdim)))
        if self.q_norm is not None:
            q, k = O.unit_rms(q, EPS) * self.q_norm.double(), O.unit_rms(k, EPS) * self.k_norm.double()
        if self.rot["dims"]:
            q, k = O.rotate_halves(q, self.rot), O.rotate_halves(k, self.rot)
        if self.mix is not None:
            v = O.mix_values(v, self.first.double().view(v.shape), torch.tensor(self.mix))
        return O.attend(q, k, v, self.scale, self.cap or None).reshape(T, -1)

    def inputs(self, dev):
        """Columns in the kernels' order: the partners of a rotation side by side."""
        half = self.rot["dims"] // 2
        turn = [d for i in range(half) for d in (i, i + half)] + list(range(2 * half, self.dim))
        p = self.p.clone()
        for off, n in ((0, self.H), (self.off_k, self.G)):
            w = p[:, off:off + n * self.dim].view(self.T, n, self.dim)
            w.copy_(w[..., turn].clone())
        kw = dict(heads=self.H, scale=self.scale, window=1 << 30, off_q=0, off_k=self.off_k, off_v=self.off_v, softcap=self.cap)
        if half:
            kw["inv_freq"] = O.frequencies(self.rot).to(dev)
        if self.q_norm is not None:
            kw.update(unit_eps=EPS, q_norm=self.q_norm[turn].to(dev), k_norm=self.k_norm[turn].to(dev))
        return p, kw


def run_portions(dev, case, cuts, path=0, split=False, ring=None):
    from lit_llama_amd import ops

    p, kw = case.inputs(dev)
    ring = ring or case.T
    kr = torch.full((3, case.G, ring, case.dim), 7.0, dtype=case.dtype, device=dev)  # (a slot somebody used before)
    vr = torch.full((3, case.G, ring, case.vdim), 9.0, dtype=case.dtype, device=dev)
    part = torch.zeros(1 << 20, device=dev) if split else None
    out, at = [], 0
    for n in cuts:
        b = ops.PackedBatch([n], [1], [at], dev)
        mixed = {} if case.mix is None else dict(v_first=case.first[at:at + n].contiguous().to(dev), v_mix=case.mix)
        out.append(ops.window_attention(p[at:at + n].contiguous().to(dev), b, kr, vr, path=path, partials=part, **kw, **mixed))
        at += n
    assert at == case.T
    assert (kr[0] == 7).all() and (kr[2] == 7).all() and (vr[0] == 9).all() and (vr[2] == 9).all()
    return torch.cat(out)


SCALING = {"factor": 3.0, "low": 1.0, "high": 3.5, "original": 60}
ATTENTION = {
    "norms, some dimensions": (4, 2, 40, 24, {"base": 300.0, "dims": 16}, dict(norm=True)),
    "norms, mixed values": (6, 1, 64, 64, {"base": 1e4, "dims": 64}, dict(norm=True, mix=0.3)),
    "norms, no rotation, odd size": (3, 3, 13, 11, {"base": 1.0, "dims": 0}, dict(norm=True, mix=0.8)),
    "bounded, scaled": (8, 2, 128, 128, {"base": 5e3, "dims": 128, "scaling": SCALING}, dict(cap=2.0)),
    "bounded, odd pairs": (10, 2, 22, 18, {"base": 50.0, "dims": 6, "scaling": {"factor": 9.0, "low": 0.5, "high": 40.0, "original": 33}}, dict(cap=5.0, mix=0.5)),
    "plain, value far wider": (2, 1, 32, 200, {"base": 700.0, "dims": 30}, dict(mix=1.0)),
    "key wider": (5, 5, 96, 32, {"base": 1e4, "dims": 96}, dict(norm=True, cap=3.0, mix=0.25)),
    "wide": (2, 2, 200, 152, {"base": 1e4, "dims": 100}, dict(cap=1.0, mix=0.0)),
}


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", ATTENTION)
def test_attention(dev, dtype, name):
    H, G, dim, vdim, rot, kw = ATTENTION[name]
    T = 190
    case = Case(T, H, G, dim, vdim, rot, dtype, **kw)
    ref = case.reference()
    assert rel(run_portions(dev, case, [T]), ref) < TOL[dtype]
    for cuts in ([2] * 3 + [T - 6], [64, 1, 65, T - 130], [T - 60] + [1] * 60):
        assert rel(run_portions(dev, case, cuts), ref) < TOL[dtype], cuts
    assert rel(run_portions(dev, case, [90, T - 90], path=1), ref) < TOL[dtype]
    assert rel(run_portions(dev, case, [90, T - 130] + [1] * 40, ring=T + 5), ref) < TOL[dtype]


def test_attention_token_by_token_and_split(dev):
    for name in ("norms, mixed values", "bounded, odd pairs"):
        H, G, dim, vdim, rot, kw = ATTENTION[name]
        case = Case(90, H, G, dim, vdim, rot, torch.float32, seed=3, **kw)
        assert rel(run_portions(dev, case, [1] * 90), case.reference()) < TOL[torch.float32]
        case = Case(700, H, G, dim, vdim, rot, torch.float32, seed=4, **kw)
        assert rel(run_portions(dev, case, [660] + [1] * 40, split=True), case.reference()) < TOL[torch.float32]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_scores_far_beyond_their_bound(dev, dtype):
    """Without the bound one key would take everything; with it the weights of all that stand out are equal."""
    case = Case(150, 4, 2, 32, 16, {"base": 1e4, "dims": 8}, dtype, cap=1.5, gain=40.0, loud=3.0)
    free = Case(150, 4, 2, 32, 16, {"base": 1e4, "dims": 8}, dtype, gain=40.0, loud=3.0)
    ref = case.reference()
    assert rel(free.reference(), ref) > 1  # (it matters here)
    for cuts in ([150], [100] + [1] * 50):
        assert rel(run_portions(dev, case, cuts), ref) < TOL[dtype]


def test_far_key_among_thousands(dev):
    """One key at the start holds the answer of the last queries, in a prompt and decoded."""
    T = 1500
    case = Case(T, 2, 1, 64, 32, {"base": 1e4, "dims": 32}, torch.bfloat16, norm=True, gain=16.0, mix=0.4)
    ref = case.reference()
    assert rel(run_portions(dev, case, [T]), ref) < TOL[torch.bfloat16]
    assert rel(run_portions(dev, case, [700, 780] + [1] * 20, split=True), ref) < TOL[torch.bfloat16]


def test_bad_attention_arguments_are_errors_on_the_host(dev):
    from lit_llama_amd import _native as nat

    H, G, dim, vdim, rot, kw = ATTENTION["key wider"]
    case = Case(8, H, G, dim, vdim, rot, torch.float32, **kw)
    case.cap = -1.0
    with pytest.raises(nat.NativeError):
        run_portions(dev, case, [8])
    case.cap = 0.0
    inputs = case.inputs
    case.inputs = lambda d: (lambda p, k: (p, {n: v for n, v in k.items() if n != "unit_eps"}))(*inputs(d))  # factors without a norm
    with pytest.raises(nat.NativeError):
        run_portions(dev, case, [8])


# ---------------------------------------------------------------------------------------- state-space recurrence
def ssd_case(T, H, G, N, vdim, taps, dtype, seed=0, strong=False, bias=True):
    gen = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(s, generator=gen)
    sizes = {"g": H * vdim, "v": H * vdim, "k": G * N, "q": G * N, "a": H}
    off, n = {}, 0
    for name, s in sizes.items():
        off[name] = n
        n += pad16(s)
    p = rnd(T, n)
    if strong:  # steps that nearly erase the state next to ones that keep it
        p[::9, off["a"]:off["a"] + H] += 25
        p[1::2, off["a"]:off["a"] + H] -= 12
    p = p.to(dtype)
    w = dict(conv=tuple(0.5 * rnd(c, taps) for c in (G * N, G * N, H * vdim)), a_log=rnd(H) - 1, dt_bias=rnd(H), skip=1 + 0.5 * rnd(H))
    if bias:
        w["conv_bias"] = tuple(0.5 * rnd(c) for c in (G * N, G * N, H * vdim))
    d = p.double()
    part = lambda name: d[:, off[name]:off[name] + sizes[name]]
    zero = [torch.zeros(c).double() for c in (G * N, G * N, H * vdim)]
    q, k, v = (O.silu(O.short_conv(part(x), w["conv"][i].double(), w["conv_bias"][i].double() if bias else zero[i])) for i, x in enumerate("qkv"))
    o = O.state_space(v.view(T, H, vdim), k.view(T, G, N), q.view(T, G, N), O.softplus(part("a") + w["dt_bias"].double()), w["a_log"].double(), w["skip"].double())
    return p, o.reshape(T, -1) * O.silu(part("g")), off, w


def run_ssd(dev, p, off, w, H, G, N, vdim, taps, cuts, path=0):
    from lit_llama_amd import ops

    state = torch.full((3, H, N, vdim), 5.0, device=dev)
    ring = torch.full((3, taps, 2 * G * N + H * vdim), 3.0, dtype=p.dtype, device=dev)
    state[1] = 0
    kw = {n: tuple(t.to(dev) for t in v) if isinstance(v, tuple) else v.to(dev) for n, v in w.items()}
    out, at = [], 0
    for n in cuts:
        b = ops.PackedBatch([n], [1], [at], dev)
        out.append(ops.recurrent("ssd", p[at:at + n].contiguous().to(dev), b, state, off=off, kv_heads=G, conv_ring=ring, path=path, **kw))
        at += n
    assert at == p.shape[0]
    assert (state[0] == 5).all() and (state[2] == 5).all() and (ring[0] == 3).all()
    return torch.cat(out)


SSD = [(4, 2, 24, 40, 4), (3, 3, 64, 32, 2), (6, 1, 130, 70, 5), (2, 2, 16, 144, 1), (1, 1, 33, 17, 9), (8, 4, 128, 64, 3), (4, 1, 200, 16, 4), (5, 1, 7, 5, 2)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,N,vdim,taps", SSD)
def test_state_space(dev, dtype, H, G, N, vdim, taps):
    T = 150
    p, ref, off, w = ssd_case(T, H, G, N, vdim, taps, dtype, bias=H != 6)
    args = (off, w, H, G, N, vdim, taps)
    for cuts, path in (([T], 2), ([T], 1), ([64, T - 64], 0), ([2, 3, 60, T - 65], 0), ([T - 40] + [1] * 40, 0), ([1] * 12 + [T - 12], 2)):
        assert rel(run_ssd(dev, p, *args, cuts, path), ref) < 3e-5, (cuts, path)


def test_state_space_with_strong_decays(dev):
    p, ref, off, w = ssd_case(260, 4, 2, 32, 24, 4, torch.float32, strong=True)
    for cuts, path in (([260], 2), ([260], 1), ([100, 100] + [1] * 60, 0)):
        assert rel(run_ssd(dev, p, off, w, 4, 2, 32, 24, 4, cuts, path), ref) < 3e-5


def test_state_space_in_a_batch_of_unequal_portions(dev):
    from lit_llama_amd import ops

    H, G, N, vdim, taps = 4, 2, 48, 32, 4
    counts = (130, 3, 64, 65)
    cases = [ssd_case(n, H, G, N, vdim, taps, torch.float32) for n in counts]  # (one seed: the weights are the same)
    w0 = cases[0][3]
    gen = torch.Generator().manual_seed(5)
    ps = [torch.randn(c[0].shape, generator=gen) for c in cases]
    state = torch.zeros((4, H, N, vdim), device=dev)
    ring = torch.full((4, taps, 2 * G * N + H * vdim), 3.0, device=dev)
    kw = {n: tuple(t.to(dev) for t in v) if isinstance(v, tuple) else v.to(dev) for n, v in w0.items()}
    slots = [2, 0, 3, 1]
    whole = ops.recurrent("ssd", torch.cat(ps).to(dev), ops.PackedBatch(counts, slots, [0] * 4, dev), state, off=cases[0][2], kv_heads=G, conv_ring=ring, **kw)
    for p, part in zip(ps, whole.split(counts)):
        assert torch.equal(part, run_ssd(dev, p, cases[0][2], w0, H, G, N, vdim, taps, [len(p)], 2))


# ---------------------------------------------------------------------------------------- between sublayers
JOINS = [(1, 96), (5, 61), (3, 256), (7, 1024), (2, 1536), (6, 4096), (3, 5120), (2, 9000), (4, 130)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,W", JOINS)
def test_join(dev, dtype, rows, W):
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(W)
    rnd = lambda *s: torch.randn(s, generator=gen)
    tol = 2e-5 if dtype == torch.float32 else 6e-3  # (h alone is rounded)
    x, t, gate = rnd(rows, W) * 3, rnd(rows, W) * 7, rnd(rows, W) * 2
    post, nxt = (0.4 * rnd(W)).to(dtype), (0.4 * rnd(W)).to(dtype)
    g = lambda v: v.to(dev)
    norm = lambda v, w: O.rms_norm(v, w.double(), EPS)
    for n in (0, 1, 2, 5, 9):
        stream, avg = [rnd(rows, W) for _ in range(n)], rnd(n + 1)
        gate_dtype = (dtype, torch.float32)[n % 2]
        lg = gate.to(gate_dtype)
        want = x.double() + norm(t.double() * O.sigmoid(lg.double()), post)
        mean = O.depth_average(avg.double(), [*(s.double() for s in stream), want]) if n else want
        got = ops.join_rows(g(x), g(t), eps=EPS, gate=g(lg), post=g(post), stream=[g(s) for s in stream] if n else None, average=g(avg) if n else None,
                            next=g(nxt) if n != 2 else None, norm_add=1.0, dtype=dtype)
        assert rel(got[1], want) < 2e-5 and rel(got[0], mean) < 2e-5
        assert (got[2] is None) if n == 2 else rel(got[2], norm(mean, nxt)) < tol
    emb = rnd(17, W).to(dtype)
    toks = torch.randint(0, 17, (rows,), generator=gen, dtype=torch.int32)
    want = norm(emb[toks.long()].double(), post)
    got = ops.join_rows(None, eps=EPS, tokens=g(toks), embed=g(emb), post=g(post), next=g(nxt), norm_add=1.0, dtype=dtype)
    assert rel(got[0], want) < 2e-5 and rel(got[1], want) < 2e-5 and rel(got[2], norm(want, nxt)) < tol
    got = ops.join_rows(g(x), g(t), eps=EPS, dtype=dtype)  # a plain sum
    assert torch.equal(got[0].cpu(), x + t)


def test_norm_in_groups_that_are_not_heads(dev):
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(3)
    for H, vdim, groups in ((6, 20, 4), (3, 50, 1), (8, 48, 2), (4, 36, 12), (128, 64, 8)):
        y, z, w = (torch.randn(s, generator=gen) for s in ((5, H * vdim), (5, H * vdim), (H * vdim,)))
        for dtype in (torch.float32, torch.bfloat16):
            wd = w.to(dtype)
            want = O.gated_group_norm(y.double(), z.double(), wd.double(), groups, EPS)
            got = ops.norm_groups((y * O.silu(z)).to(dev), wd.to(dev), groups, EPS)
            assert rel(got, want) < (2e-5 if dtype == torch.float32 else 6e-3)


@pytest.mark.parametrize("M", [1, 6, 40, 300])
@pytest.mark.parametrize("N,K,f32", [(80, 128, True), (272, 384, False), (1024, 1024, False), (64, 4096, True)])
def test_products_with_a_bias(dev, M, N, K, f32):
    from lit_llama_amd import _native as nat
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(M)
    x = torch.randn((M, K), generator=gen).to(torch.bfloat16).to(dev)
    w = (torch.randn((N, K), generator=gen) * K ** -0.5).to(torch.bfloat16).to(dev)
    b = (torch.randn(N, generator=gen) * 2).to(dev)
    ref = x.cpu().double() @ w.cpu().double().T + b.cpu().double()
    stream = ops.repack_bf16(w, None, 1)
    y = torch.zeros((M, N), dtype=torch.float32 if f32 else torch.bfloat16, device=dev)
    a = nat.LinearArgs()
    a.fmt, a.R, a.w, a.N, a.K, a.x, a.x_dtype, a.M, a.ldx = nat.W_BF16, 1, nat.ptr(stream), N, K, nat.ptr(x), nat.BF16, M, K
    a.epi, a.y, a.y_dtype, a.ldy, a.alpha, a.bias, a.sz_dtype = nat.EPI_STORE, nat.ptr(y), nat.dtype_code(y.dtype), N, 1.0, nat.ptr(b), nat.dtype_code(torch.float32)
    ws = torch.empty(nat.lib().mi355_linear_gemm_workspace_bytes(M, K), dtype=torch.uint8, device=dev)
    if M <= 6:
        nat.check(nat.lib().mi355_linear_fast(C.byref(a), nat.stream_ptr()))
        assert rel(y, ref) < 1e-3
        y.zero_()
    nat.check(nat.lib().mi355_linear_gemm(C.byref(a), nat.ptr(ws), ws.numel(), nat.stream_ptr()))
    assert rel(y, ref) < 1e-3
    a.epi = nat.EPI_ACCUM
    assert nat.lib().mi355_linear_gemm(C.byref(a), nat.ptr(ws), ws.numel(), nat.stream_ptr()) == nat.E_ARG


# ---------------------------------------------------------------------------------------- experts
def experts_reference(h, w, spec):
    """The layer's sum, and the rows where no choice was close to another."""
    r = spec["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    clear = []
    for row in h:
        z = row @ w["router"].T
        c = torch.softmax(z, -1) + w["correction"]
        best = c.view(g["count"], -1).max(-1).values.sort(descending=True).values
        inside = c.view(g["count"], -1)[c.view(g["count"], -1).max(-1).values.argsort(descending=True)[:g["keep"]]].flatten().sort(descending=True).values
        gaps = [1.0]
        if g["keep"] < g["count"]:
            gaps.append(float(best[g["keep"] - 1] - best[g["keep"]]))
        if r["top"] < len(inside):
            gaps.append(float(inside[r["top"] - 1] - inside[r["top"]]))
        clear.append(min(gaps))
    return O.experts_ff(w, "", spec, h), torch.tensor(clear)


EXPERTS = [  # rows, width, experts, identity, top, groups, keep, ff
    (1, 72, 5, 3, 2, 4, 2, 24), (3, 200, 9, 0, 9, 1, 1, 17), (2, 136, 6, 2, 4, 2, 1, 40), (8, 384, 60, 10, 4, 7, 3, 130), (9, 130, 12, 4, 8, 4, 2, 33),
    (300, 64, 3, 1, 2, 2, 2, 40), (700, 256, 10, 6, 5, 4, 3, 96), (2500, 96, 4, 4, 3, 2, 1, 24), (40, 520, 1, 7, 3, 2, 2, 48), (5, 128, 200, 56, 16, 64, 9, 16)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,W,E,I,top,groups,keep,ff", EXPERTS)
def test_experts(dev, dtype, rows, W, E, I, top, groups, keep, ff):
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(rows)
    rnd = lambda *s, gain=1.0: (torch.randn(s, generator=gen) * gain * s[-1] ** -0.5).to(dtype)
    x = torch.randn((rows, W), generator=gen) * 3
    norm, router = (0.3 * torch.randn(W, generator=gen)).to(dtype), rnd(E + I, W, gain=2)
    corr = 0.3 * torch.randn(E + I, generator=gen) - 0.5  # (most choice scores are negative: a score of 0 would win)
    ws = [(rnd(ff, W, gain=2), rnd(W, ff, gain=2)) for _ in range(E)]
    w = {"router": router, **{f"e{e}.{n}": t for e, ts in enumerate(ws) for n, t in zip(("up", "down"), ts)}}
    w = {**{n: t.double() for n, t in w.items()}, "correction": corr.double()}
    spec = {"router": {"experts": E, "identity": I, "top": top, "groups": {"count": groups, "keep": keep}}}
    to = lambda ts: tuple(t.to(dev) for t in ts)
    common = dict(top=top, score="softmax", correction=corr.to(dev), groups=groups, keep_groups=keep, identity=I)
    fits = (lambda a, b: rel(a, b) < 5e-5) if dtype == torch.float32 else (lambda a, b: rows_off(a, b) < 0.02)
    hb = O.rms_norm(x.double(), norm.double(), 1e-4).to(dtype)  # rows as the sublayer's norm hands them over, with their logits: no choice is close
    logits = (hb.double() @ w["router"].T).float()
    ref, _ = experts_reference(hb.double(), w, spec)
    for path in ((0, 1, 2) if dtype == torch.bfloat16 else (0,)):
        if path == 1 and rows > 300:
            continue
        got = ops.experts(None, None, None, [to(t) for t in ws], h=hb.to(dev), logits=logits.to(dev), path=path, **common).cpu()
        assert torch.isfinite(got).all() and fits(got, ref), path
        if rows > 2 and path != 1:  # a row's result does not depend on its batch
            one = ops.experts(None, None, None, [to(t) for t in ws], h=hb[1:2].to(dev), logits=logits[1:2].to(dev), path=path, **common).cpu()
            assert rel(one, got[1:2]) < (2e-5 if dtype == torch.float32 else 0.02)
    h = O.rms_norm(x.double(), norm.double(), 1e-4)  # norm and router in the same launch
    want, gap = experts_reference(h, w, spec)
    clear = gap > (0.01 if dtype == torch.bfloat16 else 1e-5)
    got = ops.experts(x.to(dev), norm.to(dev), router.to(dev), [to(t) for t in ws], scale=1.0, eps=1e-4, norm_add=1.0, alpha=0.6, **common).cpu()
    if clear.any():
        assert fits((got - x)[clear], 0.6 * want[clear])


def test_all_choices_are_the_row_itself(dev):
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(1)
    for dtype in (torch.float32, torch.bfloat16):
        for rows in (1, 30):
            h = torch.randn((rows, 48), generator=gen).to(dtype)
            ws = [tuple(torch.randn(s, generator=gen).to(dtype).to(dev) for s in ((16, 48), (48, 16))) for _ in range(2)]
            corr = torch.tensor([-5.0, -5.0, 0.0, 0.0])
            logits = torch.randn((rows, 4), generator=gen)
            got = ops.experts(None, None, None, ws, h=h.to(dev), logits=logits.to(dev), top=2, score="softmax", correction=corr.to(dev), groups=2, keep_groups=1, identity=2)
            assert rel(got, h.double() * torch.softmax(logits.double(), -1)[:, 2:].sum(-1, keepdim=True)) < 1e-5


def test_bad_routers_are_errors_on_the_host(dev):
    from lit_llama_amd import _native as nat
    from lit_llama_amd import ops

    h = torch.zeros((2, 32), device=dev)
    ws = [(torch.zeros((16, 32), device=dev), torch.zeros((32, 16), device=dev))] * 6
    call = lambda **kw: ops.experts(None, None, None, ws, h=h, logits=torch.zeros((2, 6 + kw.get("identity", 0)), device=dev), **{"top": 2, "score": "softmax", **kw})
    call(groups=3, keep_groups=1)
    for kw in (dict(groups=4, keep_groups=1), dict(groups=3, keep_groups=4), dict(groups=6, keep_groups=1), dict(top=7), dict(score="sigmoid", groups=3, keep_groups=1)):
        with pytest.raises(nat.NativeError):
            call(**kw)


# ---------------------------------------------------------------------------------------- the model
def moe(experts=7, identity=2, top=3, ff=40, groups=(3, 2)):
    r = {"experts": experts, "top": top, "identity": identity, "groups": {"count": groups[0], "keep": groups[1]} if groups else None}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r}


def ssd(mlp=None, **kw):
    return {"type": "mamba2", "mixer": {"heads": 6, "groups": 2, "state": 24, "vdim": 20, "conv": 3, "norm_groups": 4, **kw}, "mlp": mlp}


def att(mlp=None, **kw):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": 6, "kv_heads": 2, "dim": 24, "vdim": 16, "rot": {"base": 900.0, "dims": 16}, "scale": 0.27, "v_mix": True, **kw}}


def cap(mlp=None, scaling=SCALING, **kw):
    return {"type": "attention_2", "mlp": mlp,
            "mixer": {"heads": 4, "kv_heads": 2, "dim": 40, "vdim": 16, "rot": {"base": 5e3, "dims": 40, "scaling": scaling}, "scale": 0.2, "softcap": 3.0,
                      "v_mix": True, **kw}}


def small_config(layers, **kw):
    return {"architecture": "Gurolix", "vocab": 211, "width": 104, "norm": {"eps": 3e-4}, "layers": layers, **kw}


CONFIGS = {
    "mixed": small_config([ssd(moe()), att(moe(groups=None)), ssd(None), cap(moe(9, 0, 3, 24, (3, 1))), att(None, v_mix=False), cap(moe(3, 5, 2, 16, (4, 2)))]),
    "odd sizes": small_config([cap(moe(4, 1, 2, 18, (1, 1)), heads=3, kv_heads=3, dim=10, vdim=7, rot={"base": 90.0, "dims": 6}, softcap=1.0),
                               ssd(moe(2, 1, 1, 9, None), heads=5, groups=1, state=18, vdim=9, conv=1, norm_groups=3),
                               att(None, heads=3, kv_heads=3, dim=14, vdim=7, rot={"base": 30.0, "dims": 14})], width=61, vocab=130, norm={"eps": 1e-3}),
    "whole tiles": small_config([att(moe(12, 4, 4, 128, (4, 2)), heads=8, kv_heads=2, dim=128, vdim=64, rot={"base": 1e4, "dims": 64}, scale=128 ** -0.5),
                                 ssd(moe(12, 4, 4, 128, (4, 2)), heads=16, groups=4, state=64, vdim=64, conv=4, norm_groups=4),
                                 cap(moe(12, 4, 4, 128, (4, 2)), scaling=None, heads=8, kv_heads=2, dim=64, vdim=64, rot={"base": 1e4, "dims": 64}, softcap=30.0)],
                                width=512, norm={"eps": 1e-5}),
}


def build(config, dtype, dev, seed=1):
    from lit_llama_amd import synth
    from lit_llama_amd.registry import build_model

    sd = synth.make_hybrid_state_dict(config, seed=seed)
    gen = torch.Generator().manual_seed(seed)
    for n in sd:
        if n.endswith("router"):
            sd[n] = (sd[n].float() * 2).to(sd[n].dtype)
        if n.endswith("correction") and dtype == torch.bfloat16:  # no choice is a rounding apart: every row goes where the restatement sends it
            sd[n] = (2.0 * torch.randperm(len(sd[n]), generator=gen) - len(sd[n])).to(sd[n].dtype)
    m = build_model(config, dtype, dev)
    m.load_state_dict(sd)
    return m, sd


def tokens_of(n, vocab=211, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close(got, ref, dtype):
    """float32: every value; bfloat16: rows (a norm behind a small result multiplies the rounding of a few)."""
    if dtype == torch.float32:
        return rel(got, ref) < 1e-4
    err = (got.double().cpu() - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()
    return float(torch.quantile(err, 0.97)) < 0.04 and float(err.mean()) < 0.015 and float(err.max()) < 0.3


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", CONFIGS)
def test_model_layer_by_layer_and_logits(dev, name, dtype):
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS[name]
    m, sd = build(config, dtype, dev)
    eng = m.engine()
    eng.ensure(2, 128)
    toks = tokens_of(61, config["vocab"])
    logits, trail = O.forward(config, sd, toks)
    for r in range(1, len(trail) + 1):
        s = eng.acquire()
        assert close(eng.residual_after([Entry(s, 0, toks, [])], r), trail[r - 1], dtype), r
        eng.release(s)
    s = eng.acquire()
    assert close(eng.step([Entry(s, 0, toks, range(61))]), logits, dtype)
    eng.release(s)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("name", CONFIGS)
def test_portions_batches_slots_and_decoding(dev, name, dtype):
    """Unequal requests in one batch, cut differently, decoded together, their slots used again: the logits of each alone."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS[name]
    m, sd = build(config, dtype, dev)
    eng = m.engine()
    eng.ensure(4, 200)
    seqs = [tokens_of(n, config["vocab"], seed=n) for n in (120, 9, 64, 33)]
    refs = [O.forward(config, sd, s)[0] for s in seqs]
    for first in ((80, 2, 31, 32), (64, 8, 1, 3), (1, 1, 1, 1)):  # (the second and third time in the slots of the first)
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


def test_a_large_batch_decodes_like_each_alone(dev):
    """Enough sequences that the products are tiled in a decode step."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS["whole tiles"]
    m, sd = build(config, torch.bfloat16, dev)
    eng = m.engine()
    eng.ensure(40, 64)
    seqs = [tokens_of(38 + i % 3, seed=i) for i in range(40)]
    slots = [eng.acquire() for _ in seqs]
    eng.step([Entry(s, 0, t[:30], []) for s, t in zip(slots, seqs)])
    rows = torch.stack([eng.step([Entry(s, 30 + k, t[30 + k:31 + k], [0]) for s, t in zip(slots, seqs)]).clone() for k in range(8)], 1)
    ref = torch.cat([O.forward(config, sd, seqs[i][:38])[0][30:] for i in (0, 11, 39)])
    assert close(torch.cat([rows[i] for i in (0, 11, 39)]), ref, torch.bfloat16)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_step_larger_than_the_scratch_is_cut(dev, dtype):
    from lit_llama_amd.hybrid_engine import Entry, HybridEngine

    config = CONFIGS["mixed"]
    m, sd = build(config, dtype, dev)
    eng = HybridEngine(m, max_rows=48)
    eng.ensure(3, 140)
    eng.ensure(3, 200)  # (longer sequences: caches are laid out anew)
    seqs = [tokens_of(n, seed=n) for n in (130, 17, 60)]
    slots = [eng.acquire() for _ in seqs]
    places = [sorted({0, 5, len(t) // 2, len(t) - 2, len(t) - 1}) for t in seqs]
    out = eng.step([Entry(s, 0, t, w) for s, t, w in zip(slots, seqs, places)])
    ref = torch.cat([O.forward(config, sd, t)[0][w] for t, w in zip(seqs, places)])
    assert close(out, ref, dtype)


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
    x = generate_batch(m, [prompts[0], prompts[2]], 8, temperature=0.9, top_k=50, seed=3)
    assert x == generate_batch(m, [prompts[0], prompts[2]], 8, temperature=0.9, top_k=50, seed=3)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_long_decoding_matches_the_prompt_pass(dev, dtype):
    """Hundreds of decoded tokens (graphs replayed, eager work in between) against one prompt pass."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS["mixed"]
    m, sd = build(config, dtype, dev)
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
    ref = O.forward(config, sd, toks)[0]
    assert close(whole, ref, dtype) and close(torch.cat(rows), ref, dtype)


def test_a_far_token_reaches_the_logits(dev):
    """Another first token changes the last logits as the restatement says, decoded and in a prompt."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS["mixed"]
    m, sd = build(config, torch.float32, dev)
    eng = m.engine()
    eng.ensure(2, 300)
    toks = tokens_of(260, seed=4)
    other = [(toks[0] + 1) % 211, *toks[1:]]
    want = O.forward(config, sd, toks)[0][-1] - O.forward(config, sd, other)[0][-1]
    rows = []
    for seq in (toks, other):
        s = eng.acquire()
        eng.step([Entry(s, 0, seq[:250], [])])
        for i in range(250, 260):
            out = eng.step([Entry(s, i, seq[i:i + 1], [0])]).clone()
        rows.append(out[0])
        eng.release(s)
        s = eng.acquire()
        assert rel(eng.step([Entry(s, 0, seq, [259])])[0], out[0]) < 1e-4
        eng.release(s)
    got = (rows[0] - rows[1]).double().cpu()
    assert float((got - want).abs().max()) < 0.1 * float(want.abs().max())


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
