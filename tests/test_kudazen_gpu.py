"""The Kudazen design on the GPU against the plain restatement in oracle/kudazen.py: each mechanism's kernels alone, then the model through its
engine, scheduler and generate().  Inputs are made so that a fault shows: keys that stand out just inside and just outside a chunk, far keys
among hundreds, loud sinks, states that decay slowly and at once, sizes that differ from each other."""
import ctypes as C
import json

import pytest
import torch

from oracle import kudazen as O

pytestmark = pytest.mark.gpu


def rel(got, ref):
    """Largest deviation over the reference's root mean square; a bf16 result has its last rounding (2^-8 of the value) for free."""
    free = 2.0 ** -8 if got.dtype == torch.bfloat16 else 0.0
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    assert got.shape == ref.shape
    return float(((got - ref).abs() - free * ref.abs()).max() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


TOL = {torch.float32: 2e-5, torch.bfloat16: 4e-2}


def rows(got, ref):
    """The largest error of a row over the row's own size, root mean squares (bf16 operands round every score a little)."""
    e = got.detach().double().cpu() - ref
    return float((e.pow(2).mean(-1) / ref.pow(2).mean(-1)).sqrt().max())


def near(got, ref):
    return rel(got, ref) < TOL[torch.float32] if got.dtype == torch.float32 else rows(got, ref) < TOL[torch.bfloat16]


EPS = 2e-3
pad16 = lambda n: (n + 15) // 16 * 16


# ---------------------------------------------------------------------------------------- norm in groups, token shift
NORMS = [(96, 3), (100, 4), (61, 1), (512, 2), (768, 1), (2048, 8), (4096, 2), (5120, 4), (9000, 2), (640, 64), (1280, 5)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W,groups", NORMS)
def test_norm_in_groups(dev, dtype, W, groups):
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(W)
    x = torch.randn((37, W), generator=gen) * 10.0 ** torch.randint(-2, 3, (groups,), generator=gen).repeat_interleave(W // groups)
    scale = (1 + 0.2 * torch.randn(W, generator=gen)).to(dtype)
    ref = O.group_norm(x.double(), scale.double(), groups, EPS)
    assert rel(ops.norm_groups(x.to(dev), scale.to(dev), groups, EPS), ref) < (2e-6 if dtype == torch.float32 else 1e-6)
    want = torch.tensor([36, 0, 7, 7, 19], dtype=torch.int32)
    assert rel(ops.norm_groups(x.to(dev), scale.to(dev), groups, EPS, want=want.to(dev)), ref[want.long()]) < 2e-6


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("W,groups", NORMS)
def test_token_shift(dev, dtype, W, groups):
    """Unequal sequences in portions; a used slot starts from zero; slots of others stay as they are."""
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(W)
    xs = [torch.randn((n, W), generator=gen) for n in (31, 8, 17)]
    scale, mu = (1 + 0.2 * torch.randn(W, generator=gen)).to(dtype), torch.rand((5, W), generator=gen)
    hs = [O.group_norm(x.double(), scale.double(), groups, EPS) for x in xs]
    refs = [torch.stack([h, *(O.token_mix(h, m.double()) for m in mu)]) for h in hs]
    shift = torch.full((5, W), 7.0, device=dev)
    slots, at = [3, 0, 2], [0, 0, 0]
    got = [[] for _ in xs]
    for counts in ((9, 1, 2), (1, 1, 1), (4, 0, 6), (2, 2, 2), (15, 4, 6)):
        live = [i for i in range(3) if counts[i]]
        b = ops.PackedBatch([counts[i] for i in live], [slots[i] for i in live], [at[i] for i in live], dev)
        x = torch.cat([xs[i][at[i]:at[i] + counts[i]] for i in live]).to(dev)
        h, mix = ops.norm_groups(x, scale.to(dev), groups, EPS, batch=b, mu=mu.to(dev), shift=shift)
        r = 0
        for i in live:
            got[i].append(torch.cat([h[None], mix])[:, r:r + counts[i]])
            r += counts[i]
            at[i] += counts[i]
    for i in range(3):
        assert at[i] == len(xs[i])
        assert rel(torch.cat(got[i], 1), refs[i]) < (3e-6 if dtype == torch.float32 else 2e-3)
        assert rel(shift[slots[i]], hs[i][-1]) < 3e-6
    assert (shift[[1, 4]] == 7).all()


# ---------------------------------------------------------------------------------------- chunk attention
class Chunks:
    """Packed projections of one sequence: keys at the first and last place of chunks (and far inside them) stand out for the queries at both
    sides of an edge."""

    def __init__(self, T, H, G, dim, vdim, size, dtype, seed=0):
        gen = torch.Generator().manual_seed(seed)
        self.T, self.H, self.G, self.dim, self.vdim, self.size, self.dtype = T, H, G, dim, vdim, size, dtype
        self.off_k = pad16(H * dim)
        self.off_v = self.off_k + pad16(G * dim)
        p = torch.randn((T, self.off_v + pad16(G * vdim)), generator=gen)
        q, k, v = p[:, :H * dim].view(T, H, dim), p[:, self.off_k:self.off_k + G * dim].view(T, G, dim), p[:, self.off_v:self.off_v + G * vdim].view(T, G, vdim)
        v *= 5.0 ** torch.randint(-2, 3, (T, 1, 1), generator=gen)  # (the size of a value must not count)
        self.temp = 0.5 + torch.rand(H, generator=gen)
        if H > 2:
            self.temp[1] *= -1
        step = size or T
        for c in range(0, T, step):
            for j, at in ((c, (c + step - 1, c + step)), (c + step - 1, (c + step - 1, c + step, c + step + 3)), (c + step // 2, (c + step - 1, c + step + 1))):
                if j < T:
                    loud = torch.randn((G, dim), generator=gen)
                    loud *= dim ** 0.5 / loud.norm(dim=-1, keepdim=True)
                    k[j] = 2 * loud
                    for i in at:
                        if i < T:
                            q[i] = 3 * (loud.repeat_interleave(H // G, 0) * self.temp.sign()[:, None])
        self.p, self.scale = p.to(dtype), 10.0 / (6 * dim)  # (keys that stand out: a score of 10)

    def reference(self):
        d, T = self.p.double(), self.T
        q, k = d[:, :self.H * self.dim].view(T, self.H, self.dim), d[:, self.off_k:self.off_k + self.G * self.dim].view(T, self.G, self.dim)
        v = O.unit_rms(d[:, self.off_v:self.off_v + self.G * self.vdim].view(T, self.G, self.vdim), EPS)
        return O.chunk_attention(q, k, v, self.scale * self.temp.double(), O.slopes(self.H), self.size).reshape(T, -1)

    def run(self, dev, cuts, ring, path=0, split=False):
        from lit_llama_amd import ops

        shape = (3, self.G, ring)
        kr, vr = (torch.full((*shape, n), f, dtype=self.dtype, device=dev) for n, f in ((self.dim, 7.0), (self.vdim, 9.0)))
        part = torch.zeros(1 << 20, device=dev) if split else None
        slope = torch.tensor(O.slopes(self.H), dtype=torch.float32, device=dev)
        out, at = [], 0
        for n in cuts:
            b = ops.PackedBatch([n], [1], [at], dev)
            out.append(ops.window_attention(self.p[at:at + n].contiguous().to(dev), b, kr, vr, heads=self.H, scale=self.scale, window=self.size or 1 << 30,
                                            chunked=self.size is not None, off_q=0, off_k=self.off_k, off_v=self.off_v, path=path, partials=part,
                                            head_scale=self.temp.to(dev), slope=slope, unit_v_eps=EPS))
            at += n
        assert at == self.T and (kr[0] == 7).all() and (kr[2] == 7).all() and (vr[0] == 9).all()
        return torch.cat(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,dim,vdim,size", [(4, 2, 40, 24, 37), (6, 1, 64, 64, 64), (3, 3, 18, 10, 20), (8, 2, 128, 128, 130), (10, 1, 72, 200, 1),
                                               (2, 1, 32, 16, 500), (5, 5, 24, 56, 3), (16, 1, 96, 80, 48), (2, 2, 160, 96, 70), (4, 1, 16, 16, None)])
def test_chunk_attention(dev, dtype, H, G, dim, vdim, size):
    T = 210
    case = Chunks(T, H, G, dim, vdim, size, dtype)
    ref = case.reference()
    ring = min(size or T, T)
    assert rel(case.run(dev, [T], ring), ref) < TOL[dtype]
    for cuts in ([2] * 3 + [T - 6], [100, 1, 64, T - 165], [1, 1, 1, T - 3], [T - 70] + [1] * 70, [37, 37, 63, T - 137]):
        assert rel(case.run(dev, cuts, ring), ref) < TOL[dtype], cuts
    assert rel(case.run(dev, [90, T - 90], ring, path=1), ref) < TOL[dtype]
    assert rel(case.run(dev, [90, T - 140] + [1] * 50, ring + 5), ref) < TOL[dtype]


def test_chunk_attention_token_by_token_and_split(dev):
    case = Chunks(90, 4, 2, 32, 16, 21, torch.float32, seed=3)
    assert rel(case.run(dev, [1] * 90, 21), case.reference()) < TOL[torch.float32]
    case = Chunks(700, 4, 1, 64, 32, 640, torch.float32)
    assert rel(case.run(dev, [580] + [1] * 120, 640, split=True), case.reference()) < TOL[torch.float32]


# ---------------------------------------------------------------------------------------- latent attention
class Latents:
    """Input projections of one sequence.  A few positions' latents or rotated parts stand out for far queries."""

    def __init__(self, T, H, dim, rot, vdim, rq, R, dtype, seed=0, sink=None):
        gen = torch.Generator().manual_seed(seed)
        self.T, self.dtype, self.m = T, dtype, {"heads": H, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": rq, "kv_rank": R,
                                                "rot": {"base": 300.0, "dims": rot}}
        rnd = lambda *s: torch.randn(s, generator=gen)
        self.w = {"uq": rnd(H * (dim + rot), rq) * rq ** -0.5, "uk": rnd(H * dim, R) * R ** -0.5, "uv": rnd(H * vdim, R) * R ** -0.5}
        self.w = {n: t.to(dtype) for n, t in self.w.items()}
        self.n = {"q_norm": 1 + 0.2 * rnd(rq), "c_norm": 1 + 0.2 * rnd(R), "sink": rnd(H) * 2 + 1 if sink is None else torch.full((H,), float(sink))}
        self.off_c = pad16(rq)
        p = rnd(T, self.off_c + pad16(R + rot)) * 4.0 ** torch.randint(-2, 2, (T, 1), generator=gen)
        c = p[:, self.off_c:self.off_c + R + rot]
        c[:, R:] = rnd(T, rot)
        # the key that a query of latent z looks for: pull z through head 0's weights
        back = self.w["uk"].float()[:dim].T @ self.w["uq"].float()[:dim]
        for j in {0, 1, T // 3, 63 % T, 64 % T, T // 2}:
            z = rnd(rq)
            c[j, :R] = back @ (z * self.n["q_norm"] / z.pow(2).mean().sqrt()) * 3
            for i in (j, T - 1 - j // 2, min(T - 1, j + 100)):
                if i >= j:
                    p[i, :rq] = z * 2
        self.p = p.to(dtype)
        q, k, _ = self.parts()
        self.m["scale"] = 9.0 / float((q.transpose(0, 1) @ k.permute(1, 2, 0)).tril().abs().max()) if T > 1 else 1.0  # (the loudest score: 9)

    def parts(self):
        d, m, T = self.p.double(), self.m, self.T
        H, n, R = m["heads"], m["dim"], m["kv_rank"]
        w = {k: t.double() for k, t in {**self.w, **self.n}.items()}
        eye = {"dq": torch.eye(m["q_rank"]), "dkv": torch.eye(R + m["rot_dim"])}
        parts = {"x." + k: t.double() for k, t in {**eye, "dq.norm": w["q_norm"], "dkv.norm": w["c_norm"], "uq": w["uq"]}.items()}
        q = O.latent_parts({**parts, "x.dkv": torch.zeros((R + m["rot_dim"], m["q_rank"])).double()}, "x.", m, d[:, :m["q_rank"]], EPS)[0]
        parts["x.dq"] = torch.zeros((m["q_rank"], R + m["rot_dim"])).double()
        _, c, kr = O.latent_parts(parts, "x.", m, d[:, self.off_c:self.off_c + R + m["rot_dim"]], EPS)
        return q, torch.cat([(c @ w["uk"].T).view(T, H, n), kr[:, None].expand(T, H, m["rot_dim"])], -1), (c @ w["uv"].T).view(T, H, -1)

    def reference(self):
        return O.sink_attention(*self.parts(), self.m["scale"], self.n["sink"].double()).reshape(self.T, -1)

    def kw(self, dev):
        m = self.m
        inv = torch.tensor([m["rot"]["base"] ** (-2.0 * i / m["rot_dim"]) for i in range(m["rot_dim"] // 2)], dtype=torch.float64, device=dev)
        w = {n: t.to(dev) for n, t in {**self.w, **self.n}.items()}
        return dict(w=w, heads=m["heads"], dim=m["dim"], rot_dim=m["rot_dim"], vdim=m["vdim"], off_q=0, off_c=self.off_c, scale=m["scale"], eps=EPS, inv_freq=inv)

    def cache(self, dev, slots=3, rows=None):
        return torch.full((slots, rows or self.T, self.m["kv_rank"] + self.m["rot_dim"]), float("nan"), dtype=self.dtype, device=dev)

    def run(self, dev, cuts, **kw):
        from lit_llama_amd import ops

        cache, out, at = self.cache(dev), [], 0
        for n in cuts:
            b = ops.PackedBatch([n], [1], [at], dev)
            out.append(ops.latent_attention(self.p[at:at + n].contiguous().to(dev), b, cache, **self.kw(dev), **kw))
            at += n
        assert at == self.T and cache[[0, 2]].isnan().all()
        return torch.cat(out)


LATENTS = [(8, 32, 16, 48, 80, 72), (3, 24, 16, 40, 40, 48), (5, 18, 6, 10, 33, 29), (20, 128, 64, 128, 192, 512), (1, 64, 8, 32, 24, 160), (33, 16, 16, 24, 64, 264),
           (2, 40, 24, 72, 136, 40)]


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,dim,rot,vdim,rq,R", LATENTS)
def test_latent_attention(dev, dtype, H, dim, rot, vdim, rq, R):
    T = 170
    case = Latents(T, H, dim, rot, vdim, rq, R, dtype)
    ref = case.reference()
    assert near(case.run(dev, [T]), ref)
    for cuts in ([2] * 3 + [T - 6], [100, 1, 64, T - 165], [1, 1, 1, T - 3], [T - 70] + [1] * 70, [63, 2, T - 65], [64, 9, 7, T - 80]):
        assert near(case.run(dev, cuts), ref), cuts
    vec = dtype == torch.bfloat16 and not (dim % 8 or rot % 8 or vdim % 8 or R % 8)
    for path in (1, 2, 3) if vec else (1,):
        assert near(case.run(dev, [60, T - 60], path=path), ref), path
    # few records: rows one after the other, whole sequences without splits
    assert near(case.run(dev, [90] + [5] * 16, partials_bytes=4 * H * (R + 4) * 3, path=1), ref)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("sink", [-60.0, 25.0])
def test_latent_sinks_far_above_and_below_the_scores(dev, dtype, sink):
    case = Latents(150, 4, 32, 16, 24, 48, 64, dtype, sink=sink)
    for cuts in ([150], [100] + [1] * 50):
        got = case.run(dev, cuts)
        assert torch.isfinite(got).all() and (rel(got, case.reference()) < 1e-4 if dtype == torch.float32 else rows(got, case.reference()) < 0.1)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_latent_batches_of_unequal_sequences(dev, dtype):
    """Three sequences over slots in another order, expanded two at a time and all at once, then decoded together; long caches."""
    from lit_llama_amd import ops

    T = 150
    cases = [Latents(T, 6, 32, 16, 24, 48, 64, dtype, seed=s) for s in range(3)]
    for c in cases[1:]:
        c.w, c.n, c.m = cases[0].w, cases[0].n, cases[0].m
    refs = [c.reference() for c in cases]
    for expand in (None, 300, 150):
        cache, at, got, slots = cases[0].cache(dev, 4, 400), [0, 0, 0], [[], [], []], [2, 3, 0]
        for counts in ((120, 9, 60), (20, 3, 70), *[(1, 1, 1)] * 10):
            b = ops.PackedBatch(counts, slots, at, dev)
            x = torch.cat([c.p[a:a + n] for c, a, n in zip(cases, at, counts)]).to(dev)
            y = ops.latent_attention(x, b, cache, **cases[0].kw(dev), expand_rows=expand)
            for i, part in enumerate(y.split(list(counts))):
                got[i].append(part)
                at[i] += counts[i]
        for i in range(3):
            assert near(torch.cat(got[i]), refs[i][:at[i]])
        assert cache[1].isnan().all()


# ---------------------------------------------------------------------------------------- WKV
def wkv_case(T, H, dim, rank, dtype, seed=0, strong=False):
    gen = torch.Generator().manual_seed(seed)
    sizes = dict(q=H * dim, k=H * dim, v=H * dim, g=H * dim, a=rank)
    off, n = {}, 0
    for name, s in sizes.items():
        off[name] = n
        n += pad16(s)
    p = torch.randn((T, n), generator=gen)
    w = dict(head_norm=1 + 0.2 * torch.randn(H * dim, generator=gen), eps=3e-3, bonus=torch.randn(H * dim, generator=gen),
             a2=torch.randn((H * dim, rank), generator=gen) * rank ** -0.5, a2_bias=torch.randn(H * dim, generator=gen) - 3)
    if strong:  # channels that forget at once, at some tokens, next to ones that never do
        w["a2_bias"][::3] += 8
        w["a2_bias"][1::3] -= 6
        w["a2"][::2] *= 6
    p = p.to(dtype)
    d = p.double()
    cut = lambda name: d[:, off[name]:off[name] + sizes[name]]
    z = torch.tanh(cut("a")) @ w["a2"].double().T + w["a2_bias"].double()
    o = O.wkv(*(cut(s).view(T, H, dim) for s in "qkv"), O.channel_decay(z).view(T, H, dim), w["bonus"].double().view(H, dim))
    g = cut("g")
    ref = O.unit_rms(o, 3e-3).reshape(T, -1) * w["head_norm"].double() * (g * torch.sigmoid(g))
    return p, ref, off, w


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,dim,rank,strong", [(6, 40, 12, False), (3, 20, 5, False), (2, 128, 64, False), (1, 200, 33, False), (9, 8, 1, False), (4, 64, 24, True),
                                               (2, 100, 96, True)])
def test_wkv(dev, dtype, H, dim, rank, strong):
    from lit_llama_amd import ops

    T = 150
    p, ref, off, w = wkv_case(T, H, dim, rank, dtype, strong=strong)
    w = {n: t.to(dev) if torch.is_tensor(t) else t for n, t in w.items()}
    tol = 5e-5 if dtype == torch.float32 else 2e-3
    for cuts, path in (([T], 0), ([T], 1), ([T], 2), ([2, 2, 64, 3, T - 71], 0), ([1, 63, 65, 1, T - 130], 2), ([T - 40] + [1] * 40, 0), ([17] * 8 + [T - 136], 0)):
        state = torch.zeros((3, H, dim, dim), device=dev)
        state[[0, 2]] = 5.0
        out, at = [], 0
        for n in cuts:
            b = ops.PackedBatch([n], [1], [at], dev)
            out.append(ops.recurrent("wkv", p[at:at + n].contiguous().to(dev), b, state, off=off, kv_heads=H, path=path if n > 1 else 0, **w))
            at += n
        assert at == T and rel(torch.cat(out), ref) < tol, (cuts, path)
        assert (state[[0, 2]] == 5).all()


# ---------------------------------------------------------------------------------------- products
def linear_args(x, w, y, epi, K, N, R=1):
    from lit_llama_amd import _native as nat

    a = nat.LinearArgs()
    a.fmt, a.R, a.w, a.N, a.K, a.x, a.x_dtype, a.M, a.ldx = nat.W_BF16, R, nat.ptr(w), N, K, nat.ptr(x), nat.BF16, x.shape[0], x.stride(0)
    a.epi, a.y, a.y_dtype, a.ldy, a.alpha = epi, nat.ptr(y), nat.BF16, y.stride(0), 1.0
    return a


@pytest.mark.parametrize("M", [1, 5, 40, 300])
@pytest.mark.parametrize("N,K,limit", [(80, 128, 1.5), (272, 384, 0.3), (1024, 256, 7.0)])
def test_clamped_gate_product(dev, M, N, K, limit):
    from lit_llama_amd import _native as nat
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(M)
    x = (torch.randn((M, K), generator=gen) * 2).to(torch.bfloat16).to(dev)
    g, u = ((torch.randn((N, K), generator=gen) * K ** -0.5).to(torch.bfloat16).to(dev) for _ in range(2))
    xd = x.cpu().double()
    ref = O.clamped_gate(xd @ g.cpu().double().T, xd @ u.cpu().double().T, limit)
    y = torch.zeros((M, N), dtype=torch.bfloat16, device=dev)
    w = ops.repack_bf16(g, u, 2)
    a = linear_args(x, w, y, nat.EPI_CLAMPGLU, K, N, 2)
    a.limit = limit
    ws = torch.empty(nat.lib().mi355_linear_gemm_workspace_bytes(M, K), dtype=torch.uint8, device=dev)
    if M <= 5:
        nat.check(nat.lib().mi355_linear_fast(C.byref(a), nat.stream_ptr()))
        assert rel(y, ref) < 0.01
        y.zero_()
    nat.check(nat.lib().mi355_linear_gemm(C.byref(a), nat.ptr(ws), ws.numel(), nat.stream_ptr()))
    assert rel(y, ref) < 0.01


@pytest.mark.parametrize("M", [9, 130, 600])
@pytest.mark.parametrize("part,n,K", [(256, 3, 256), (512, 4, 128), (256, 1, 1024)])
def test_product_of_operand_slices(dev, M, part, n, K):
    from lit_llama_amd import _native as nat
    from lit_llama_amd import ops

    gen = torch.Generator().manual_seed(M)
    x = torch.randn((n, M + 3, K), generator=gen).to(torch.bfloat16).to(dev)
    w = (torch.randn((n * part, K), generator=gen) * K ** -0.5).to(torch.bfloat16).to(dev)
    y = torch.zeros((M, n * part), dtype=torch.bfloat16, device=dev)
    stream = ops.repack_bf16(w, None, 1)
    a = linear_args(x[0, :M], stream, y, nat.EPI_STORE, K, n * part)
    a.slice_rows, a.slice_stride = part, x.stride(0)
    ws = torch.empty(nat.lib().mi355_linear_gemm_workspace_bytes(M, K), dtype=torch.uint8, device=dev)
    nat.check(nat.lib().mi355_linear_gemm(C.byref(a), nat.ptr(ws), ws.numel(), nat.stream_ptr()))
    ref = torch.cat([x[i, :M].cpu().double() @ w[i * part:(i + 1) * part].cpu().double().T for i in range(n)], 1)
    assert rel(y, ref) < 0.01
    a.slice_rows = 128  # (not whole row blocks)
    assert nat.lib().mi355_linear_gemm(C.byref(a), nat.ptr(ws), ws.numel(), nat.stream_ptr()) == nat.E_ARG


# ---------------------------------------------------------------------------------------- the model
def latent(**kw):
    return {"type": "latent_attention", "mlp": {"kind": "dense", "ff": 72, "limit": 0.9},
            "mixer": {"heads": 5, "dim": 24, "rot_dim": 16, "vdim": 40, "q_rank": 56, "kv_rank": 48, "rot": {"base": 2000.0, "dims": 16}, "scale": 0.21, **kw}}


def chunk(**kw):
    return {"type": "attention", "mlp": {"kind": "dense", "ff": 100, "limit": 2.0},
            "mixer": {"heads": 6, "kv_heads": 2, "dim": 24, "vdim": 16, "scale": 0.3, "mask": {"size": 19}, **kw}}


def wkv(heads=4, dim=24, limit=1.1, ff=60):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "mlp": {"kind": "dense", "ff": ff, "limit": limit}}


def small_config(layers, **kw):
    return {"architecture": "Kudazen", "vocab": 211, "width": 104, "norm": {"eps": 3e-4, "groups": 4}, "layers": layers, **kw}


CONFIGS = {
    "mixed": small_config([chunk(), latent(), wkv(), {**wkv(3, 40), "mlp": None}, {**chunk(), "weights_of": 0}, {**latent(), "weights_of": 1},
                           {**wkv(), "weights_of": 2}]),
    "odd sizes": small_config([latent(heads=3, dim=10, rot_dim=6, vdim=14, q_rank=21, kv_rank=18, rot={"base": 90.0, "dims": 6}), wkv(3, 18, 0.4, 33),
                               {**chunk(heads=3, kv_heads=3, dim=10, vdim=18, mask={"size": 33}), "mlp": None}, chunk(heads=2, kv_heads=1, dim=6, vdim=10, mask=None)],
                              width=61, vocab=130, norm={"eps": 1e-3, "groups": 1}),
    "whole tiles": small_config([wkv(4, 64, 1.5, 256), latent(heads=18, dim=32, rot_dim=32, vdim=32, q_rank=128, kv_rank=264, rot={"base": 2000.0, "dims": 32}),
                                 chunk(heads=4, kv_heads=4, dim=160, vdim=64, mask={"size": 40}), {**wkv(4, 64, 1.5, 256), "weights_of": 0}],
                                width=512, norm={"eps": 1e-5, "groups": 2}),
}


def build(config, dtype, dev, seed=1):
    from lit_llama_amd import synth
    from lit_llama_amd.registry import build_model

    sd = synth.make_hybrid_state_dict(config, seed=seed, rank=11)
    m = build_model(config, dtype, dev)
    m.load_state_dict(sd)
    return m, sd


def tokens_of(n, vocab=211, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close(got, ref, dtype):
    if dtype == torch.float32:
        return rel(got, ref) < 1e-4
    err = (got.double().cpu() - ref).pow(2).mean(-1).sqrt() / ref.pow(2).mean().sqrt()
    return float(err.max()) < 0.06 and float(err.mean()) < 0.02


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
    for i in (0, 11, 39):
        assert close(rows[i], O.forward(config, sd, seqs[i][:38])[0][30:], torch.bfloat16)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_a_step_larger_than_the_scratch_is_cut(dev, dtype):
    from lit_llama_amd.hybrid_engine import Entry, HybridEngine

    config = CONFIGS["mixed"]
    m, sd = build(config, dtype, dev)
    eng = HybridEngine(m, max_rows=48)
    eng.ensure(3, 140)
    eng.ensure(3, 200)  # (longer sequences: caches and scratch are laid out anew)
    seqs = [tokens_of(n, seed=n) for n in (130, 17, 60)]
    slots = [eng.acquire() for _ in seqs]
    out = eng.step([Entry(s, 0, t, [0, len(t) - 1]) for s, t in zip(slots, seqs)])
    ref = torch.cat([O.forward(config, sd, t)[0][[0, len(t) - 1]] for t in seqs])
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
    fresh, _ = build(config, torch.float32, dev)  # a batch behind generate() that needs a longer cache than its sequence
    lit_llama_amd.generate(fresh, torch.tensor([1, 2, 3], device=dev), 2, top_k=1)
    assert generate_batch(fresh, prompts[:2], 10, top_k=1) == outs[:2]
    x = generate_batch(m, [prompts[0], prompts[2]], 8, temperature=0.9, top_k=50, seed=3)
    assert x == generate_batch(m, [prompts[0], prompts[2]], 8, temperature=0.9, top_k=50, seed=3)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_long_decoding_matches_the_prompt_pass(dev, dtype):
    """Hundreds of decoded tokens (chunks end inside them, graphs replayed, eager work in between) against one prompt pass."""
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
