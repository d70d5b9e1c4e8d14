"""The Sekulorn design on the GPU against the plain restatement in oracle/sekulorn.py: each mechanism's kernels alone, then the model through
its engine, scheduler and generate().  Inputs are made so that a fault shows: keys that stand out just inside and just outside a window,
states that decay slowly, sizes that differ from each other."""
import json

import pytest
import torch

from oracle import sekulorn as O

pytestmark = pytest.mark.gpu


def rel(got, ref):
    """Largest deviation over the reference's root mean square; a bf16 result has its last rounding (2^-8 of the value) for free."""
    free = 2.0 ** -8 if got.dtype == torch.bfloat16 else 0.0
    got, ref = got.detach().double().cpu(), ref.detach().double().cpu()
    assert got.shape == ref.shape
    return float(((got - ref).abs() - free * ref.abs()).max() / ref.pow(2).mean().sqrt().clamp_min(1e-30))


TOL = {torch.float32: 2e-5, torch.bfloat16: 4e-2}  # (the tiles round rotated q and the weights to bf16 in front of loud scores)


# ---------------------------------------------------------------------------------------- window attention
def attention_case(T, H, G, dim, vdim, window, rot, dtype, seed=0, gate=True):
    """Packed projections of one sequence and the oracle's output.  Row window is asked for by three queries: it is the largest key for
    the query that just sees it and for the one that just does not."""
    gen = torch.Generator().manual_seed(seed)
    pad = lambda n: (n + 15) // 16 * 16
    off_q, off_k = 0, pad(H * dim)
    off_v = off_k + pad(G * dim)
    off_g = off_v + pad(G * vdim)
    p = torch.randn((T, off_g + pad(H)), generator=gen)
    q, k, v = p[:, :H * dim].view(T, H, dim), p[:, off_k:off_k + G * dim].view(T, G, dim), p[:, off_v:off_v + G * vdim].view(T, G, vdim)
    for j in range(0, T - 1, max(1, T // 7)):  # key j stands out for the queries at both sides of the window's edge
        loud = torch.randn((G, dim), generator=gen)
        loud[:, :rot] = 0  # (unrotated dimensions: the same direction at every position)
        if dim > rot:
            loud = loud / loud.norm(dim=-1, keepdim=True) * dim ** 0.5
            k[j] = 2 * loud
            for i in (j + window - 1, j + window):
                if i < T:
                    q[i] = 2 * loud.repeat_interleave(H // G, 0)
            v[j] += 3
    p = p.to(dtype)
    pd = p.double()
    base = 5000.0
    q, k = pd[:, :H * dim].view(T, H, dim), pd[:, off_k:off_k + G * dim].view(T, G, dim)
    v, g = pd[:, off_v:off_v + G * vdim].view(T, G, vdim), pd[:, off_g:off_g + H]
    scale = 1.3 * dim ** -0.5
    ref = O.window_attention(O.rotate_pairs(q, rot, base), O.rotate_pairs(k, rot, base), v, scale, window)
    if gate:
        ref = ref * torch.sigmoid(g)[:, :, None]
    inv = torch.tensor([base ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=torch.float64) if rot else None
    kw = dict(heads=H, scale=scale, window=window, off_q=off_q, off_k=off_k, off_v=off_v, off_g=off_g if gate else -1)
    return p, ref.reshape(T, -1), kw, inv


def run_portions(dev, p, kw, inv, dims, cuts, ring, slot=1, path=0, split=False):
    from lit_llama_amd import ops

    G, dim, vdim = dims
    kr = torch.full((3, G, ring, dim), 7.0, dtype=p.dtype, device=dev)  # (a slot somebody used before)
    vr = torch.full((3, G, ring, vdim), 9.0, dtype=p.dtype, device=dev)
    part = torch.zeros(1 << 20, device=dev) if split else None
    out, at = [], 0
    for n in cuts:
        b = ops.PackedBatch([n], [slot], [at], dev)
        out.append(ops.window_attention(p[at:at + n].contiguous().to(dev), b, kr, vr, inv_freq=inv.to(dev) if inv is not None else None,
                                        path=path, partials=part, **kw))
        at += n
    assert at == p.shape[0]
    assert (kr[0] == 7).all() and (kr[2] == 7).all() and (vr[0] == 9).all()
    return torch.cat(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,dim,vdim,window,rot", [(4, 2, 40, 24, 37, 16), (6, 1, 64, 64, 64, 32), (3, 3, 18, 10, 20, 6), (8, 2, 128, 128, 130, 64),
                                                     (10, 1, 72, 200, 1, 8), (2, 1, 32, 16, 500, 0)])
def test_window_attention(dev, dtype, H, G, dim, vdim, window, rot):
    T = 210
    p, ref, kw, inv = attention_case(T, H, G, dim, vdim, window, rot, dtype)
    ring = min(window, T)
    whole = run_portions(dev, p, kw, inv, (G, dim, vdim), [T], ring)
    assert rel(whole, ref) < TOL[dtype]
    for cuts in ([2] * 3 + [T - 6], [100, 1, 64, T - 165], [T - 70] + [1] * 70):
        assert rel(run_portions(dev, p, kw, inv, (G, dim, vdim), cuts, ring), ref) < TOL[dtype], cuts
    assert rel(run_portions(dev, p, kw, inv, (G, dim, vdim), [T], ring, path=1), ref) < TOL[dtype]


def test_window_attention_split_decode_and_larger_ring(dev):
    T, H, G, dim, vdim, window, rot = 700, 4, 1, 64, 32, 600, 64
    p, ref, kw, inv = attention_case(T, H, G, dim, vdim, window, rot, torch.float32, gate=False)
    out = run_portions(dev, p, kw, inv, (G, dim, vdim), [T - 60] + [1] * 60, 640, split=True)
    assert rel(out, ref) < TOL[torch.float32]


def test_far_positions_keep_their_angle(dev):
    """Two rows a million positions in: rotation depends on the distance only."""
    from lit_llama_amd import ops

    H, G, dim, vdim, window, rot = 2, 1, 32, 16, 8, 32
    p, ref, kw, inv = attention_case(6, H, G, dim, vdim, window, rot, torch.float32)
    kr, vr = torch.zeros((1, G, 8, dim), device=dev), torch.zeros((1, G, 8, vdim), device=dev)
    b = ops.PackedBatch([6], [0], [1_000_003], dev)
    kr.zero_()
    kw = dict(kw, window=6)
    y = ops.window_attention(p.to(dev), b, kr, vr, inv_freq=inv.to(dev), **kw)
    # rows 0..4 see cached rows that were never written (zeros here); the last row sees exactly the portion
    ref6 = attention_case(6, H, G, dim, vdim, 6, rot, torch.float32)[1]
    want = O.window_attention(O.rotate_pairs(p[:, :H * dim].double().view(6, H, dim), rot, 5000.0),
                              O.rotate_pairs(p[:, kw["off_k"]:kw["off_k"] + G * dim].double().view(6, G, dim), rot, 5000.0),
                              p[:, kw["off_v"]:kw["off_v"] + G * vdim].double().view(6, G, vdim), kw["scale"], 6)
    want = want * torch.sigmoid(p[:, kw["off_g"]:kw["off_g"] + H].double())[:, :, None]
    assert ref6.shape == want.reshape(6, -1).shape
    assert rel(y[5], want[5].reshape(-1)) < 2e-5


# ---------------------------------------------------------------------------------------- recurrences
def rec_case(kind, T, H, G, dim, vdim, dtype, taps=4, rank=8, tau=8.0, seed=0, strong=False):
    gen = torch.Generator().manual_seed(seed)
    pad = lambda n: (n + 15) // 16 * 16
    sizes = dict(q=G * dim, k=G * dim, v=H * vdim, g=H * vdim, **({"a": H, "b": H} if kind == "delta" else {"a": rank}))
    off, n = {}, 0
    for name, s in sizes.items():
        off[name] = n
        n += pad(s)
    p = torch.randn((T, n), generator=gen)
    if strong:  # decays that nearly erase the state next to ones that keep it, repeated keys with beta near 1
        p[::9, off["a"]:off["a"] + sizes["a"]] *= 30
        p[1::2, off["k"]:off["k"] + G * dim] = p[:1, off["k"]:off["k"] + G * dim]
        if kind == "delta":
            p[:, off["b"]:off["b"] + H] += 4
    p = p.to(dtype)
    w = dict(head_norm=1 + 0.2 * torch.randn(vdim, generator=gen), eps=3e-3)
    if kind == "delta":
        w.update(conv=tuple(0.5 * torch.randn((c, taps), generator=gen) for c in (G * dim, G * dim, H * vdim)),
                 a_log=torch.randn(H, generator=gen) - 1, dt_bias=torch.randn(H, generator=gen))
    else:
        w.update(a2=torch.randn((H * dim, rank), generator=gen) * rank ** -0.5, a2_bias=torch.randn(H * dim, generator=gen) + 1, tau=tau)
    d = p.double()
    part = lambda name: d[:, off[name]:off[name] + sizes[name]]
    if kind == "delta":
        q, k, v = (O.silu(O.short_conv(part(x), w["conv"][i].double())) for i, x in enumerate("qkv"))
        q = O.unit_vector(q.view(T, G, dim)) * dim ** -0.5
        k = O.unit_vector(k.view(T, G, dim))
        g = torch.exp(-torch.exp(w["a_log"].double()) * O.softplus(part("a") + w["dt_bias"].double()))
        o = O.delta_rule(q, k, v.view(T, H, vdim), g, torch.sigmoid(part("b")))
    else:
        z = part("a") @ w["a2"].double().T + w["a2_bias"].double()
        alpha = torch.exp(-O.softplus(-z) / tau).view(T, H, dim)
        o = O.gated_linear_attention(part("q").view(T, H, dim) * dim ** -0.5, part("k").view(T, H, dim), part("v").view(T, H, vdim), alpha)
    ref = O.rms_norm(o, w["head_norm"].double(), w["eps"]).reshape(T, -1) * O.silu(part("g"))
    return p, ref, off, w


def run_rec(dev, kind, p, off, w, H, G, dim, vdim, cuts, path=0, taps=4, slots=(1,)):
    from lit_llama_amd import ops

    state = torch.full((3, H, dim, vdim), 5.0, device=dev)
    ring = torch.full((3, taps, 2 * G * dim + H * vdim), 3.0, dtype=p.dtype, device=dev)
    state[slots[0]] = 0
    kw = {k: (tuple(t.to(dev) for t in v) if isinstance(v, tuple) else v.to(dev) if torch.is_tensor(v) else v) for k, v in w.items()}
    out, at = [], 0
    for n in cuts:
        b = ops.PackedBatch([n], [slots[0]], [at], dev)
        out.append(ops.recurrent(kind, p[at:at + n].contiguous().to(dev), b, state, off=off, kv_heads=G, conv_ring=ring, path=path, **kw))
        at += n
    assert at == p.shape[0]
    assert (state[0] == 5).all() and (state[2] == 5).all() and (ring[0] == 3).all()
    return torch.cat(out)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("kind,H,G,dim,vdim,taps", [("delta", 4, 2, 24, 40, 4), ("delta", 3, 3, 64, 32, 2), ("delta", 2, 1, 130, 70, 5), ("delta", 2, 2, 16, 144, 1),
                                                    ("delta", 1, 1, 33, 17, 9),
                                                    ("gla", 3, 3, 24, 40, 0), ("gla", 2, 2, 130, 70, 0), ("gla", 1, 1, 64, 128, 0)])
def test_recurrences(dev, dtype, kind, H, G, dim, vdim, taps):
    T = 203
    p, ref, off, w = rec_case(kind, T, H, G, dim, vdim, dtype, taps=taps or 4)
    args = (dev, kind, p, off, w, H, G, dim, vdim)
    tol = 5e-5  # (bf16: only the inputs and the stored outputs are rounded)
    for path, cuts in ((1, [T]), (2, [T]), (0, [2, 2, 3, 64, 65, T - 136]), (0, [T - 40] + [1] * 40), (2, [1, 1, 127, T - 129])):
        assert rel(run_rec(*args, cuts, path=path, taps=taps or 4), ref) < tol, (path, cuts)


@pytest.mark.parametrize("kind,tau", [("delta", 1.0), ("gla", 1.0), ("gla", 16.0)])
def test_recurrences_with_strong_decays_and_repeated_keys(dev, kind, tau):
    T, H, G, dim, vdim = 300, 2, 2, 48, 32
    p, ref, off, w = rec_case(kind, T, H, G, dim, vdim, torch.float32, tau=tau, strong=True, seed=3)
    for path in (1, 2):
        out = run_rec(dev, kind, p, off, w, H, G, dim, vdim, [T], path=path)
        assert torch.isfinite(out).all()
        assert rel(out, ref) < 2e-4, path


# ---------------------------------------------------------------------------------------- the model
def small_config(**kw):
    att = lambda **m: {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 24, "vdim": 40, "scale": 0.3, "mask": {"size": 19},
                                                      "rot": {"base": 900.0, "dims": 8}, **m}, "mlp": {"kind": "dense", "ff": 72}}
    gla = {"type": "gla", "mixer": {"heads": 3, "dim": 20, "vdim": 28, "tau": 4.0}, "mlp": {"kind": "dense", "ff": 40}}
    delta = {"type": "delta", "mixer": {"heads": 6, "kv_heads": 2, "dim": 12, "vdim": 20, "conv": 3}, "mlp": None}
    return {"architecture": "Sekulorn", "vocab": 211, "width": 104, "norm": {"eps": 3e-5}, "residual_mult": 0.45,
            "layers": [delta, att(), {**att(kv_heads=4, dim=32, vdim=8), "mlp": None}, gla], "loop": {"start": 1, "stop": 3, "times": 3}, **kw}


def build(config, dtype, dev, seed=1):
    from lit_llama_amd import synth
    from lit_llama_amd.registry import build_model

    sd = synth.make_hybrid_state_dict(config, seed=seed, rank=5)
    m = build_model(config, dtype, dev)
    m.load_state_dict(sd)
    return m, sd


def tokens_of(n, vocab=211, seed=0):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


CONFIGS = {
    "mixed": small_config(),
    "no loop, unit multiplier": small_config(loop=None, residual_mult=1.0),
    "no rotation, no window": small_config(layers=[{"type": "attention", "mixer": {"heads": 3, "kv_heads": 1, "dim": 16, "vdim": 16, "scale": 0.25},
                                                    "mlp": None}], loop=None, width=64),
    "all looped": small_config(loop={"start": 0, "stop": 4, "times": 2}, width=97, vocab=130),
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
    assert eng.run_layers == O.layer_order(config)
    for r in range(1, len(trail) + 1):
        s = eng.acquire()
        assert rel(eng.residual_after([Entry(s, 0, toks, [])], r), trail[r - 1]) < 5e-5, r
        eng.release(s)
    s = eng.acquire()
    assert rel(eng.step([Entry(s, 0, toks, range(61))]), logits) < 5e-5
    eng.release(s)


@pytest.mark.parametrize("name,dtype,tol", [("mixed", torch.float32, 1e-4), ("mixed", torch.bfloat16, 0.12), ("all looped", torch.bfloat16, 0.12)])
def test_portions_batches_slots_and_decoding(dev, name, dtype, tol):
    """Unequal requests in one batch, cut differently, decoded together, their slots used again: the logits of each alone."""
    from lit_llama_amd.hybrid_engine import Entry

    config = CONFIGS[name]
    m, sd = build(config, dtype, dev)
    eng = m.engine()
    eng.ensure(4, 200)
    seqs = [tokens_of(n, config["vocab"], seed=n) for n in (150, 9, 64, 33)]
    refs = [O.forward(config, sd, s)[0] for s in seqs]
    for first in ((100, 2, 31, 32), (64, 8, 1, 3)):  # (the second time in the slots of the first)
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
            assert rel(torch.cat(got[i]), refs[i]) < tol, (i, first)
        for s in slots:
            eng.release(s)
    assert eng.slots.live == 0


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


def test_bad_input_is_an_error_on_the_host(dev):
    from lit_llama_amd._native import NativeError
    from lit_llama_amd.hybrid_engine import Entry

    m, _ = build(CONFIGS["mixed"], torch.float32, dev)
    eng = m.engine()
    eng.ensure(1, 16)
    s = eng.acquire()
    for entry in (Entry(s, 0, [0] * 17, []), Entry(s, 0, [211], []), Entry(s, 0, [-1], []), Entry(s, 0, [1, 2], [1, 0])):
        with pytest.raises(NativeError):
            eng.step([entry])


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
    refs = [greedy_reference(config, sd, p, 12, 1e-3) for p in prompts]
    assert sum(map(len, refs)) > 30
    outs = generate_batch(m, prompts, 12, top_k=1, max_batch=3, portion=16)  # (requests wait, enter late, are cut)
    for o, r in zip(outs, refs):
        assert len(o) == 12 and o[:len(r)] == r
    assert m.engine().slots.live == 0
    for p, r in zip(prompts[:2], refs):
        y = lit_llama_amd.generate(m, torch.tensor(p, device=dev), 12, top_k=1).tolist()
        assert y[:len(p)] == p and len(y) == len(p) + 12 and y[len(p):len(p) + len(r)] == r
    again = lit_llama_amd.generate(m, torch.tensor(prompts[0], device=dev), 12, top_k=1).tolist()
    assert again[len(prompts[0]):] == outs[0]
    # a batch behind generate() that needs longer rings than its sequence
    fresh, _ = build(config, torch.float32, dev)
    lit_llama_amd.generate(fresh, torch.tensor([1, 2, 3], device=dev), 2, top_k=1)
    assert generate_batch(fresh, prompts[:2], 12, top_k=1) == outs[:2]
    # eos ends a request early and the others go on
    eos = outs[0][4]
    cut = generate_batch(m, prompts, 12, top_k=1, eos_id=eos)
    assert cut[0] == outs[0][:outs[0].index(eos)]


def test_sampled_generation(dev):
    import lit_llama_amd
    from lit_llama_amd.batching import generate_batch

    config = CONFIGS["mixed"]
    m, _ = build(config, torch.bfloat16, dev)
    p = tokens_of(20)
    torch.manual_seed(5)
    a = lit_llama_amd.generate(m, torch.tensor(p, device=dev), 40, temperature=0.7, top_k=20)
    torch.manual_seed(5)
    b = lit_llama_amd.generate(m, torch.tensor(p, device=dev), 40, temperature=0.7, top_k=20)
    assert torch.equal(a, b) and int(a.max()) < 211
    x = generate_batch(m, [p, p[:7]], 15, temperature=0.9, top_k=50, seed=3)
    y = generate_batch(m, [p, p[:7]], 15, temperature=0.9, top_k=50, seed=3)
    assert x == y and [len(o) for o in x] == [15, 15]


def test_a_dropped_model_frees_its_engine_without_the_collector(dev):
    import gc
    import weakref

    from lit_llama_amd.hybrid_engine import Entry

    m, _ = build(CONFIGS["mixed"], torch.float32, dev)
    eng = m.engine()
    eng.ensure(1, 16)
    s = eng.acquire()
    for i in range(4):  # (a captured step included)
        eng.step([Entry(s, i, [i], [0])])
    alive = weakref.ref(eng)
    gc.collect()
    gc.disable()
    try:
        del eng, m
        assert alive() is None
    finally:
        gc.enable()


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


def test_module_forward_and_cache_reset(dev):
    config = CONFIGS["mixed"]
    m, sd = build(config, torch.float32, dev)
    toks = torch.tensor([tokens_of(30, seed=1), tokens_of(30, seed=2)], device=dev)
    out = m(toks)
    for i in range(2):
        assert rel(out[i], O.forward(config, sd, toks[i].tolist())[0]) < 1e-4
    for _ in range(2):
        a = m(toks[:1, :29], 64, torch.arange(29, device=dev))
        b = m(toks[:1, 29:], 64, torch.tensor([29], device=dev))
        assert rel(torch.cat([a[0], b[0]]), out[0]) < 1e-4
        m.reset_cache()


def test_trace_replay_and_command_line(dev, tmp_path, capsys, monkeypatch):
    import io

    import numpy as np
    from safetensors.torch import save_file

    from lit_llama_amd import __main__ as cli
    from lit_llama_amd import synth, trace

    config = CONFIGS["all looped"]
    sd = synth.make_hybrid_state_dict(config, seed=9, rank=3)
    (tmp_path / "config.json").write_text(json.dumps(config))
    save_file(sd, str(tmp_path / "model.safetensors"))
    a, b = tokens_of(25, 130, 1), tokens_of(11, 130, 2)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:20], "want": [0, 19]}, {"id": "b", "tokens": b[:8], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[20:21], "want": [0]}, {"id": "b", "tokens": b[8:9], "want": [0]}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[21:22], "want": []}], "end": ["a"]}]
    monkeypatch.setattr("sys.stdin", io.StringIO("\n".join(map(json.dumps, steps)) + "\n"))
    assert trace.main(["--model", str(tmp_path), "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "64"]) == 0
    assert capsys.readouterr().out.split("\n")[:3] == ["done 0", "done 1", "done 2"]
    ra, rb = O.forward(config, sd, a)[0], O.forward(config, sd, b)[0]
    got = [torch.from_numpy(np.fromfile(tmp_path / f"{i}.f32", "<f4").reshape(-1, 130)) for i in (0, 1)]
    assert rel(got[0], ra[[0, 19]]) < 1e-4 and rel(got[1], torch.stack([ra[20], rb[8]])) < 1e-4
    assert not (tmp_path / "2.f32").exists()
    assert cli.main(["--model", str(tmp_path), "--dtype", "float32", "--prompt-ids", ",".join(map(str, a)), "--prompt-ids", "1,2", "--top-k", "1",
                     "--max-new-tokens", "5"]) == 0
    lines = capsys.readouterr().out.strip().split("\n")
    assert len(lines) == 2 and lines[0].startswith(",".join(map(str, a))) and len(lines[0].split(",")) == 30
