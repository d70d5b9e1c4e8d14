"""Host side of the Kudazen design: configuration, registry, weight names, shared weights; and the plain restatement in oracle/kudazen.py
checked against closed forms of its mechanisms."""
import copy
import json
import math

import pytest
import torch

from lit_llama_amd import registry, synth
from lit_llama_amd.hybrid import HybridConfig, HybridLM, projections, tensor_shapes
from oracle import kudazen as O

MLP = {"kind": "dense", "ff": 20, "limit": 2.5}
CONFIG = {
    "architecture": "Kudazen", "vocab": 90, "width": 36, "norm": {"eps": 3e-4, "groups": 3},
    "layers": [
        {"type": "latent_attention", "mixer": {"heads": 3, "dim": 10, "rot_dim": 6, "vdim": 14, "q_rank": 22, "kv_rank": 18,
                                               "rot": {"base": 500.0, "dims": 6}, "scale": 0.3}, "mlp": MLP},
        {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 8, "scale": 0.4, "mask": {"size": 7}}, "mlp": None},
        {"type": "wkv", "mixer": {"heads": 3, "dim": 8}, "mlp": {**MLP, "limit": 1.0}},
    ],
}
CONFIG["layers"] += [{**copy.deepcopy(CONFIG["layers"][i]), "weights_of": i} for i in (2, 0)]


def test_configuration_reads_every_constant():
    c = HybridConfig.from_dict(CONFIG)
    l, a, w = (x.mixer for x in c.layers[:3])
    assert (c.vocab_size, c.width, c.eps, c.norm_groups, c.residual_mult, c.logit_scale) == (90, 36, 3e-4, 3, 1.0, 1.0)
    assert (l.heads, l.dim, l.rot_dim, l.vdim, l.q_rank, l.kv_rank, l.scale, l.rot_dims, l.rot_base) == (3, 10, 6, 14, 22, 18, 0.3, 6, 500.0)
    assert l.sink and not l.gated and not l.chunked
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.rot_dims) == (4, 2, 12, 8, 0.4, 7, 0)
    assert a.chunked and a.temp and a.bias and a.unit_v and not (a.unit_qk or a.sink or a.gated)
    assert (w.heads, w.dim, w.vdim) == (3, 8, 8)
    assert [x.mlp and (x.mlp.kind, x.mlp.ff, x.mlp.limit) for x in c.layers] == [("clampglu", 20, 2.5), None, ("clampglu", 20, 1.0), ("clampglu", 20, 1.0),
                                                                                ("clampglu", 20, 2.5)]
    assert [x.weights_of for x in c.layers] == [None, None, None, 2, 0] and c.runs() == [0, 1, 2, 3, 4]
    assert c.design.tied and c.design.parallel and c.design.norm_add == 0
    assert projections(l) == ("dq", "dkv") and projections(a) == ("q", "k", "v") and projections(w) == ("r", "k", "v", "g", "w1")
    plain = copy.deepcopy(CONFIG)
    plain["layers"][1]["mixer"]["mask"] = None
    assert not HybridConfig.from_dict(plain).layers[1].mixer.chunked


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "gla"), (("layers", 0, "mixer", "rot", "dims"), 4), (("layers", 0, "mixer", "mask"), {"size": 4}),
    (("layers", 1, "mixer", "rot"), {"base": 1.0, "dims": 4}), (("layers", 1, "mixer", "mask", "keep_first"), 8), (("layers", 1, "mixer", "kv_heads"), 3),
    (("layers", 2, "mixer", "vdim"), 8), (("layers", 0, "mlp", "kind"), "moe"), (("norm", "groups"), 5), (("layers", 3, "weights_of"), 4),
    (("layers", 3, "weights_of"), 9), (("layers", 3, "mixer", "heads"), 2), (("logit_scale",), 0.5), (("loop",), {"start": 0, "stop": 2, "times": 2})])
def test_what_the_framework_does_not_know_is_refused(path, value):
    c = copy.deepcopy(CONFIG)
    at = c
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ValueError):
        HybridConfig.from_dict(c)


def test_folder_loads_and_is_checked(tmp_path):
    from safetensors.torch import save_file

    sd = synth.make_hybrid_state_dict(CONFIG, rank=5)
    assert {"l0.mix.dq.norm", "l0.mix.sink", "l1.mix.temp", "l2.mix.mu.w", "l2.mix.w2", "l2.mix.u", "l0.mlp.gate"} <= set(sd)
    assert not {"head", "l0.norm2", "l1.mlp.gate", "l1.mix.g", "l3.norm1", "l4.mix.uq"} & set(sd)
    assert sd["l0.mix.uq"].shape == (48, 22) and sd["l0.mix.dkv"].shape == (24, 36) and sd["l2.mix.w2"].shape == (24, 5) and sd["l2.mix.norm"].shape == (24,)
    (tmp_path / "config.json").write_text(json.dumps(CONFIG))
    save_file(sd, str(tmp_path / "model.safetensors"))
    m = registry.load_model(tmp_path, torch.float32, "cpu")
    assert isinstance(m, HybridLM) and all(torch.equal(m.tensors[n], t.float()) for n, t in sd.items())
    for bad in ("missing", "extra", "shape"):
        d = dict(sd)
        if bad == "missing":
            del d["l0.mix.dkv.norm"]
        elif bad == "extra":
            d["l3.norm1"] = torch.zeros(36)
        else:
            d["l2.mix.u"] = torch.zeros((8, 3))
        with pytest.raises(ValueError):
            registry.build_model(CONFIG, device="cpu").load_state_dict(d)


# ---------------------------------------------------------------------------------------- the restatement itself
def test_oracle_sees_its_chunk():
    T, size = 14, 5
    q = torch.zeros((T, 2, 1)).double()
    v = torch.arange(T).double().view(T, 1, 1)
    out = O.chunk_attention(q, q[:, :1], v, torch.ones(2).double(), [0.0, 0.0], size)[:, 1, 0]  # equal scores: the mean of what is seen
    assert torch.allclose(out, torch.tensor([sum(range(i - i % size, i + 1)) / (i % size + 1) for i in range(T)]).double())
    # a slope of log 2 halves the weight per position of distance
    out = O.chunk_attention(q, q[:, :1], v, torch.ones(2).double(), [math.log(2)] * 2, None)[:, 0, 0]
    want = [sum(j * 2.0 ** (j - i) for j in range(i + 1)) / sum(2.0 ** (j - i) for j in range(i + 1)) for i in range(T)]
    assert torch.allclose(out, torch.tensor(want).double())
    assert O.slopes(4) == [0.25, 0.0625, 0.015625, 0.00390625]


def test_oracle_sink_counts_once():
    q = torch.zeros((6, 1, 2)).double()
    v = torch.ones((6, 1, 1)).double()
    out = O.sink_attention(q, q, v, 0.5, torch.tensor([math.log(3)]).double())[:, 0, 0]
    n = torch.arange(1, 7).double()
    assert torch.allclose(out, n / (n + 3))


def test_oracle_rotation_depends_on_the_distance():
    x, y = torch.randn((2, 4), dtype=torch.float64, generator=torch.Generator().manual_seed(1))
    r = lambda z: O.rotate_pairs(z.expand(9, 4), 70.0)
    a, b = r(x), r(y)
    assert torch.allclose(a[5] @ b[2], a[8] @ b[5]) and torch.allclose(a.norm(dim=-1), x.norm().expand(9)) and torch.equal(a[0], x)
    assert torch.allclose(O.rotate_pairs(torch.tensor([[0, 0], [1.0, 0]]).double(), 9.0)[1], torch.tensor([math.cos(1), math.sin(1)]).double())


def test_oracle_group_norm_and_shift():
    x = torch.randn((3, 8), dtype=torch.float64, generator=torch.Generator().manual_seed(2))
    big = x * torch.tensor([1e3] * 4 + [1e-3] * 4)
    assert torch.allclose(O.group_norm(big, torch.ones(8).double(), 2, 0.0), O.group_norm(x, torch.ones(8).double(), 2, 0.0))
    assert torch.allclose(O.group_norm(x, torch.ones(8).double(), 1, 0.5), x / (x.pow(2).mean(-1, keepdim=True) + 0.5) ** 0.5)
    s = O.token_mix(x, torch.full((8,), 0.25).double())
    assert torch.allclose(s[0], 0.75 * x[0]) and torch.allclose(s[2], 0.75 * x[2] + 0.25 * x[1])


def test_oracle_wkv_is_a_weighted_sum_of_the_past():
    gen = torch.Generator().manual_seed(3)
    r, k, v = torch.randn((3, 7, 2, 4), dtype=torch.float64, generator=gen)
    w, u = torch.rand((7, 2, 4), dtype=torch.float64, generator=gen), torch.randn((2, 4), dtype=torch.float64, generator=gen)
    out = O.wkv(r, k, v, w, u)
    want = torch.zeros_like(out)
    for t in range(7):
        for j in range(t):
            want[t] += (r[t] * k[j] * w[j + 1:t].prod(0)).sum(-1, keepdim=True) * v[j]
        want[t] += (r[t] * u * k[t]).sum(-1, keepdim=True) * v[t]
    assert torch.allclose(out, want)


def test_oracle_clamped_gate():
    g, u = torch.tensor([-30.0, 0.0, 1.0, 9.0]).double(), torch.tensor([-5.0, -5.0, 0.5, 5.0]).double()
    out = O.clamped_gate(g, u, 2.0)
    f = lambda x: x / (1 + math.exp(-1.702 * x))
    assert torch.allclose(out, torch.tensor([f(-30.0) * -1, 0.0, f(1.0) * 1.5, f(2.0) * 3]).double())


def test_oracle_is_causal_and_layers_share_weights():
    sd = synth.make_hybrid_state_dict(CONFIG, rank=4)
    assert set(tensor_shapes(HybridConfig.from_dict(CONFIG), {2: 4})) == set(sd)
    toks = torch.randint(0, 90, (20,), generator=torch.Generator().manual_seed(0)).tolist()
    a, trail = O.forward(CONFIG, sd, toks)
    b, _ = O.forward(CONFIG, sd, toks[:11])
    assert torch.allclose(a[:11], b) and trail.shape == (5, 20, 36)
    own = copy.deepcopy(CONFIG)
    own["layers"][3]["weights_of"] = None
    same = {**sd, **{n.replace("l2.", "l3."): t for n, t in sd.items() if n.startswith("l2.")}}
    assert torch.allclose(O.forward(own, same, toks)[0], a)
