"""Host side of the Kovalorn design: configuration, registry, weight names, lent caches; and the plain restatement in oracle/kovalorn.py
checked against closed forms of its mechanisms."""
import copy
import json
import math

import pytest
import torch

from lit_llama_amd import registry, synth
from lit_llama_amd.hybrid import HybridConfig, HybridLM, tensor_shapes
from oracle import kovalorn as O


def attention(**kw):
    return {"heads": 6, "kv_heads": 2, "dim": 20, "vdim": 12, "scale": 0.3, "mask": {"size": 9, "keep_first": 2}, **kw}


CONFIG = {
    "architecture": "Kovalorn", "vocab": 90, "width": 36, "norm": {"eps": 3e-4}, "logit_scale": 0.7,
    "layers": [
        {"type": "attention", "mixer": attention(), "mlp": {"kind": "moe", "expert": {"ff": 10}, "router": {"experts": 5, "scale": 1.5, "top": 2},
                                                           "shared": {"ff": 14}}},
        {"type": "attention", "mixer": attention(kv_heads=1, mask={"size": 5, "keep_first": 0}), "mlp": {"kind": "dense", "ff": 20}},
        {"type": "attention", "mixer": attention(kv_from=0, mask={"size": 30, "keep_first": 7}), "mlp": None},
        {"type": "attention", "mixer": attention(kv_heads=1, heads=3, kv_from=1, mask=None, scale=0.2),
         "mlp": {"kind": "moe", "expert": {"ff": 8}, "router": {"experts": 3, "scale": 1.0, "top": 1}, "shared": None}},
    ],
}


def test_configuration_reads_every_constant():
    c = HybridConfig.from_dict(CONFIG)
    a, b, d, e = (l.mixer for l in c.layers)
    assert (c.vocab_size, c.width, c.eps, c.logit_scale, c.residual_mult) == (90, 36, 3e-4, 0.7, 1.0)
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.window, a.keep, a.kv_from) == (6, 2, 20, 12, 0.3, 9, 2, None)
    assert a.unit_qk and a.sink and a.gate_values and a.rot_dims == 0
    assert (b.window, b.keep, d.window, d.keep, d.kv_from, e.keep, e.kv_from) == (5, 0, 30, 7, 0, 0, 1) and e.window > 1 << 20
    m = [l.mlp for l in c.layers]
    assert (m[0].kind, m[0].ff, m[0].experts, m[0].top, m[0].scale, m[0].ff_shared) == ("experts", 10, 5, 2, 1.5, 14)
    assert (m[1].kind, m[1].ff, m[2], m[3].ff_shared) == ("geglu", 20, None, 0)
    assert c.design.norm_add == 1 and c.design.tied and c.lenders() == [None, None, 0, 1]


def test_a_lent_cache_is_the_latest_run_of_its_layer():
    c = HybridConfig.from_dict(CONFIG)
    c.loop = (0, 3, 2)
    assert c.runs() == [0, 1, 2, 0, 1, 2, 3] and c.lenders() == [None, None, 0, None, None, 3, 4]


@pytest.mark.parametrize("path,value", [
    (("layers", 0, "type"), "delta"), (("layers", 0, "mixer", "rot"), {"base": 1.0, "dims": 4}), (("layers", 0, "mixer", "mask", "chunk"), 8),
    (("layers", 0, "mlp", "kind"), "sparse"), (("layers", 0, "mlp", "router", "groups"), 2), (("layers", 0, "mlp", "router", "top"), 6),
    (("layers", 1, "mixer", "kv_heads"), 4), (("layers", 1, "mixer", "kv_from"), 1), (("layers", 3, "mixer", "kv_from"), 2),
    (("layers", 2, "mixer", "kv_from"), 1), (("loop",), {"start": 0, "stop": 2, "times": 2}), (("architecture",), "Nothing")])
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

    sd = synth.make_hybrid_state_dict(CONFIG)
    assert {"l0.mix.sink", "l0.mlp.e4.down", "l0.mlp.shared.gate", "l0.mlp.router", "l1.mlp.gate", "l2.mix.g"} <= set(sd)
    assert not {"head", "l2.mix.k", "l2.norm2", "l3.mix.v", "l3.mlp.shared.up", "l0.mlp.e5.up"} & set(sd)
    assert sd["l0.mix.g"].shape == (72, 36) and sd["l3.mix.o"].shape == (36, 36)
    (tmp_path / "config.json").write_text(json.dumps(CONFIG))
    save_file(sd, str(tmp_path / "model.safetensors"))
    m = registry.load_model(tmp_path, torch.float32, "cpu")
    assert isinstance(m, HybridLM) and all(torch.equal(m.tensors[n], t.float()) for n, t in sd.items())
    for bad in ("missing", "extra", "shape"):
        d = dict(sd)
        if bad == "missing":
            del d["l0.mlp.e3.up"]
        elif bad == "extra":
            d["l2.mix.k"] = torch.zeros((40, 36))
        else:
            d["l0.mix.sink"] = torch.zeros(5)
        with pytest.raises(ValueError):
            registry.build_model(CONFIG, device="cpu").load_state_dict(d)


# ---------------------------------------------------------------------------------------- the restatement itself
def test_oracle_sees_the_window_and_the_first_tokens():
    T, window, keep = 14, 4, 2
    q = torch.zeros((T, 1, 1)).double()
    v = torch.arange(T).double().view(T, 1, 1)
    out = O.sink_attention(q, q, v, 1.0, window, keep, None)[:, 0, 0]  # equal scores: the mean of what is seen
    want = [sum(s) / len(s) for s in ([j for j in range(i + 1) if j > i - 4 or j < 2] for i in range(T))]
    assert torch.allclose(out, torch.tensor(want).double())
    # the sink is one more term that adds nothing: log 3 counts as three keys of score 0
    sunk = O.sink_attention(q, q, v, 1.0, window, keep, torch.tensor([math.log(3)]).double())[:, 0, 0]
    n = torch.tensor([len(O.visible(i, window, keep)) for i in range(T)]).double()
    assert torch.allclose(sunk, out * n / (n + 3))


def test_oracle_unit_rms_ignores_size_and_norm_weight_is_around_one():
    x = torch.randn((3, 8), dtype=torch.float64)
    assert torch.allclose(O.unit_rms(1e3 * x, 1e-9), O.unit_rms(x, 1e-9))
    assert torch.allclose(O.unit_rms(x, 0.5), x / (x.pow(2).mean(-1, keepdim=True) + 0.5) ** 0.5)
    assert torch.equal(O.rms_norm(x, torch.zeros(8).double(), 1e-5), O.unit_rms(x, 1e-5))


def test_oracle_activations():
    z = torch.linspace(-6, 6, 41, dtype=torch.float64)
    assert torch.allclose(O.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    assert torch.allclose(O.silu(z), torch.nn.functional.silu(z))


def test_oracle_router_weights():
    h = torch.tensor([[1.0, 0.0], [0.0, 1.0]], dtype=torch.float64)
    r = torch.tensor([[0.5, -1.0], [3.0, 0.2], [-2.0, 0.1]], dtype=torch.float64)
    ids, w = O.route(h, r, 2, 2.5)
    assert ids.tolist() == [[1, 0], [1, 2]] and torch.allclose(w.sum(1), torch.full((2,), 2.5).double())
    s = torch.sigmoid(torch.tensor([3.0, 0.5], dtype=torch.float64))
    assert torch.allclose(w[0], 2.5 * s / s.sum())


def test_oracle_is_causal_and_prefix_stable():
    sd = synth.make_hybrid_state_dict(CONFIG)
    toks = torch.randint(0, 90, (20,), generator=torch.Generator().manual_seed(0)).tolist()
    a, trail = O.forward(CONFIG, sd, toks)
    b, _ = O.forward(CONFIG, sd, toks[:11])
    assert torch.allclose(a[:11], b) and trail.shape == (4, 20, 36)
    assert set(tensor_shapes(HybridConfig.from_dict(CONFIG), {})) == set(sd)
    # the borrowing layer's logits depend on what it borrows
    other = {**sd, "l0.mix.k": -sd["l0.mix.k"]}
    assert not torch.allclose(O.forward(CONFIG, other, toks)[1][2], trail[2])
