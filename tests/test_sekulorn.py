"""Host side of the Sekulorn design: configuration, registry, weight loading, slots, cutting of steps, the scheduler; and the plain
restatement in oracle/sekulorn.py checked against closed forms of its mechanisms."""
import copy
import json

import pytest
import torch

from lit_llama_amd import checkpoint, registry, synth
from lit_llama_amd.batching import BatchScheduler, Request
from lit_llama_amd.hybrid import HybridConfig, HybridLM, tensor_shapes
from lit_llama_amd.hybrid_engine import Entry, HybridEngine
from lit_llama_amd.state import SlotManager
from oracle import sekulorn as O

CONFIG = {
    "architecture": "Sekulorn", "vocab": 90, "width": 36, "norm": {"eps": 2e-5}, "residual_mult": 0.6,
    "loop": {"start": 0, "stop": 2, "times": 3},
    "layers": [
        {"type": "delta", "mixer": {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 10, "conv": 3}, "mlp": {"kind": "dense", "ff": 20}},
        {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 8, "scale": 0.4, "mask": {"size": 5},
                                        "rot": {"base": 700.0, "dims": 6}}, "mlp": None},
        {"type": "gla", "mixer": {"heads": 2, "dim": 8, "vdim": 14, "tau": 3.0}, "mlp": {"kind": "dense", "ff": 11}},
    ],
}


def test_configuration_reads_every_constant():
    c = HybridConfig.from_dict(CONFIG)
    d, a, g = (l.mixer for l in c.layers)
    assert (c.vocab_size, c.width, c.eps, c.residual_mult) == (90, 36, 2e-5, 0.6)
    assert (d.heads, d.kv_heads, d.dim, d.vdim, d.taps) == (4, 2, 6, 10, 3)
    assert (a.scale, a.window, a.rot_dims, a.rot_base, a.vdim) == (0.4, 5, 6, 700.0, 8)
    assert (g.heads, g.kv_heads, g.tau) == (2, 2, 3.0) and [l.ff for l in c.layers] == [20, 0, 11]
    assert c.runs() == [0, 1, 0, 1, 0, 1, 2] == O.layer_order(CONFIG)
    assert HybridConfig.from_dict({**CONFIG, "loop": None}).runs() == [0, 1, 2]


@pytest.mark.parametrize("path,value", [(("layers", 0, "type"), "mamba"), (("layers", 1, "mixer", "sinks"), 4), (("layers", 0, "mlp", "kind"), "moe"),
                                        (("layers", 1, "mixer", "mask", "chunk"), 8), (("loop", "stop"), 4), (("layers", 1, "mixer", "kv_heads"), 3)])
def test_what_the_framework_does_not_know_is_refused(path, value):
    c = copy.deepcopy(CONFIG)
    at = c
    for k in path[:-1]:
        at = at[k]
    at[path[-1]] = value
    with pytest.raises(ValueError):
        HybridConfig.from_dict(c)


def test_registry_builds_by_architecture():
    m = registry.build_model(CONFIG, device="cpu")
    assert isinstance(m, HybridLM) and m.config.width == 36
    with pytest.raises(ValueError, match="unknown architecture"):
        registry.build_model({**CONFIG, "architecture": "Nothing"})
    llama = registry.build_model({"architecture": "LLaMA", "n_layer": 1, "n_head": 2, "n_embd": 64, "block_size": 32}, torch.float32, "cpu")
    assert type(llama).__name__ == "LLaMA" and llama.config.n_embd == 64


def test_safetensors_folder_loads_lazily_and_is_checked(tmp_path):
    from safetensors.torch import save_file

    sd = synth.make_hybrid_state_dict(CONFIG, rank=4)
    (tmp_path / "config.json").write_text(json.dumps(CONFIG))
    save_file(sd, str(tmp_path / "model.safetensors"))
    with checkpoint.lazy_load(tmp_path / "model.safetensors") as lazy:
        reader = lazy["embed"]._storage.reader
        assert set(lazy) == set(sd) and reader.bytes_mapped == 0
        assert torch.equal(lazy["l0.mix.q"].materialize(), sd["l0.mix.q"])
        assert torch.equal(lazy["l0.mix.k"][2:5].materialize(), sd["l0.mix.k"][2:5])
        assert reader.bytes_mapped == 2 * (sd["l0.mix.q"].numel() + 3 * 36)
    m = registry.load_model(tmp_path, torch.float32, "cpu")
    assert all(torch.equal(m.tensors[n], t.float()) for n, t in sd.items())
    for bad in ("missing", "extra", "shape"):
        d = dict(sd)
        if bad == "missing":
            del d["l2.mix.a2.b"]
        elif bad == "extra":
            d["l1.mix.sink"] = torch.zeros(4)
        else:
            d["head"] = torch.zeros((91, 36))
        with pytest.raises(ValueError):
            registry.build_model(CONFIG, device="cpu").load_state_dict(d)


def test_a_damaged_safetensors_file_is_refused(tmp_path):
    p = tmp_path / "x.safetensors"
    head = json.dumps({"t": {"dtype": "F32", "shape": [4], "data_offsets": [0, 16]}}).encode()
    p.write_bytes(len(head).to_bytes(8, "little") + head + b"\0" * 12)
    with pytest.raises(ValueError):
        checkpoint.lazy_load(p)


def test_slots_are_dealt_reused_and_grown():
    sizes = []
    s = SlotManager(sizes.append)
    s.reserve(2)
    assert [s.acquire(), s.acquire(), s.acquire()] == [0, 1, 2] and sizes == [2, 4] and s.live == 3
    s.release(1)
    assert s.acquire() == 1
    s.release(0)
    for bad in (0, 9):
        with pytest.raises(ValueError):
            s.release(bad)


class _Cutter:
    """The host part of HybridEngine that cuts steps, without a device."""

    max_rows, max_logits_rows, max_len = 10, 4, 100
    cfg = HybridConfig.from_dict(CONFIG)
    _cut = HybridEngine._cut


def test_steps_are_cut_to_the_scratch_without_losing_rows_or_wishes():
    import random

    rnd = random.Random(5)
    for _ in range(200):
        entries = []
        for s in range(rnd.randint(1, 5)):
            n = rnd.randint(1, 25)
            entries.append(Entry(s, rnd.randint(0, 50), [rnd.randrange(90) for _ in range(n)], sorted(rnd.sample(range(n), rnd.randint(0, min(n, 9))))))
        subs = _Cutter()._cut(entries)
        seen = {e.slot: (e.pos, [], []) for e in entries}
        order = []
        for sub in subs:
            assert sum(len(e.tokens) for e in sub) <= 10 and sum(len(e.want) for e in sub) <= 4
            assert len({e.slot for e in sub}) == len(sub) > 0
            for e in sub:
                pos, toks, want = seen[e.slot]
                assert e.pos == pos + len(toks) and len(e.tokens) > 0
                want.extend(len(toks) + k for k in e.want)
                order.extend((e.slot, len(toks) + k) for k in e.want)
                toks.extend(e.tokens)
        for e in entries:
            assert seen[e.slot][1] == list(e.tokens) and seen[e.slot][2] == list(e.want)
        assert order == [(e.slot, k) for e in entries for k in e.want]


class _FakeEngine:
    """An engine whose next token is (last token + 1) mod 90: records what the scheduler asks of it."""

    max_rows, device = 64, "cpu"

    def __init__(self):
        self.slots = SlotManager(lambda n: None)
        self.max_len, self.steps, self.seen = 0, [], {}

    def ensure(self, n, length):
        self.slots.reserve(n)
        self.max_len = max(self.max_len, length)

    def acquire(self):
        s = self.slots.acquire()
        self.seen[s] = []
        return s

    def release(self, s):
        self.slots.release(s)

    def step(self, entries):
        self.steps.append([(e.slot, e.pos, len(e.tokens)) for e in entries])
        out = []
        for e in entries:
            assert e.pos == len(self.seen[e.slot])
            self.seen[e.slot].extend(e.tokens)
            for k in e.want:
                row = torch.zeros(90)
                row[(e.tokens[k] + 1) % 90] = 1
                out.append(row)
        return torch.stack(out) if out else torch.zeros((0, 90))


def test_scheduler_admits_cuts_decodes_and_frees():
    eng = _FakeEngine()
    s = BatchScheduler(eng, max_batch=2, portion=4, max_len=40)
    reqs = [s.submit(Request([10 * i + j for j in range(n)], new, top_k=1, eos_id=eos))
            for i, (n, new, eos) in enumerate([(9, 3, None), (2, 10, 13), (5, 1, None), (1, 2, None)])]
    s.run()
    assert [r.out for r in reqs] == [[9, 10, 11], [12, 13], [25], [31, 32]]
    assert eng.slots.live == 0 and max(len(x) for x in eng.steps) == 2 and max(n for x in eng.steps for _, _, n in x) == 4
    assert {slot for x in eng.steps for slot, _, _ in x} == {0, 1}  # the third and fourth request took freed slots
    with pytest.raises(ValueError):
        s.submit(Request(list(range(39)), 2))
    with pytest.raises(ValueError):
        s.submit(Request([], 2))


# ---------------------------------------------------------------------------------------- the restatement itself
def test_oracle_window_is_exact_at_both_edges():
    T, w = 12, 4
    q = torch.ones((T, 1, 1)).double()
    k, v = torch.zeros((T, 1, 1)).double(), torch.arange(T).double().view(T, 1, 1)
    out = O.window_attention(q, k, v, 1.0, w)  # equal scores: the mean of the visible rows
    assert torch.allclose(out[:, 0, 0], torch.tensor([sum(range(max(0, i - w + 1), i + 1)) / min(i + 1, w) for i in range(T)]).double())


def test_oracle_rotation_depends_on_distance_only_and_leaves_the_rest():
    q, k = torch.randn((1, 1, 10), dtype=torch.float64).expand(30, 1, 10), torch.randn((1, 1, 10), dtype=torch.float64).expand(30, 1, 10)
    rq, rk = O.rotate_pairs(q, 6, 50.0), O.rotate_pairs(k, 6, 50.0)
    s = (rq[:, 0] @ rk[:, 0].T)
    assert torch.allclose(s[7:, :23].diagonal(), s[7, 0].expand(23)) and torch.equal(rq[..., 6:], q[..., 6:])


def test_oracle_delta_rule_replaces_a_value_and_gla_sums():
    k = torch.zeros((3, 1, 4), dtype=torch.float64)
    k[..., 1] = 1
    v = torch.randn((3, 1, 5), dtype=torch.float64)
    one = torch.ones((3, 1), dtype=torch.float64)
    assert torch.allclose(O.delta_rule(k, k, v, one, one), v)  # the same key with beta 1: the last value
    assert torch.allclose(O.gated_linear_attention(k, k, v, torch.full((3, 1, 4), 0.5, dtype=torch.float64))[2], 0.25 * v[0] + 0.5 * v[1] + v[2])


def test_oracle_is_causal_and_prefix_stable():
    sd = synth.make_hybrid_state_dict(CONFIG, rank=4)
    toks = torch.randint(0, 90, (20,), generator=torch.Generator().manual_seed(0)).tolist()
    a, trail = O.forward(CONFIG, sd, toks)
    b, _ = O.forward(CONFIG, sd, toks[:11])
    assert torch.allclose(a[:11], b) and trail.shape == (7, 20, 36)
    assert set(tensor_shapes(HybridConfig.from_dict(CONFIG), {2: 4})) == set(sd)
