"""Zimorax without a GPU: configuration, the way from a configuration to parts and to the order in which layers run, the
checkpoint adapter, what the layers ask of the cache (every pass through a looped layer has its own), the stretched
frequencies, and the plain implementation's own mechanisms against hand-made cases."""

import math

import pytest
import torch

import fms_amd
import plain_zimorax as P
from fms_amd.architectures import get_architecture
from fms_amd.architectures.registry import variant_config
from fms_amd.cache import KVNeed, SequenceCache
from fms_amd.engine.model import DecoderModel
from fms_amd.kernels import ops
from fms_amd.parts import ModelSpec, PartSpec, ScheduleEntry
from fms_amd.parts.position import rope_frequencies, rope_gain
from fms_amd.weights.adapters import get_adapter, pairs_to_neighbours

SCALING = {"factor": 4.0, "original": 40, "fast": 5.0, "slow": 0.5}


def _attention(**over):
    m = {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 6, "mask": {"size": 70}, "rot": {"base": 100.0, "dims": 4, "scaling": dict(SCALING)}, "scale": 0.3}
    m.update(over)
    return {"type": "attention", "mixer": m}


def _mamba(**over):
    m = {"heads": 4, "vdim": 6, "state": 10, "groups": 2, "conv": 3, "norm_groups": 3}
    m.update(over)
    return {"type": "mamba2", "mixer": m}


def _delta(**over):
    m = {"heads": 4, "kv_heads": 2, "dim": 5, "vdim": 7, "conv": 2}
    m.update(over)
    return {"type": "delta", "mixer": m}


def _config(**over):
    layers = [dict(_mamba(conv=1), mlp={"kind": "dense", "ff": 20}), dict(_attention(), mlp=None), dict(_delta(), mlp={"kind": "dense", "ff": 12}),
              dict(_mamba(), mlp={"kind": "dense", "ff": 8})]
    kw = dict(vocab=40, width=16, layers=layers, norm={"eps": 1e-5}, loop={"start": 1, "stop": 3, "times": 3}, max_positions=512)
    kw.update(over)
    return fms_amd.ZimoraxConfig(**kw)


def test_the_configuration_round_trips_and_refuses_what_no_model_can_be_built_from(tmp_path):
    config = _config()
    config.save(tmp_path / "config.json")
    again = fms_amd.ZimoraxConfig.load(tmp_path / "config.json")
    assert again == config and again.nlayers == 4
    assert _config(loop=None).loop is None
    bad = [dict(layers=[dict(_mamba(), type="convolution", mlp=None)]),
           dict(layers=[dict(_attention(heads=3), mlp=None)]),                      # heads no multiple of key/value heads
           dict(layers=[dict(_mamba(groups=3), mlp=None)]),                         # heads no multiple of groups
           dict(layers=[dict(_mamba(norm_groups=5), mlp=None)]),                    # norm groups that do not divide the channels
           dict(layers=[{"type": "delta", "mixer": {"heads": 2, "kv_heads": 1, "dim": 8}, "mlp": None}]),
           dict(layers=[dict(_attention(rot={"base": 10.0, "dims": 10}), mlp=None)]),  # rotation wider than the head
           dict(layers=[dict(_attention(rot={"base": 10.0, "dims": 4, "scaling": {"factor": 2.0}}), mlp=None)]),
           dict(layers=[dict(_attention(mask={"size": 0}), mlp=None)]),
           dict(layers=[dict(_mamba(), mlp={"kind": "moe", "ff": 4})]),
           dict(loop={"start": 1, "stop": 1, "times": 2}), dict(loop={"start": 0, "stop": 5, "times": 1}), dict(loop={"start": 0, "times": 1}),
           dict(loop={"start": 0, "stop": 2, "times": 0}), dict(norm={}), dict(vocab=0)]
    for kw in bad:
        with pytest.raises(ValueError):
            config_kw = dict(kw)
            if "layers" in kw:
                config_kw["loop"] = None
            _config(**config_kw)


def test_from_the_configuration_to_parts_their_order_and_what_they_ask_of_the_cache():
    arch = get_architecture("Zimorax")  # as config.json writes it
    config = _config()
    spec = arch.build_spec(config)
    assert not spec.tie_heads and spec.final_norm.args == {"eps": 1e-5, "use_mean": True}
    assert [(l.mixer.kind, l.block.kind, l.feed_forward.kind if l.feed_forward else None) for l in spec.layers] == [
        ("mamba2", "pre_norm", "mlp"), ("attention", "pre_norm", None), ("gated_delta", "pre_norm", "mlp"), ("mamba2", "pre_norm", "mlp")]
    # layers 1 and 2 three times in a row, every pass entered once, right before its first layer
    assert [(e.layer, e.enter) for e in spec.schedule] == [
        (0, None), (1, ("loop", 0)), (2, None), (1, ("loop", 1)), (2, None), (1, ("loop", 2)), (2, None), (3, None)]
    a = spec.layers[1].mixer.args
    assert a["window"] == 70 and a["sink"] == 0.0 and a["value_norm"] and a["talking_heads"] and a["qkv_bias"] and not a["out_bias"]
    assert all(l.feed_forward is None or l.feed_forward.args["activation"] == "relu2" for l in spec.layers)
    model = DecoderModel(spec, torch.float32, config=config)
    mixer = model.layers[1].mixer
    assert mixer.fixed_sink == 0.0 and not mixer.has_sink and mixer.extended
    kv, state = model.cache_needs()
    assert kv == [(n, KVNeed(2, 8, 70, value_dim=6)) for n in (1, 3, 5)]
    assert [n for n, _ in state] == [0, 2, 4, 6, 7]
    sizes = {n: dict((name, shape) for name, shape, _ in need.tensors) for n, need in state}
    assert sizes[0] == {"S": (4, 6, 10)}  # a convolution of one tap keeps nothing
    assert sizes[7] == {"S": (4, 6, 10), "conv": (2, 64)}
    assert sizes[2] == sizes[4] == sizes[6] == {"S": (4, 7, 5), "conv": (1, 48)}
    assert all(dtype == "float32" for _, need in state for _, _, dtype in need.tensors)
    names = {n for n, *_ in model.named_specs()}
    for n in ("embed.weight", "head.weight", "loop.in.weight", "loop.step", "l0.ls1", "l0.ls2", "l0.mix.A_log", "l0.mix.D", "l0.mix.conv.bias",
              "l1.mix.talk", "l1.mix.in_proj.qkv_fused.bias", "l2.mlp.up.bias", "l2.mlp.down.bias", "final.norm.weight"):
        assert n in names, n
    assert not names & {"final.norm.bias", "l0.norm1.bias", "l1.norm2.weight", "l1.ls2", "l1.mix.sink", "l1.mix.dense.bias"}
    assert variant_config("zimorax", "micro").nlayers == 5
    assert DecoderModel(arch.build_spec(_config(loop=None)), torch.float32).schedule == [ScheduleEntry(i) for i in range(4)]
    # a schedule cannot enter through what the model does not have
    with pytest.raises(ValueError):
        ModelSpec(8, 8, 8, spec.layers[:1], PartSpec("rmsnorm"), schedule=[ScheduleEntry(0, enter=("other", 0))]).resolved_schedule()


def test_states_of_every_pass_are_zeroed_when_a_slot_is_handed_out_again():
    config = _config()
    model = DecoderModel(get_architecture("zimorax").build_spec(config), torch.float32, config=config)
    kv, state = model.cache_needs()
    cache = SequenceCache(kv, state, max_tokens=64 * 4, max_slots=2, max_seq_len=512, device="cpu")
    a, b = cache.alloc_slot(), cache.alloc_slot()
    for tensors in cache.state.values():
        for t in tensors.values():
            t.fill_(3.0)
    cache.free_slot(a)
    assert cache.alloc_slot() == a
    for tensors in cache.state.values():
        for t in tensors.values():
            assert float(t[a].abs().max()) == 0.0 and float(t[b].min()) == 3.0
    cache.extend(a, 140)
    cache.extend(a, 1)  # a window of 70 at position 140: the first page goes back in every pass's group
    assert [p >= 0 for p in cache.groups[0].pages[a]] == [False, True, True]
    cache.check()


def test_the_adapter_gives_every_tensor_its_place():
    config = _config()
    arch = get_architecture("zimorax")
    gen = torch.Generator().manual_seed(0)
    sd = {name: torch.randn(shape, generator=gen) for name, shape, _ in arch.hf_tensor_layout(config)}
    out = get_adapter("zimorax", "hf")(dict(sd), model_config=config)
    model = DecoderModel(arch.build_spec(config), torch.float32, config=config)
    assert {n: tuple(t.shape) for n, t in out.items()} == {full: spec.shape for full, spec, _, _ in model.named_specs()}
    # 4 of a head's 8 entries turn: rows 0, 2, 1, 3 of every head's rotated run, then the rest as they were; values as they are
    fused, src = out["l1.mix.in_proj.qkv_fused.weight"], sd["l1.mix.q"].view(4, 8, 16)
    assert torch.equal(fused[:32].view(4, 8, 16)[:, :4], src[:, [0, 2, 1, 3]]) and torch.equal(fused[:32].view(4, 8, 16)[:, 4:], src[:, 4:])
    bias = out["l1.mix.in_proj.qkv_fused.bias"]
    assert torch.equal(bias[32:48].view(2, 8)[:, :4], sd["l1.mix.k.b"].view(2, 8)[:, [0, 2, 1, 3]]) and torch.equal(bias[48:], sd["l1.mix.v.b"])
    assert torch.equal(fused[48:], sd["l1.mix.v"]) and torch.equal(out["l1.mix.talk"], sd["l1.mix.talk"])
    assert torch.equal(out["l2.mix.in_proj.weight"], torch.cat([sd[f"l2.mix.{n}"] for n in ("q", "k", "v", "b", "a", "g")]))
    assert torch.equal(out["l2.mix.conv.weight"], torch.cat([sd[f"l2.mix.{n}.conv"] for n in ("q", "k", "v")]))
    assert torch.equal(out["l3.mix.in_proj.weight"], sd["l3.mix.in"]) and torch.equal(out["l3.mix.conv.bias"], sd["l3.mix.conv.b"])
    assert torch.equal(out["loop.in.weight"], sd["loop.in"]) and torch.equal(out["loop.step"], sd["loop.step"])
    # the parts that the fused projection is made of, in the order of its rows
    rows = dict(model.layers[3].mixer.unfused_parameters()["in_proj"])
    assert list(rows) == ["z", "x", "B", "C", "dt"] and sum(rows.values()) == sd["l3.mix.in"].shape[0]


def test_stretched_frequencies():
    """The library's against the plain ones, and the three regions: dimensions that turn often keep their frequency, slow
    ones are divided by the factor, those between lie between."""
    for dims, base, s in ((24, 1e4, dict(factor=8.0, original=4096, fast=32.0, slow=1.0)), (6, 100.0, SCALING), (64, 5e5, dict(SCALING, factor=1.0)),
                          (16, 1e4, dict(factor=4.0, original=64, fast=1.0, slow=1.0))):  # the last one: both bounds fall together
        want, gain = P.yarn_frequencies({"dims": dims, "base": base, "scaling": s})
        kw = {"rope_type": "yarn", "factor": s["factor"], "original_max_position_embeddings": s["original"], "beta_fast": s["fast"], "beta_slow": s["slow"]}
        got = rope_frequencies(dims, base, kw, exact=True)
        assert got.dtype == torch.float32 and torch.allclose(got.double(), torch.tensor(want, dtype=torch.float64), rtol=1e-7)
        assert rope_gain(kw) == pytest.approx(gain) == pytest.approx(0.1 * math.log(s["factor"]) + 1)
    plain = [1e4 ** (-2 * i / 24) for i in range(12)]
    f, _ = P.yarn_frequencies({"dims": 24, "base": 1e4, "scaling": dict(factor=8.0, original=4096, fast=32.0, slow=1.0)})
    assert f[0] == plain[0] and f[11] == pytest.approx(plain[11] / 8)
    assert any(plain[i] / 8 < f[i] * (1 - 1e-9) and f[i] < plain[i] * (1 - 1e-9) for i in range(12))
    assert rope_gain(None) == rope_gain({"rope_type": "linear", "factor": 2.0}) == 1.0


def test_turning_neighbours_equals_turning_halves():
    gen = torch.Generator().manual_seed(1)
    rot = {"base": 100.0, "dims": 6, "scaling": SCALING}
    q, k = torch.randn(5, 1, 10, generator=gen, dtype=torch.float64), torch.randn(5, 1, 10, generator=gen, dtype=torch.float64)
    pos = torch.tensor([0, 3, 4, 90, 1000])
    want = (P.rotate_halves(q, pos, rot) * P.rotate_halves(k, pos, rot)).sum(-1)
    freqs, gain = P.yarn_frequencies(rot)

    def neighbours(v):
        v = pairs_to_neighbours(v[:, 0].T.contiguous(), 1, 0, 6).T  # rows of a weight are a vector's entries
        angle = pos.double()[:, None] * torch.tensor(freqs, dtype=torch.float64)[None, :]
        a, b = v[:, 0:6:2], v[:, 1:6:2]
        turned = torch.stack([a * torch.cos(angle) - b * torch.sin(angle), b * torch.cos(angle) + a * torch.sin(angle)], dim=-1).reshape(5, 6)
        return torch.cat([gain * turned, v[:, 6:]], dim=1)

    assert torch.allclose((neighbours(q) * neighbours(k)).sum(-1), want[:, 0], atol=1e-9)


def test_what_the_host_decides():
    assert ops.talking_splits(1, 16, 8192, 1024) == 9 and ops.talking_splits(64, 16, 8192, 1024) == 4  # 33 tiles, four a block
    assert ops.talking_splits(300, 16, 8192, 1024) == 1 and ops.talking_splits(1, 16, 8192, 0) == 64
    assert ops.talking_splits(1, 40, 64, 0) == 1
    with pytest.raises(RuntimeError):
        ops.stream_rows(torch.zeros(2, 4), None, None, torch.zeros(2, 4))  # no CPU path
    from fms_amd.parts import Mamba2, MultiHeadAttention

    with pytest.raises(ValueError):
        Mamba2(16, heads=4, vdim=8, state=300, groups=2)
    with pytest.raises(ValueError):
        Mamba2(16, heads=4, vdim=8, state=16, groups=2, norm_groups=5)
    for kw in (dict(soft_cap=5.0), dict(chunk=4), dict(window=4, keep_first=1)):
        with pytest.raises(NotImplementedError):
            MultiHeadAttention(16, 2, 1, 8, talking_heads=True, **kw)
    with pytest.raises(NotImplementedError):
        MultiHeadAttention(16, 2, 1, 8, value_norm=True, qk_norm="head")
    assert MultiHeadAttention(16, 2, 1, 8, sink=True).has_sink and MultiHeadAttention(16, 2, 1, 8, sink=-2).fixed_sink == -2.0
    assert MultiHeadAttention(16, 2, 1, 8).fixed_sink is None


def test_the_plain_mechanisms_on_cases_worked_by_hand():
    f64 = lambda *v: torch.tensor(v, dtype=torch.float64)  # noqa: E731
    # layer norm: the variance is the mean of the squared deviations, no shift
    assert torch.allclose(P.layer_norm(f64([1.0, 3.0])[None], f64(2.0, 2.0), 0.0), f64([-2.0, 2.0])[None])
    # a convolution: the last column is the token's own, zeros before the start
    assert torch.allclose(P.causal_conv(f64([1.0], [2.0], [4.0]), f64([10.0, 1.0]), f64(0.5)), f64([1.5], [12.5], [24.5]))
    # a sink of score zero takes half of the weight of one key of score zero, and the window counts the token itself
    assert torch.allclose(P.softmax_with_null_sink(torch.zeros(1, 1, 1, dtype=torch.float64), torch.ones(1, 1, dtype=torch.bool)), f64([[0.5]]))
    assert P.window(4, 2)[3].tolist() == [False, False, True, True]
    # mixed scores: head 0 takes head 1's, head 1 the sum of both
    q, k = f64([[1.0, 0.0], [0.0, 2.0]]), f64([[3.0, 5.0]])
    assert P.talking_scores(q, k, 0.5, f64([0.0, 1.0], [1.0, 1.0])).flatten().tolist() == [5.0, 6.5]
    # a quarter turn without stretching: (u, v) -> (-v, u)
    rot = {"base": 7.0, "dims": 2, "scaling": {"factor": 1.0, "original": 10, "fast": 2.0, "slow": 1.0}}
    assert torch.allclose(P.rotate_halves(f64([[1.0, 2.0, 9.0]]), f64(math.pi / 2), rot), f64([[-2.0, 1.0, 9.0]]), atol=1e-12)
    # the state-space recurrence, two tokens: S = d B x, then decayed by exp(-d)
    x, B, C, dt = f64([[2.0]], [[1.0]]), f64([[3.0]], [[1.0]]), f64([[1.0]], [[10.0]]), f64([0.5], [1.0])
    y = P.ssd_recurrence(x, B, C, dt, f64(0.0), f64(100.0))
    assert y.flatten().tolist() == pytest.approx([3.0 + 200.0, 10 * (3.0 * math.exp(-1) + 1.0) + 100.0])
    # the delta rule reads its own write; a second write of the same key replaces the first with beta = 1
    one = f64([[1.0]], [[1.0]])
    o = P.delta_recurrence(one, one, f64([[5.0]], [[7.0]]), f64([1.0], [1.0]), f64([1.0], [1.0]))
    assert o.flatten().tolist() == [5.0, 7.0]
    # the gate comes before the norm, and every part has its own
    got = P.gated_group_norm(f64([3.0, 4.0, 100.0, 100.0])[None], f64([50.0] * 4)[None], f64(1.0, 1.0, 2.0, 2.0), 2, 0.0)
    assert torch.allclose(got, f64([3 / math.sqrt(12.5), 4 / math.sqrt(12.5), 2.0, 2.0])[None])
    assert P.run_order({"layers": [0, 0, 0], "loop": {"start": 1, "stop": 2, "times": 2}}) == [(0, None), (1, 0), (1, 1), (2, None)]
