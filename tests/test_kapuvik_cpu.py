"""Kapuvik without a GPU: configuration, the way from a configuration to parts and to the order in which layers run, the
checkpoint adapter, what the layers ask of the cache (every pass through a looped layer has its own), projections that
join, and the plain implementation's own mechanisms against hand-made cases."""

import copy
import math

import pytest
import torch

import fms_amd
import plain_kapuvik as P
from fms_amd.architectures import get_architecture
from fms_amd.architectures.registry import variant_config
from fms_amd.cache import KVNeed, SequenceCache
from fms_amd.engine.model import DecoderModel
from fms_amd.kernels import ops
from fms_amd.parts import JointProjection, LinearRecurrence, ParallelMixers, ScheduleEntry
from fms_amd.parts.linear import Linear
from fms_amd.weights.adapters import get_adapter


def _parallel(**over):
    m = {"left": {"heads": 4, "kv_heads": 2, "dim": 8, "vdim": 6, "rot": {"base": 100.0, "dims": 4}, "scale": 0.3, "softcap": 9.0},
         "right": {"heads": 3, "dim": 6, "vdim": 5, "rot": {"base": 50.0, "dims": 4}, "decay": [0.5, 0.9, 1.0]}, "left_scale": 0.5, "right_scale": 2.0}
    m.update(over)
    return {"type": "parallel", "mixer": m}


def _latent(**over):
    m = {"heads": 2, "dim": 6, "rot_dim": 4, "vdim": 7, "kv_rank": 10, "scale": 0.2, "rot": {"base": 70.0, "dims": 4}}
    m.update(over)
    return {"type": "latent_attention", "mixer": m}


def _gla(**over):
    m = {"heads": 2, "dim": 5, "vdim": 9, "tau": 4.0, "decay_rank": 3}
    m.update(over)
    return {"type": "gla", "mixer": m}


def _config(**over):
    layers = [dict(_gla(), mlp={"kind": "dense", "ff": 20, "limit": 1.0}), dict(_parallel(), mlp=None), dict(_latent(), mlp={"kind": "dense", "ff": 12, "limit": 2.0}),
              dict(_gla(heads=1), mlp={"kind": "dense", "ff": 8, "limit": 7.0})]
    kw = dict(vocab=40, width=16, embedding={"scale": 2.5}, layers=layers, norm={"eps": 1e-5}, loop={"start": 1, "stop": 3, "times": 3},
              logit_softcap=11.0, max_positions=512)
    kw.update(over)
    return fms_amd.KapuvikConfig(**kw)


def test_the_configuration_round_trips_and_refuses_what_no_model_can_be_built_from(tmp_path):
    config = _config()
    config.save(tmp_path / "config.json")
    again = fms_amd.KapuvikConfig.load(tmp_path / "config.json")
    assert again == config and again.nlayers == 4
    assert _config(loop=None).loop is None and _config(logit_softcap=None).logit_softcap is None
    left, right = _parallel()["mixer"]["left"], _parallel()["mixer"]["right"]
    bad = [dict(layers=[dict(_gla(), type="convolution", mlp=None)]),
           dict(layers=[dict(_parallel(left=dict(left, heads=3)), mlp=None)]),                    # heads no multiple of key/value heads
           dict(layers=[dict(_parallel(left=dict(left, rot={"base": 10.0, "dims": 10})), mlp=None)]),  # rotation wider than the head
           dict(layers=[dict(_parallel(right=dict(right, rot={"base": 10.0, "dims": 3})), mlp=None)]),  # an odd number of rotated entries
           dict(layers=[dict(_parallel(right=dict(right, decay=[0.5])), mlp=None)]),              # a decay for every head
           dict(layers=[{"type": "parallel", "mixer": {"left": left, "right": right}, "mlp": None}]),  # no scales
           dict(layers=[{"type": "gla", "mixer": {"heads": 2, "dim": 5, "vdim": 9}, "mlp": None}]),
           dict(layers=[dict(_gla(tau=0.0), mlp=None)]), dict(layers=[dict(_latent(rot_dim=3), mlp=None)]),
           dict(layers=[dict(_gla(), mlp={"kind": "moe", "ff": 4, "limit": 1.0})]), dict(layers=[dict(_gla(), mlp={"kind": "dense", "ff": 4})]),
           dict(loop={"start": 1, "stop": 1, "times": 2}), dict(loop={"start": 0, "stop": 5, "times": 1}), dict(loop={"start": 0, "times": 1}),
           dict(loop={"start": 0, "stop": 2, "times": 0}), dict(norm={}), dict(vocab=0), dict(logit_softcap=-1.0)]
    for kw in bad:
        with pytest.raises(ValueError):
            config_kw = dict(kw)
            if "layers" in kw:
                config_kw["loop"] = None
            _config(**config_kw)


def test_the_rank_of_the_decays_comes_from_the_tensors():
    arch = get_architecture("kapuvik")
    layers = copy.deepcopy(_config().layers)
    for entry in layers:
        entry["mixer"].pop("decay_rank", None)
    config = _config(layers=layers)
    with pytest.raises(ValueError):
        arch.build_spec(config)
    config = arch.sizes_from_tensors(config, {"l0.mix.a1": (7, 16), "l3.mix.a1": (2, 16), "l1.mix.left.q": (32, 16)})
    assert config.layers[0]["mixer"]["decay_rank"] == 7 and config.layers[3]["mixer"]["decay_rank"] == 2 and "decay_rank" not in layers[0]["mixer"]


def test_from_the_configuration_to_parts_their_order_and_what_they_ask_of_the_cache():
    arch = get_architecture("Kapuvik")  # as config.json writes it
    config = _config()
    spec = arch.build_spec(config)
    assert not spec.tie_heads and spec.embedding.args == {"scale": 2.5} and spec.head.args == {"soft_cap": 11.0}
    assert arch.build_spec(_config(logit_softcap=None)).head.args == {"soft_cap": 0.0}
    assert [(l.mixer.kind, l.block.kind, l.feed_forward.kind if l.feed_forward else None) for l in spec.layers] == [
        ("linear_recurrence", "parallel", "glu"), ("parallel", "parallel", None), ("latent_attention", "parallel", "glu"), ("linear_recurrence", "parallel", "glu")]
    # layers 1 and 2 three times in a row, every pass entered once, right before its first layer
    assert [(e.layer, e.enter) for e in spec.schedule] == [
        (0, None), (1, ("loop", 0)), (2, None), (1, ("loop", 1)), (2, None), (1, ("loop", 2)), (2, None), (3, None)]
    assert not spec.entrances["loop"].args["at_start"]
    assert arch.build_spec(_config(loop={"start": 0, "stop": 2, "times": 1})).entrances["loop"].args["at_start"]
    assert [l.feed_forward.args["limit"] for l in spec.layers if l.feed_forward] == [1.0, 2.0, 7.0]
    model = DecoderModel(spec, torch.float32, config=config)
    mixer = model.layers[1].mixer
    left, right = mixer.sides
    assert left.soft_cap == 9.0 and left.scale == 0.3 and mixer.scales == (0.5, 2.0) and right.decay == [0.5, 0.9, 1.0]
    # every side of the parallel mixer turns by its own table
    assert (left.position_encoder.rot_dim, left.position_encoder.theta) == (4, 100.0) and (right.position_encoder.rot_dim, right.position_encoder.theta) == (4, 50.0)
    assert not right.has_norm_weight and model.layers[0].mixer.has_norm_weight and model.layers[0].mixer.position_encoder is None
    kv, state = model.cache_needs()
    assert kv == [e for n in (1, 3, 5) for e in ((n, KVNeed(2, 8, value_dim=6)), (n + 1, KVNeed(1, 14, values=False)))]
    assert [(n, need.tensors) for n, need in state] == [(0, (("S", (2, 9, 5), "float32"),))] + [
        (n, (("right.S", (3, 5, 6), "float32"),)) for n in (1, 3, 5)] + [(7, (("S", (1, 9, 5), "float32"),))]
    names = {n for n, *_ in model.named_specs()}
    for n in ("embed.weight", "head.weight", "loop.step", "l0.norm1.weight", "l0.mix.decay_up.bias", "l0.mix.norm.weight", "l1.mix.left.dense.weight",
              "l1.mix.right.out.weight", "l2.mix.kv_norm.weight", "l2.mlp.wg1_fused.bias", "l2.mlp.w2.bias", "final.norm.weight"):
        assert n in names, n
    assert not names & {"l0.norm2.weight", "l1.mix.right.norm.weight", "l1.mix.left.in_proj.qkv_fused.bias", "loop.in.weight", "l2.mix.sink"}
    assert variant_config("kapuvik", "micro").nlayers == 5
    assert DecoderModel(arch.build_spec(_config(loop=None)), torch.float32).schedule == [ScheduleEntry(i) for i in range(4)]


def test_states_of_every_pass_are_zeroed_when_a_slot_is_handed_out_again():
    config = _config()
    model = DecoderModel(get_architecture("kapuvik").build_spec(config), torch.float32, config=config)
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
    assert all(p >= 0 for group in cache.groups for p in group.pages[a])  # nothing is given back: every key stays visible
    cache.check()


def test_the_adapter_gives_every_tensor_its_place():
    config = _config()
    arch = get_architecture("kapuvik")
    gen = torch.Generator().manual_seed(0)
    sd = {name: torch.randn(shape, generator=gen) for name, shape, _ in arch.hf_tensor_layout(config)}
    assert arch.detect_source(list(sd)) == "hf"
    out = get_adapter("kapuvik", "hf")(dict(sd), model_config=config)
    assert arch.detect_source(list(out)) == "fms"
    model = DecoderModel(arch.build_spec(config), torch.float32, config=config)
    assert {n: tuple(t.shape) for n, t in out.items()} == {full: spec.shape for full, spec, _, _ in model.named_specs()}
    # retention turns halves: rows 0, 2, 1, 3 of every head's rotated run, then the rest; attention's neighbours stay
    fused, src = out["l1.mix.right.in_proj.weight"], sd["l1.mix.right.k"].view(3, 6, 16)
    assert torch.equal(fused[18:36].view(3, 6, 16)[:, :4], src[:, [0, 2, 1, 3]]) and torch.equal(fused[18:36].view(3, 6, 16)[:, 4:], src[:, 4:])
    assert torch.equal(fused[36:], torch.cat([sd["l1.mix.right.v"], sd["l1.mix.right.g"]]))
    assert torch.equal(out["l1.mix.left.in_proj.qkv_fused.weight"], torch.cat([sd[f"l1.mix.left.{n}"] for n in "qkv"]))
    assert torch.equal(out["l2.mix.down.weight"], torch.cat([sd["l2.mix.q"], sd["l2.mix.dkv"]]))
    assert torch.equal(out["l0.mix.in_proj.weight"], torch.cat([sd[f"l0.mix.{n}"] for n in ("q", "k", "v", "g", "a1")]))
    assert torch.equal(out["l0.mix.decay_up.weight"], sd["l0.mix.a2"]) and torch.equal(out["l0.mix.decay_up.bias"], sd["l0.mix.a2.b"])
    assert torch.equal(out["l2.mlp.wg1_fused.bias"], torch.cat([sd["l2.mlp.gate.b"], sd["l2.mlp.up.b"]]))
    assert torch.equal(out["l2.mlp.w2.bias"], sd["l2.mlp.down.b"]) and torch.equal(out["loop.step"], sd["loop.step"])
    # the parts that the fused projection is made of, in the order of its rows
    rows = dict(model.layers[3].mixer.unfused_parameters()["in_proj"])
    assert list(rows) == ["q", "k", "v", "g", "a1"] and sum(rows.values()) == out["l3.mix.in_proj.weight"].shape[0]


def test_projections_that_join_keep_their_names_and_become_views():
    gen = torch.Generator().manual_seed(1)
    a, b, c = Linear(4, 6), Linear(3, 6), Linear(5, 6, bias=True)
    weights = [torch.randn(6, n, generator=gen) for n in (4, 3, 5)]
    for lin, w in zip((a, b, c), weights):
        lin.bind("weight", w.clone())
    c.bind("bias", torch.arange(6.0))
    joint = JointProjection([a, b, c])
    joint.join()
    x = torch.randn(2, 12, generator=gen)
    want = x[:, :4] @ weights[0].T + x[:, 4:7] @ weights[1].T + x[:, 7:] @ weights[2].T + torch.arange(6.0)
    assert torch.allclose(x @ joint.w["weight"].T + joint.w["bias"], want, atol=1e-5)
    for lin, w in zip((a, b, c), weights):
        assert torch.equal(lin.w["weight"], w) and lin.w["weight"].untyped_storage().data_ptr() == joint.w["weight"].untyped_storage().data_ptr()
    with pytest.raises(NotImplementedError):
        JointProjection([Linear(2, 3, bias=True), Linear(2, 3, bias=True)])
    with pytest.raises(NotImplementedError):
        JointProjection([Linear(2, 3), Linear(2, 4)])
    # a block of a parallel mixer and a feed-forward joins three projections, and the mixer leaves its own to the block
    config = _config(layers=[dict(_parallel(), mlp={"kind": "dense", "ff": 12, "limit": 1.0})], loop=None)
    block = DecoderModel(get_architecture("kapuvik").build_spec(config), torch.float32, config=config).layers[0]
    assert [l.in_features for l in block.joint.layers] == [24, 15, 12] and block.joint.has_bias and block.mixer._joint is None


def test_what_the_host_refuses():
    with pytest.raises(RuntimeError):
        ops.stream_enter(torch.zeros(2, 4))  # no CPU path
    with pytest.raises(RuntimeError):
        ops.soft_cap_(torch.zeros(4), 1.0)
    for kw in (dict(), dict(decay=[0.5, 0.5], decay_rank=3), dict(decay=[0.5]), dict(decay=[0.5, 0.0]), dict(decay=[0.5, 1.5]), dict(decay_rank=2, tau=0.0),
               dict(decay_rank=2, gate_activation="none")):
        with pytest.raises(ValueError):
            LinearRecurrence(16, heads=2, dim=4, vdim=4, **kw)
    with pytest.raises(ValueError):
        LinearRecurrence(16, heads=2, dim=300, vdim=4, decay_rank=2)
    from fms_amd.parts import GatedLinearUnit, LinearHead

    with pytest.raises(ValueError):
        GatedLinearUnit(16, 8, limit=0.0)
    with pytest.raises(ValueError):
        LinearHead(8, 8, soft_cap=-1.0)
    with pytest.raises(ValueError):  # two mixers that both keep keys and values
        side = {"kind": "attention", "args": {"nheads": 2, "kvheads": 1, "head_dim": 8}}
        ParallelMixers(16, side, side)


def test_the_plain_mechanisms_on_cases_worked_by_hand():
    f64 = lambda *v: torch.tensor(v, dtype=torch.float64)  # noqa: E731
    # a scale stored around zero
    assert torch.allclose(P.zero_centred_norm(f64([3.0, 4.0])[None], f64(0.0, 1.0), 0.0), f64([3 / math.sqrt(12.5), 8 / math.sqrt(12.5)])[None])
    # a quarter turn: (u, v) -> (-v, u), of neighbours and of halves, the rest as it was
    rot = {"base": 1e9, "dims": 4}
    v = f64([[1.0, 2.0, 3.0, 4.0, 9.0]])
    quarter = f64(math.pi / 2)
    assert torch.allclose(P.rotate(v, quarter, rot, halves=False)[0, 0, [0, 1, 4]], f64(-2.0, 1.0, 9.0), atol=1e-12)
    assert torch.allclose(P.rotate(v, quarter, rot, halves=True)[0, 0, [0, 2, 4]], f64(-3.0, 1.0, 9.0), atol=1e-12)
    assert P.soft_cap(f64(1e9), 5.0).item() == 5.0 and P.soft_cap(f64(3.0), None).item() == 3.0
    # the recurrence, two tokens: the decay acts on what was there, the read-out sees the token's own write
    o = P.linear_recurrence(f64([[1.0, 1.0]], [[1.0, 10.0]]), f64([[1.0, 2.0]], [[1.0, 0.0]]), f64([[3.0]], [[5.0]]), f64([[0.1, 0.1]], [[0.5, 0.25]]))
    assert o.flatten().tolist() == [9.0, 0.5 * 3 + 5 + 10 * 0.25 * 6]
    # sigmoid to the power 1 / tau
    d = P.channel_decays(f64([0.0]), {"a1": f64([1.0]), "a2": f64([1.0], [1.0]), "a2.b": f64(0.0, math.log(3.0))}, {"tau": 2.0, "heads": 1, "dim": 2})
    assert torch.allclose(d.flatten(), f64(math.sqrt(0.5), math.sqrt(0.75)))
    # the clamped unit: gate clamped above only, up on both sides, plus one
    one = f64([1.0])
    w = {"gate": one, "gate.b": f64(0.0), "up": f64([-5.0]), "up.b": f64(0.0), "down": one, "down.b": f64(0.25)}
    g = 2.0 / (1 + math.exp(-1.702 * 2.0))
    assert P.feed_forward(f64([7.0]), w, {"limit": 2.0}).item() == pytest.approx(g * (-2.0 + 1) + 0.25)
    assert P.feed_forward(f64([-7.0]), w, {"limit": 2.0}).item() == pytest.approx(-7.0 / (1 + math.exp(1.702 * 7.0)) * (2.0 + 1) + 0.25)
    assert P.run_order({"layers": [0, 0, 0], "loop": {"start": 1, "stop": 2, "times": 2}}) == [(0, None), (1, 0), (1, 1), (2, None)]
