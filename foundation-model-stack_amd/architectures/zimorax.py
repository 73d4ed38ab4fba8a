"""Zimorax: from its configuration to parts, and from its checkpoint's tensor names to the model's.

The model: a token embedding; layers in the order config.json lists them, some of them run several times in a row with
the same weights; each a pre-norm block with layer norms (a weight, no shift) and a learned scale per channel on every
branch; three kinds of mixers (see config/zimorax.py); a plain feed-forward with the square of relu, or none; a final
layer norm and a head of its own.  Every pass through the looped layers owns a cache and states of its own (a schedule
entry each) and is entered by replacing the stream x with W_in [x; x0] + step_t, x0 the embedding's output.

A checkpoint names a layer's tensors ``l<i>.<part>`` without a ".weight" and a bias ``<tensor>.b``; the adapter gives them
the model's names and fuses what the model runs as one product (everything that reads a mixer's input).  The checkpoint
pairs rotated entry i of a head with entry i + dims/2; the rotation kernels turn neighbouring pairs, so the adapter moves
the rows of queries and keys alike (a score is a sum over entries and does not care about their order).
"""

from __future__ import annotations

import re
from typing import List, Tuple

import torch

from ..config import ZimoraxConfig
from ..parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from ..weights.adapters import fuse_gated_delta, pairs_to_neighbours, register_adapter, register_adapter_step
from .registry import Architecture, register_architecture, register_model

NAME = "zimorax"
# what the design fixes
ACTIVATION = "relu2"  # the feed-forward's activation
SINK = 0.0  # the score of the sink in the attention's softmax
LOOP = "loop"  # the name of the loop's entry among the model's parts


def _rope_key(rot: dict, size: int) -> str:
    sc = rot.get("scaling") or {}
    return f"rope_{size}_{rot['dims']}_{rot['base']!r}_" + "_".join(f"{k}{sc[k]!r}" for k in sorted(sc))


def _rope_spec(rot: dict, size: int, max_positions: int) -> PartSpec:
    args = {"dim": size, "rot_dim": rot["dims"], "theta": rot["base"], "max_seq_len": max_positions, "exact_frequencies": True}
    sc = rot.get("scaling")
    if sc:
        args["scaling"] = {"rope_type": "yarn", "factor": sc["factor"], "original_max_position_embeddings": sc["original"],
                           "beta_fast": sc["fast"], "beta_slow": sc["slow"]}
    return PartSpec("rope", args)


def run_order(config: ZimoraxConfig) -> List[ScheduleEntry]:
    """The layers in the order in which they run; an entry that starts a pass through the loop names what comes before it."""
    loop, n = config.loop, len(config.layers)
    if loop is None:
        return [ScheduleEntry(i) for i in range(n)]
    out = [ScheduleEntry(i) for i in range(loop["start"])]
    for t in range(loop["times"]):
        for i in range(loop["start"], loop["stop"]):
            out.append(ScheduleEntry(i, enter=(LOOP, t) if i == loop["start"] else None))
    return out + [ScheduleEntry(i) for i in range(loop["stop"], n)]


def zimorax_spec(config: ZimoraxConfig) -> ModelSpec:
    eps = config.norm["eps"]
    norm = PartSpec("parameterized", {"eps": eps, "use_mean": True})
    layers, positions = [], {}
    for layer in config.layers:
        m, kind, key = layer["mixer"], layer["type"], None
        if kind == "attention":
            key = _rope_key(m["rot"], m["dim"])
            positions.setdefault(key, _rope_spec(m["rot"], m["dim"], config.max_positions))
            mixer = PartSpec("attention", {
                "nheads": m["heads"], "kvheads": m["kv_heads"], "head_dim": m["dim"], "value_dim": m["vdim"], "qkv_bias": True, "out_bias": False,
                "scale_factor": m["scale"], "window": m["mask"]["size"], "sink": SINK, "value_norm": True, "norm_eps": eps, "talking_heads": True,
            })
        elif kind == "mamba2":
            mixer = PartSpec("mamba2", {"heads": m["heads"], "vdim": m["vdim"], "state": m["state"], "groups": m["groups"], "conv": m["conv"],
                                        "norm_groups": m["norm_groups"], "eps": eps})
        else:
            mixer = PartSpec("gated_delta", {"heads": m["heads"], "kv_heads": m["kv_heads"], "dim": m["dim"], "vdim": m["vdim"], "conv": m["conv"],
                                             "eps": eps, "gate_activation": "silu"})
        mlp = layer.get("mlp")
        ff = PartSpec("mlp", {"hidden_dim": mlp["ff"], "activation": ACTIVATION, "use_bias": True}) if mlp is not None else None
        block = PartSpec("pre_norm", {"names": ("norm1", "mix", "norm2", "mlp"), "branch_scales": ("ls1", "ls2"), "width": config.width})
        layers.append(LayerSpec(mixer=mixer, feed_forward=ff, norm=norm, block=block, position=key))
    loops = {LOOP: PartSpec("concat_linear", {"passes": config.loop["times"]})} if config.loop is not None else {}
    return ModelSpec(
        vocab=config.vocab, width=config.width, max_seq_len=config.max_positions, layers=layers, final_norm=norm, positions=positions,
        schedule=run_order(config), entrances=loops,
        embedding_name="embed", layer_name="l{i}", final_norm_name="final.norm", head_name="head",
    )


# ---- the checkpoint's names -> the model's ----------------------------------------------------------------------
def _to_model_names(sd, model_config=None, **kw):
    out = dict(sd)
    for name in [n for n in out if n.endswith(".mix.o")]:
        p = name[: -len("o")]
        layer = model_config.layers[int(re.match(r"l(\d+)\.", name).group(1))]
        m, kind = layer["mixer"], layer["type"]
        if kind == "delta":
            fuse_gated_delta(out, p)
        elif kind == "mamba2":
            for src, dst in (("in", "in_proj.weight"), ("conv", "conv.weight"), ("conv.b", "conv.bias"), ("norm", "norm.weight"), ("o", "out.weight")):
                out[p + dst] = out.pop(p + src)
        else:
            weights = {n: out.pop(p + n) for n in ("q", "k", "v")}
            biases = {n: out.pop(p + n + ".b") for n in ("q", "k", "v")}
            for n, heads in (("q", m["heads"]), ("k", m["kv_heads"])):
                weights[n] = pairs_to_neighbours(weights[n], heads, 0, m["rot"]["dims"])
                biases[n] = pairs_to_neighbours(biases[n], heads, 0, m["rot"]["dims"])
            out[p + "in_proj.qkv_fused.weight"] = torch.cat(list(weights.values()), dim=0)
            out[p + "in_proj.qkv_fused.bias"] = torch.cat(list(biases.values()), dim=0)
            out[p + "dense.weight"] = out.pop(p + "o")
        if layer.get("mlp") is None:  # a layer without a feed-forward has no use for that branch's norm and scale
            for n in ("norm2", "ls2"):
                out.pop(name[: -len("mix.o")] + n, None)
    renamed = {}
    for name, t in out.items():
        if re.search(r"\.mlp\.(up|down)\.b$", name):
            name = name[: -len(".b")] + ".bias"
        elif re.search(r"(^embed|^head|^loop\.in|^final\.norm|\.norm[12]|\.mlp\.(up|down))$", name):
            name += ".weight"
        renamed[name] = t
    return renamed


register_adapter_step(NAME, "checkpoint_to_model_names", _to_model_names)
register_adapter(NAME, "hf", ["checkpoint_to_model_names"])


def detect_source(names: List[str]) -> str:
    return "fms" if any(n.endswith(".weight") for n in names) else "hf"


def checkpoint_tensor_layout(config: ZimoraxConfig) -> List[Tuple[str, Tuple[int, ...], str]]:
    """(name, shape, init) of every tensor of a Zimorax checkpoint of this configuration."""
    W = config.width
    out = [("embed", (config.vocab, W), "normal")]
    if config.loop is not None:
        out += [("loop.in", (W, 2 * W), "normal"), ("loop.step", (config.loop["times"], W), "normal")]
    for i, layer in enumerate(config.layers):
        p, m, kind = f"l{i}.", layer["mixer"], layer["type"]
        q = p + "mix."
        out.append((p + "norm1", (W,), "ones"))
        if kind == "mamba2":
            H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
            inner, channels = H * P, H * P + 2 * G * N
            out += [(q + "in", (inner + channels + H, W), "normal"), (q + "conv", (channels, m["conv"]), "normal"), (q + "conv.b", (channels,), "zeros"),
                    (q + "dt_bias", (H,), "zeros"), (q + "A_log", (H,), "zeros"), (q + "D", (H,), "ones"), (q + "norm", (inner,), "ones"),
                    (q + "o", (W, inner), "normal")]
        elif kind == "delta":
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for n, rows in (("q", G * D), ("k", G * D), ("v", H * V)):
                out += [(q + n, (rows, W), "normal"), (q + n + ".conv", (rows, m["conv"]), "normal")]
            out += [(q + "b", (H, W), "normal"), (q + "A_log", (H,), "zeros"), (q + "norm", (V,), "ones"), (q + "a", (H, W), "normal"),
                    (q + "dt_bias", (H,), "zeros"), (q + "g", (H * V, W), "normal"), (q + "o", (W, H * V), "normal")]
        else:
            H, G, D, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            for n, rows in (("q", H * D), ("k", G * D), ("v", G * V)):
                out += [(q + n, (rows, W), "normal"), (q + n + ".b", (rows,), "zeros")]
            out += [(q + "talk", (H, H), "normal"), (q + "o", (W, H * V), "normal")]
        out.append((p + "ls1", (W,), "ones"))
        mlp = layer.get("mlp")
        if mlp is not None:
            F = mlp["ff"]
            out += [(p + "norm2", (W,), "ones"), (p + "mlp.up", (F, W), "normal"), (p + "mlp.up.b", (F,), "zeros"),
                    (p + "mlp.down", (W, F), "normal"), (p + "mlp.down.b", (W,), "zeros"), (p + "ls2", (W,), "ones")]
    return out + [("final.norm", (W,), "ones"), ("head", (config.vocab, W), "normal")]


register_architecture(
    Architecture(
        name=NAME,
        config_class=ZimoraxConfig,
        build_spec=zimorax_spec,
        hf_architectures=(),
        from_hf_dict=ZimoraxConfig.from_dict,
        to_hf_dict=lambda config: config.as_dict(),
        hf_tensor_layout=checkpoint_tensor_layout,
        detect_source=detect_source,
    )
)


def make_config(width: int, vocab: int, pattern: str, heads: int, kv_heads: int, dim: int, vdim: int, window: int, ff: int, mamba_heads: int,
                mamba_vdim: int, state: int, groups: int, delta_heads: int, delta_kv_heads: int, delta_dim: int, delta_vdim: int, conv: int = 4,
                norm_groups: int = 1, rot_dims: int = 0, rot_base: float = 500000.0, rot_scaling: dict = None, loop: dict = None,
                max_positions: int = 131072) -> ZimoraxConfig:
    """A regular Zimorax: `pattern` has a letter per layer, "m" for mamba2, "d" for delta, "a" for attention; all layers of
    a kind share their sizes."""
    layers = []
    mlp = {"kind": "dense", "ff": ff} if ff else None
    scaling = rot_scaling or {"factor": 4.0, "original": 4096, "fast": 32.0, "slow": 1.0}
    for letter in pattern:
        if letter == "m":
            mixer = {"heads": mamba_heads, "vdim": mamba_vdim, "state": state, "groups": groups, "conv": conv, "norm_groups": norm_groups}
            layers.append({"type": "mamba2", "mixer": mixer, "mlp": mlp})
        elif letter == "d":
            mixer = {"heads": delta_heads, "kv_heads": delta_kv_heads, "dim": delta_dim, "vdim": delta_vdim, "conv": conv}
            layers.append({"type": "delta", "mixer": mixer, "mlp": mlp})
        elif letter == "a":
            mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5, "mask": {"size": window},
                     "rot": {"base": rot_base, "dims": rot_dims or dim, "scaling": dict(scaling)}}
            layers.append({"type": "attention", "mixer": mixer, "mlp": mlp})
        else:
            raise ValueError(f"layer letter {letter!r} is not 'm', 'd' or 'a'")
    return ZimoraxConfig(vocab=vocab, width=width, layers=layers, loop=loop, norm={"eps": 1e-6}, max_positions=max_positions)


def _variant(config: ZimoraxConfig):
    def factory(**overrides) -> ZimoraxConfig:
        return config.updated(**overrides)

    return factory


register_model(NAME, "micro", _variant(make_config(width=256, vocab=1024, pattern="mmdam", heads=4, kv_heads=2, dim=64, vdim=64, window=128, ff=512,
                                                   mamba_heads=8, mamba_vdim=64, state=64, groups=2, delta_heads=4, delta_kv_heads=2, delta_dim=32,
                                                   delta_vdim=64, norm_groups=2, rot_dims=32, loop={"start": 1, "stop": 4, "times": 2},
                                                   max_positions=4096)))
register_model(NAME, "3b", _variant(make_config(width=2048, vocab=65536, pattern="mm" + "mmda" * 5 + "mm", heads=16, kv_heads=4, dim=128, vdim=128,
                                                window=1024, ff=8192, mamba_heads=64, mamba_vdim=64, state=128, groups=8, delta_heads=16,
                                                delta_kv_heads=8, delta_dim=128, delta_vdim=128, norm_groups=8, rot_dims=64,
                                                loop={"start": 2, "stop": 22, "times": 2})))
