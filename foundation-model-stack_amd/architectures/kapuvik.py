"""Kapuvik: from its configuration to parts, and from its checkpoint's tensor names to the model's.

The model: a scaled token embedding; layers in the order config.json lists them, some of them run several times in a row
with the same weights; each a block with one RMS norm (scale stored around zero) whose mixer and feed-forward read the same
normed rows; three kinds of mixers (see config/kapuvik.py); a clamped gated feed-forward with biases, or none; a final norm,
a head of its own and capped logits.  Every pass through the looped layers owns a cache and states of its own (a schedule
entry each); before a pass the embedding's output (but for the first) and a learned vector are added to the stream.

A checkpoint names a layer's tensors ``l<i>.<part>`` without a ".weight" and a bias ``<tensor>.b``; the adapter gives them
the model's names and fuses what the model runs as one product (everything that reads a mixer's input; gate and up).
Retention pairs rotated entry i of a head with entry i + dims/2; the rotation kernels turn neighbouring pairs, so the
adapter moves the rows of its queries and keys alike (their products and the state's are sums over entries and do not care
about the order).  The attentions pair neighbours already.
"""

from __future__ import annotations

import re
from typing import List, Tuple

import torch

from ..config import KapuvikConfig
from ..parts import LayerSpec, ModelSpec, PartSpec, ScheduleEntry
from ..weights.adapters import pairs_to_neighbours, register_adapter, register_adapter_step
from .registry import Architecture, register_architecture, register_model

NAME = "kapuvik"
# what the design fixes
GATE_ALPHA = 1.702  # the feed-forward's unit: g sigmoid(alpha g) (u + shift)
GATE_SHIFT = 1.0
NORM_WEIGHT_OFFSET = 1.0  # the norms of the stream store their scale minus one
LOOP = "loop"  # the name of the loop's entry among the model's parts


def _rope(rot: dict, size: int, max_positions: int, positions: dict) -> str:
    """The key of a rotation among the model's position encodings (added if it is not there yet)."""
    key = f"rope_{size}_{rot['dims']}_{rot['base']!r}"
    positions.setdefault(key, PartSpec("rope", {"dim": size, "rot_dim": rot["dims"], "theta": rot["base"], "max_seq_len": max_positions,
                                                "exact_frequencies": True}))
    return key


def run_order(config: KapuvikConfig) -> List[ScheduleEntry]:
    """The layers in the order in which they run; an entry that starts a pass through the loop names what comes before it."""
    loop, n = config.loop, len(config.layers)
    if loop is None:
        return [ScheduleEntry(i) for i in range(n)]
    out = [ScheduleEntry(i) for i in range(loop["start"])]
    for t in range(loop["times"]):
        for i in range(loop["start"], loop["stop"]):
            out.append(ScheduleEntry(i, enter=(LOOP, t) if i == loop["start"] else None))
    return out + [ScheduleEntry(i) for i in range(loop["stop"], n)]


def kapuvik_spec(config: KapuvikConfig) -> ModelSpec:
    eps = config.norm["eps"]
    norm = PartSpec("rmsnorm", {"eps": eps, "weight_offset": NORM_WEIGHT_OFFSET})
    layers, positions = [], {}
    for i, layer in enumerate(config.layers):
        m, kind, key = layer["mixer"], layer["type"], None
        if kind == "parallel":
            left, right = m["left"], m["right"]
            key = {"left": _rope(left["rot"], left["dim"], config.max_positions, positions),
                   "right": _rope(right["rot"], right["dim"], config.max_positions, positions)}
            mixer = PartSpec("parallel", {
                "left": {"kind": "attention", "args": {
                    "nheads": left["heads"], "kvheads": left["kv_heads"], "head_dim": left["dim"], "value_dim": left["vdim"],
                    "scale_factor": left["scale"], "soft_cap": left.get("softcap") or 0.0}},
                "right": {"kind": "linear_recurrence", "args": {
                    "heads": right["heads"], "dim": right["dim"], "vdim": right["vdim"], "eps": eps, "decay": right["decay"], "norm_weight": False}},
                "left_scale": m["left_scale"], "right_scale": m["right_scale"],
            })
        elif kind == "latent_attention":
            key = _rope(dict(m["rot"], dims=m["rot_dim"]), m["rot_dim"], config.max_positions, positions)
            mixer = PartSpec("latent_attention", {"nheads": m["heads"], "dim": m["dim"], "rot_dim": m["rot_dim"], "vdim": m["vdim"], "q_rank": 0,
                                                  "kv_rank": m["kv_rank"], "scale": m["scale"], "eps": eps})
        else:
            if not m.get("decay_rank"):
                raise ValueError(f"layer {i}: a gla mixer needs 'decay_rank': a model folder's tensor shapes give it, a configuration made "
                                 "without one must carry it")
            mixer = PartSpec("linear_recurrence", {"heads": m["heads"], "dim": m["dim"], "vdim": m["vdim"], "eps": eps,
                                                   "decay_rank": m["decay_rank"], "tau": m["tau"]})
        mlp = layer.get("mlp")
        ff = None
        if mlp is not None:
            ff = PartSpec("glu", {"hidden_dim": mlp["ff"], "use_bias": True, "limit": mlp["limit"], "alpha": GATE_ALPHA, "shift": GATE_SHIFT})
        layers.append(LayerSpec(mixer=mixer, feed_forward=ff, norm=norm, block=PartSpec("parallel", {"names": ("norm1", "mix", "mlp")}), position=key))
    loops = {}
    if config.loop is not None:
        loops[LOOP] = PartSpec("add_embedding", {"passes": config.loop["times"], "at_start": config.loop["start"] == 0})
    return ModelSpec(
        vocab=config.vocab, width=config.width, max_seq_len=config.max_positions, layers=layers, final_norm=norm, positions=positions,
        embedding=PartSpec("table", {"scale": config.embedding.get("scale", 1.0)}),
        head=PartSpec("linear", {"soft_cap": config.logit_softcap or 0.0}), schedule=run_order(config), entrances=loops,
        embedding_name="embed", layer_name="l{i}", final_norm_name="final.norm", head_name="head",
    )


# ---- the checkpoint's names -> the model's ----------------------------------------------------------------------
def _fuse_parallel(out: dict, p: str, m: dict) -> None:
    left, right = p + "left.", p + "right."
    out[left + "in_proj.qkv_fused.weight"] = torch.cat([out.pop(left + n) for n in ("q", "k", "v")], dim=0)
    out[left + "dense.weight"] = out.pop(left + "o")
    rows = [pairs_to_neighbours(out.pop(right + n), m["right"]["heads"], 0, m["right"]["rot"]["dims"]) for n in ("q", "k")]
    out[right + "in_proj.weight"] = torch.cat(rows + [out.pop(right + n) for n in ("v", "g")], dim=0)
    out[right + "out.weight"] = out.pop(right + "o")


def _fuse_latent(out: dict, p: str) -> None:
    out[p + "down.weight"] = torch.cat([out.pop(p + "q"), out.pop(p + "dkv")], dim=0)
    for src, dst in (("dkv.norm", "kv_norm.weight"), ("uk", "uk.weight"), ("uv", "uv.weight"), ("o", "o.weight")):
        out[p + dst] = out.pop(p + src)


def _fuse_gla(out: dict, p: str) -> None:
    out[p + "in_proj.weight"] = torch.cat([out.pop(p + n) for n in ("q", "k", "v", "g", "a1")], dim=0)
    for src, dst in (("a2", "decay_up.weight"), ("a2.b", "decay_up.bias"), ("norm", "norm.weight"), ("o", "out.weight")):
        out[p + dst] = out.pop(p + src)


def _to_model_names(sd, model_config=None, **kw):
    out = dict(sd)
    for name in [n for n in out if n.endswith(".norm1")]:
        p = name[: -len("norm1")]
        layer = model_config.layers[int(p[1:-1])]
        q = p + "mix."
        if layer["type"] == "parallel":
            _fuse_parallel(out, q, layer["mixer"])
        elif layer["type"] == "latent_attention":
            _fuse_latent(out, q)
        else:
            _fuse_gla(out, q)
        if layer.get("mlp") is not None:
            f = p + "mlp."
            out[f + "wg1_fused.weight"] = torch.cat([out.pop(f + "gate"), out.pop(f + "up")], dim=0)
            out[f + "wg1_fused.bias"] = torch.cat([out.pop(f + "gate.b"), out.pop(f + "up.b")], dim=0)
            out[f + "w2.weight"], out[f + "w2.bias"] = out.pop(f + "down"), out.pop(f + "down.b")
    renamed = {}
    for name, t in out.items():
        if re.search(r"(^embed|^head|^final\.norm|\.norm1)$", name):
            name += ".weight"
        renamed[name] = t
    return renamed


register_adapter_step(NAME, "checkpoint_to_model_names", _to_model_names)
register_adapter(NAME, "hf", ["checkpoint_to_model_names"])


def detect_source(names: List[str]) -> str:
    return "fms" if any(n.endswith(".weight") for n in names) else "hf"


def checkpoint_tensor_layout(config: KapuvikConfig) -> List[Tuple[str, Tuple[int, ...], str]]:
    """(name, shape, init) of every tensor of a Kapuvik checkpoint of this configuration."""
    W = config.width
    out = [("embed", (config.vocab, W), "normal")]
    if config.loop is not None:
        out.append(("loop.step", (config.loop["times"], W), "normal"))
    for i, layer in enumerate(config.layers):
        p, m, kind = f"l{i}.", layer["mixer"], layer["type"]
        q = p + "mix."
        out.append((p + "norm1", (W,), "zeros"))
        if kind == "parallel":
            a, b = m["left"], m["right"]
            out += [(q + "left.q", (a["heads"] * a["dim"], W), "normal"), (q + "left.k", (a["kv_heads"] * a["dim"], W), "normal"),
                    (q + "left.v", (a["kv_heads"] * a["vdim"], W), "normal"), (q + "left.o", (W, a["heads"] * a["vdim"]), "normal")]
            HD, HV = b["heads"] * b["dim"], b["heads"] * b["vdim"]
            out += [(q + "right." + n, (rows, W), "normal") for n, rows in (("q", HD), ("k", HD), ("v", HV), ("g", HV))]
            out.append((q + "right.o", (W, HV), "normal"))
        elif kind == "latent_attention":
            H, D, P, V, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            out += [(q + "q", (H * (D + P), W), "normal"), (q + "dkv", (R + P, W), "normal"), (q + "dkv.norm", (R,), "ones"),
                    (q + "uk", (H * D, R), "normal"), (q + "uv", (H * V, R), "normal"), (q + "o", (W, H * V), "normal")]
        else:
            HD, HV, r = m["heads"] * m["dim"], m["heads"] * m["vdim"], m["decay_rank"]
            out += [(q + n, (rows, W), "normal") for n, rows in (("q", HD), ("k", HD), ("v", HV), ("g", HV))]
            out += [(q + "o", (W, HV), "normal"), (q + "norm", (m["vdim"],), "ones"), (q + "a1", (r, W), "normal"),
                    (q + "a2", (HD, r), "normal"), (q + "a2.b", (HD,), "zeros")]
        mlp = layer.get("mlp")
        if mlp is not None:
            F = mlp["ff"]
            out += [(p + "mlp.gate", (F, W), "normal"), (p + "mlp.gate.b", (F,), "zeros"), (p + "mlp.up", (F, W), "normal"),
                    (p + "mlp.up.b", (F,), "zeros"), (p + "mlp.down", (W, F), "normal"), (p + "mlp.down.b", (W,), "zeros")]
    return out + [("final.norm", (W,), "zeros"), ("head", (config.vocab, W), "normal")]


register_architecture(
    Architecture(
        name=NAME,
        config_class=KapuvikConfig,
        build_spec=kapuvik_spec,
        hf_architectures=(),
        from_hf_dict=KapuvikConfig.from_dict,
        to_hf_dict=lambda config: config.as_dict(),
        hf_tensor_layout=checkpoint_tensor_layout,
        detect_source=detect_source,
        sizes_from_tensors=lambda config, shapes: config.with_sizes_from_tensors(shapes),
    )
)


def make_config(width: int, vocab: int, pattern: str, heads: int, kv_heads: int, dim: int, vdim: int, ff: int, latent_heads: int, latent_dim: int,
                rot_dim: int, latent_vdim: int, kv_rank: int, ret_heads: int, ret_dim: int, ret_vdim: int, gla_heads: int, gla_dim: int,
                gla_vdim: int, decay_rank: int = 16, tau: float = 16.0, softcap: float = 30.0, rot_base: float = 500000.0, limit: float = 7.0,
                left_scale: float = 1.0, right_scale: float = 1.0, embedding_scale: float = 1.0, logit_softcap: float = 30.0, loop: dict = None,
                max_positions: int = 131072) -> KapuvikConfig:
    """A regular Kapuvik: `pattern` has a letter per layer, "p" for a parallel mixer, "l" for latent attention, "g" for gated
    linear attention; all layers of a kind share their sizes."""
    layers = []
    mlp = {"kind": "dense", "ff": ff, "limit": limit} if ff else None
    for letter in pattern:
        if letter == "p":
            mixer = {"left": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5, "softcap": softcap,
                              "rot": {"base": rot_base, "dims": dim}},
                     "right": {"heads": ret_heads, "dim": ret_dim, "vdim": ret_vdim, "decay": [1 - 2.0 ** (-5 - h * 7 / max(ret_heads, 1)) for h in range(ret_heads)],
                               "rot": {"base": rot_base, "dims": ret_dim}},
                     "left_scale": left_scale, "right_scale": right_scale}
            layers.append({"type": "parallel", "mixer": mixer, "mlp": mlp})
        elif letter == "l":
            mixer = {"heads": latent_heads, "dim": latent_dim, "rot_dim": rot_dim, "vdim": latent_vdim, "kv_rank": kv_rank,
                     "scale": (latent_dim + rot_dim) ** -0.5, "rot": {"base": rot_base, "dims": rot_dim}}
            layers.append({"type": "latent_attention", "mixer": mixer, "mlp": mlp})
        elif letter == "g":
            layers.append({"type": "gla", "mixer": {"heads": gla_heads, "dim": gla_dim, "vdim": gla_vdim, "tau": tau, "decay_rank": decay_rank}, "mlp": mlp})
        else:
            raise ValueError(f"layer letter {letter!r} is not 'p', 'l' or 'g'")
    return KapuvikConfig(vocab=vocab, width=width, embedding={"scale": embedding_scale}, layers=layers, loop=loop, norm={"eps": 1e-6},
                         logit_softcap=logit_softcap, max_positions=max_positions)


def _variant(config: KapuvikConfig):
    def factory(**overrides) -> KapuvikConfig:
        return config.updated(**overrides)

    return factory


register_model(NAME, "micro", _variant(make_config(width=256, vocab=1024, pattern="pglgg", heads=4, kv_heads=2, dim=64, vdim=64, ff=512,
                                                   latent_heads=4, latent_dim=32, rot_dim=32, latent_vdim=64, kv_rank=96, ret_heads=4, ret_dim=32,
                                                   ret_vdim=64, gla_heads=4, gla_dim=32, gla_vdim=48, loop={"start": 1, "stop": 4, "times": 2},
                                                   max_positions=4096)))
register_model(NAME, "3b", _variant(make_config(width=2048, vocab=65536, pattern="gg" + "pglg" * 5 + "gg", heads=16, kv_heads=4, dim=128, vdim=128,
                                                ff=5632, latent_heads=16, latent_dim=128, rot_dim=64, latent_vdim=128, kv_rank=512, ret_heads=16,
                                                ret_dim=64, ret_vdim=128, gla_heads=16, gla_dim=64, gla_vdim=128, loop={"start": 2, "stop": 22, "times": 2})))
