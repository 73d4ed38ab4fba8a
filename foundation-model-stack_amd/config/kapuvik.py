"""The Kapuvik configuration: config.json as it is, one entry per layer.

Kapuvik is a decoder whose layers are listed one by one.  Every entry names its mixer (``type``), the mixer's sizes and
constants (``mixer``) and its feed-forward (``mlp``: ``kind`` "dense", ``ff``, ``limit``, or null for none);
``embedding.scale``, ``norm.eps``, ``logit_softcap``, ``vocab`` and ``width`` are the model's own.  The mixers:

* ``parallel``: two mixers side by side, weighted by ``left_scale`` and ``right_scale``: ``left`` is softmax attention with
  grouped heads, rotation of a part of each head (``rot``: ``base``, ``dims``) and capped scores (``softcap``); ``right`` is
  retention, linear attention whose state decays by a constant per head (``decay``, a list), with a rotation of its own;
* ``latent_attention``: attention over a latent (``kv_rank``) and a rotated key part (``rot_dim``) shared by all heads;
* ``gla``: linear attention with a decay per key channel, sigmoid to the power 1 / ``tau``, of a projection through
  ``decay_rank`` numbers (config.json does not carry that size; the checkpoint's tensor shapes give it).

``loop`` (or null for none): the layers ``start`` .. ``stop`` - 1 run ``times`` times in a row with the same weights.
``max_positions`` is this library's bound on a sequence's length (the rotation tables are that long); config.json may carry
it, otherwise the default holds.
"""

from __future__ import annotations

import copy
import dataclasses
from typing import Dict, List, Optional, Tuple

from .base import ModelConfig

MIXERS = ("parallel", "latent_attention", "gla")
MLP_KINDS = ("dense",)
_KEYS = {
    "parallel": ("left", "right", "left_scale", "right_scale"),
    "left": ("heads", "kv_heads", "dim", "vdim", "scale", "rot"),
    "right": ("heads", "dim", "vdim", "decay", "rot"),
    "latent_attention": ("heads", "dim", "rot_dim", "vdim", "kv_rank", "scale", "rot"),
    "gla": ("heads", "dim", "vdim", "tau"),
}


@dataclasses.dataclass
class KapuvikConfig(ModelConfig):
    architecture: str = "Kapuvik"
    vocab: int = 512
    width: int = 128
    embedding: dict = dataclasses.field(default_factory=lambda: {"scale": 1.0})
    layers: List[dict] = dataclasses.field(default_factory=list)
    loop: Optional[dict] = None
    norm: dict = dataclasses.field(default_factory=lambda: {"eps": 1e-6})
    logit_softcap: Optional[float] = None
    max_positions: int = 131072

    def __post_init__(self):
        self.validate()

    @staticmethod
    def _need(where: str, kind: str, m: dict) -> None:
        for key in _KEYS[kind]:
            if key not in m:
                raise ValueError(f"{where} lacks {key!r}")

    @staticmethod
    def _check_rotation(where: str, rot: dict, size: int) -> None:
        if "dims" not in rot or "base" not in rot or rot["dims"] % 2 or not 0 < rot["dims"] <= size:
            raise ValueError(f"{where}: the rotation needs a base and an even number of dimensions within {size}")

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or self.max_positions <= 0:
            raise ValueError("vocab, width and max_positions must be positive")
        if "eps" not in self.norm:
            raise ValueError("the configuration needs norm.eps")
        if self.logit_softcap is not None and self.logit_softcap < 0:
            raise ValueError("logit_softcap must be positive, or null for none")
        for i, layer in enumerate(self.layers):
            kind = layer.get("type")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {kind!r} is not one of {MIXERS}")
            m = layer.get("mixer") or {}
            self._need(f"layer {i}: the mixer", kind, m)
            if kind == "parallel":
                left, right = m["left"], m["right"]
                self._need(f"layer {i}: the left mixer", "left", left)
                self._need(f"layer {i}: the right mixer", "right", right)
                if left["heads"] <= 0 or left["kv_heads"] <= 0 or left["heads"] % left["kv_heads"]:
                    raise ValueError(f"layer {i}: {left['heads']} query heads are no multiple of {left['kv_heads']} key/value heads")
                self._check_rotation(f"layer {i}: the left mixer", left["rot"], left["dim"])
                self._check_rotation(f"layer {i}: the right mixer", right["rot"], right["dim"])
                if len(right["decay"]) != right["heads"]:
                    raise ValueError(f"layer {i}: {right['heads']} heads need as many decays, not {len(right['decay'])}")
            elif kind == "latent_attention":
                self._check_rotation(f"layer {i}: the mixer", dict(m["rot"], dims=m["rot_dim"]), m["rot_dim"])
            elif m["tau"] <= 0:
                raise ValueError(f"layer {i}: tau must be positive")
            mlp = layer.get("mlp")
            if mlp is not None and (mlp.get("kind", "dense") not in MLP_KINDS or mlp.get("ff", 0) <= 0 or mlp.get("limit", 0) <= 0):
                raise ValueError(f"layer {i}: the feed-forward needs a kind of {MLP_KINDS}, a positive ff and a positive limit")
        if self.loop is not None:
            if any(k not in self.loop for k in ("start", "stop", "times")):
                raise ValueError("a loop needs start, stop and times")
            if not 0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers) or self.loop["times"] < 1:
                raise ValueError(f"the loop over layers {self.loop['start']} to {self.loop['stop']} (times {self.loop['times']}) "
                                 f"does not fit {len(self.layers)} layers")

    @property
    def nlayers(self) -> int:
        return len(self.layers)

    def with_sizes_from_tensors(self, shapes: Dict[str, Tuple[int, ...]]) -> "KapuvikConfig":
        """The configuration with the size that only the checkpoint's tensor shapes give: how many numbers the decays of a
        "gla" mixer go through (`l<i>.mix.a1` is [decay_rank, width])."""
        layers = copy.deepcopy(self.layers)
        for i, layer in enumerate(layers):
            shape = shapes.get(f"l{i}.mix.a1")
            if layer.get("type") == "gla" and shape is not None:
                layer["mixer"]["decay_rank"] = int(shape[0])
        return self.updated(layers=layers)
