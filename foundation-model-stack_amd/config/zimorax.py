"""The Zimorax configuration: config.json as it is, one entry per layer.

Zimorax is a decoder whose layers are listed one by one.  Every entry names its mixer (``type``), the mixer's sizes and
constants (``mixer``) and its feed-forward (``mlp``: ``kind`` "dense", or null for none); ``norm.eps``, ``vocab`` and
``width`` are the model's own.  The mixers:

* ``attention``: grouped heads whose scores are mixed over the heads before the softmax, rotation of a part of each head
  (``rot``: ``base``, ``dims``, and ``scaling`` with ``factor``, ``original``, ``fast``, ``slow``), normed values, a sliding
  window (``mask.size``), a sink of score zero;
* ``mamba2``: a state-space recurrence over a matrix per head (``state`` rows, ``vdim`` columns) behind a short convolution;
* ``delta``: the gated delta rule with a decay per head.

``loop`` (or null for none): the layers ``start`` .. ``stop`` - 1 run ``times`` times in a row with the same weights, each
pass entered through a projection of the stream and the embedding together.  ``max_positions`` is this library's bound on
a sequence's length (the rotation tables are that long); config.json may carry it, otherwise the default holds.
"""

from __future__ import annotations

import dataclasses
from typing import List, Optional

from .base import ModelConfig

MIXERS = ("attention", "mamba2", "delta")
MLP_KINDS = ("dense",)
_KEYS = {
    "attention": ("heads", "kv_heads", "dim", "vdim", "scale", "rot", "mask"),
    "mamba2": ("heads", "vdim", "state", "groups", "conv", "norm_groups"),
    "delta": ("heads", "kv_heads", "dim", "vdim", "conv"),
}
_SCALING_KEYS = ("factor", "original", "fast", "slow")


@dataclasses.dataclass
class ZimoraxConfig(ModelConfig):
    architecture: str = "Zimorax"
    vocab: int = 512
    width: int = 128
    layers: List[dict] = dataclasses.field(default_factory=list)
    loop: Optional[dict] = None
    norm: dict = dataclasses.field(default_factory=lambda: {"eps": 1e-6})
    max_positions: int = 131072

    def __post_init__(self):
        self.validate()

    def validate(self) -> None:
        if self.vocab <= 0 or self.width <= 0 or self.max_positions <= 0:
            raise ValueError("vocab, width and max_positions must be positive")
        if "eps" not in self.norm:
            raise ValueError("the configuration needs norm.eps")
        for i, layer in enumerate(self.layers):
            kind = layer.get("type")
            if kind not in MIXERS:
                raise ValueError(f"layer {i}: mixer type {kind!r} is not one of {MIXERS}")
            m = layer.get("mixer") or {}
            for key in _KEYS[kind]:
                if key not in m:
                    raise ValueError(f"layer {i}: the mixer lacks {key!r}")
            if kind == "mamba2":
                if m["heads"] <= 0 or m["groups"] <= 0 or m["heads"] % m["groups"]:
                    raise ValueError(f"layer {i}: {m['heads']} heads are no multiple of {m['groups']} groups")
                if m["norm_groups"] <= 0 or (m["heads"] * m["vdim"]) % m["norm_groups"]:
                    raise ValueError(f"layer {i}: {m['norm_groups']} norm groups do not divide {m['heads'] * m['vdim']} channels")
            elif m["heads"] <= 0 or m["kv_heads"] <= 0 or m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: {m['heads']} heads are no multiple of {m['kv_heads']} key/value heads")
            if kind == "attention":
                rot = m["rot"]
                if "dims" not in rot or "base" not in rot or rot["dims"] % 2 or not 0 < rot["dims"] <= m["dim"]:
                    raise ValueError(f"layer {i}: the rotation needs a base and an even number of dimensions within the head's {m['dim']}")
                scaling = rot.get("scaling")
                if scaling is not None and (any(k not in scaling for k in _SCALING_KEYS) or scaling["factor"] <= 0):
                    raise ValueError(f"layer {i}: rot.scaling needs {_SCALING_KEYS} with a positive factor")
                if m["mask"].get("size", 0) <= 0:
                    raise ValueError(f"layer {i}: the window needs a positive mask.size")
            mlp = layer.get("mlp")
            if mlp is not None and (mlp.get("kind") not in MLP_KINDS or mlp.get("ff", 0) <= 0):
                raise ValueError(f"layer {i}: the feed-forward needs a kind of {MLP_KINDS} and a positive ff")
        if self.loop is not None:
            if any(k not in self.loop for k in ("start", "stop", "times")):
                raise ValueError("a loop needs start, stop and times")
            if not 0 <= self.loop["start"] < self.loop["stop"] <= len(self.layers) or self.loop["times"] < 1:
                raise ValueError(f"the loop over layers {self.loop['start']} to {self.loop['stop']} (times {self.loop['times']}) "
                                 f"does not fit {len(self.layers)} layers")

    @property
    def nlayers(self) -> int:
        return len(self.layers)
