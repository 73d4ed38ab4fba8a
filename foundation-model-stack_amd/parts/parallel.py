"""Two mixers side by side: both read the same input, and the layer's mixer output is
left_scale * left(h) + right_scale * right(h).

Each side ends in a projection back to the model's width.  The two projections run as one product over the two sides'
inputs laid next to each other, each already times its scale (the kernel that writes a side's last activation applies
it in float32, before the one rounding), so the weighted sum costs no kernel and no rounding of its own.  The sides keep
what they need of the cache: at most one of them keys and values in pages, and each its fixed-size state, whose tensors
carry the side's name.
"""

from __future__ import annotations

from typing import Optional

import torch

from ..cache import StateNeed
from .base import BranchOutput, Mixer, make_part, register_part, split_normed
from .linear import JointProjection


class ParallelMixers(Mixer):
    def __init__(self, width: int, left: dict, right: dict, left_scale: float = 1.0, right_scale: float = 1.0, position_encoder=None):
        """left, right: {"kind": a registered mixer, "args": its arguments}.  The position encoding goes to the sides that
        say `"positional": True`; with encodings of their own it is a dictionary from a side's name to its encoding."""
        super().__init__()
        self.width = width
        self.scales = (float(left_scale), float(right_scale))
        self.sides = []
        for name, spec in (("left", left), ("right", right)):
            pos = position_encoder.get(name) if isinstance(position_encoder, dict) else (position_encoder if spec.get("positional") else None)
            side = make_part("mixer", spec["kind"], width=width, position_encoder=pos, **spec.get("args", {}))
            if not hasattr(side, "forward_branch"):
                raise TypeError(f"mixer {spec['kind']!r} cannot run beside another: it has no forward_branch")
            side.state_prefix = name + "."
            self.sides.append(self.add_child(name, side))
        if sum(side.kv_need() is not None for side in self.sides) > 1:
            raise ValueError("at most one of two parallel mixers can keep keys and values in the cache")
        outs = self.output_projections()
        if any(o.has_bias for o in outs):
            raise NotImplementedError("parallel mixers join output projections without biases")
        self._joint: Optional[JointProjection] = JointProjection(outs)
        self._widths = [o.in_features for o in outs]

    def kv_need(self):
        for side in self.sides:
            if side.kv_need() is not None:
                return side.kv_need()
        return None

    def state_need(self):
        tensors = []
        for side in self.sides:
            need = side.state_need()
            if need is not None:
                tensors += [(side.state_prefix + name, shape, dt) for name, shape, dt in need.tensors]
        return StateNeed(tuple(tensors)) if tensors else None

    @property
    def graph_safe(self) -> bool:
        return all(getattr(side, "graph_safe", True) for side in self.sides)

    @property
    def writes_padding_rows(self) -> bool:
        return all(side.writes_padding_rows for side in self.sides)

    def check_step(self, max_position: int) -> None:
        for side in self.sides:
            side.check_step(max_position)

    def prefill_qblock(self, n_tokens: int, dtype) -> int:
        return max(side.prefill_qblock(n_tokens, dtype) for side in self.sides)

    def output_projections(self) -> list:
        return [side.output_projection() for side in self.sides]

    def leaves_output_to_caller(self) -> None:
        self._joint = None  # the caller's joint projection holds the sides' weights

    def finalize(self, device, dtype) -> None:
        if self._joint is not None:
            self._joint.join()

    def accepts_normed_rows(self, rows: int, dtype, batch) -> bool:
        return all(side.accepts_normed_rows(rows, dtype, batch) for side in self.sides)

    def forward(self, x: torch.Tensor, batch, cache) -> torch.Tensor:
        return self.forward_branch(x, batch, cache).value()

    def forward_branch(self, x, batch, cache, out: Optional[torch.Tensor] = None) -> BranchOutput:
        """out (rows of any stride): where the inputs of the sides' output projections are written, for a caller that runs
        those itself."""
        if out is None:
            rows = split_normed(x)[0]
            out = self._joint.input_rows(rows.shape[0], rows.dtype, rows.device, batch, self.writes_padding_rows)
        at = 0
        for side, scale, k in zip(self.sides, self.scales, self._widths):
            side.forward_branch(x, batch, cache, out=out[:, at : at + k], out_scale=scale)
            at += k
        return BranchOutput(out, self._joint)


register_part("mixer", "parallel", ParallelMixers)
