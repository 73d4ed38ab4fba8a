"""Feed-forward parts.

``GatedLinearUnit`` is the reference's SwiGLU (fms/modules/feedforward.py:193-327):
one fused projection whose first half is the gate and second half the "up" path
(:288-297), out = w2(act(gate) * up).
"""

from __future__ import annotations

from typing import List, Optional

import torch

from ..kernels import ops
from .base import BranchOutput, FeedForward, register_part, split_normed
from .linear import Linear


class GatedLinearUnit(FeedForward):
    def __init__(self, width: int, hidden_dim: int, activation: str = "swish", use_bias: bool = False,
                 limit: Optional[float] = None, alpha: float = 1.0, shift: float = 0.0):
        """limit: the clamped unit instead of act(gate) * up: g sigmoid(alpha g) (u + shift) with g = min(gate, limit) and
        u = clamp(up, -limit, limit)."""
        super().__init__()
        activation = str(activation).lower()  # the reference looks names up without regard to case
        if activation not in ops.ACTIVATIONS:
            raise ValueError(f"activation {activation!r} is not one of {sorted(ops.ACTIVATIONS)}")
        self.width, self.hidden_dim, self.activation = width, int(hidden_dim), activation
        if limit is not None and limit <= 0:
            raise ValueError(f"a limit of {limit} must be positive")
        self.clamp = ops.GateClamp(float(limit), float(alpha), float(shift)) if limit is not None else None
        self.wg1 = self.add_child("wg1_fused", Linear(width, 2 * self.hidden_dim, use_bias))
        self.w2 = self.add_child("w2", Linear(self.hidden_dim, width, use_bias))

    def unfused_parameters(self) -> dict:
        """fms/modules/feedforward.py:312-327: the gate rows come first, then the "up" rows."""
        return {"wg1_fused": (("wg", self.hidden_dim), ("w1", self.hidden_dim))}

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        return self.forward_branch(x).value()

    def accepts_normed_rows(self, rows: int, dtype) -> bool:
        return self.wg1.streams(rows, dtype)

    def output_projections(self) -> List[Linear]:
        return [self.w2]

    def forward_branch(self, x, out: Optional[torch.Tensor] = None) -> BranchOutput:
        """out (rows of any stride): where the input of the last projection is written, for a caller that runs that itself."""
        x, row_norm = split_normed(x)
        hidden = ops.gated_linear(x, self.wg1.w["weight"], self.wg1.w.get("bias"), self.activation, row_norm=row_norm, clamp=self.clamp, out=out)
        return BranchOutput(hidden, self.w2)


register_part("feed_forward", "glu", GatedLinearUnit)
