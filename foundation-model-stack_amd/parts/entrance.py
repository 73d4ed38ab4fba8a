"""What replaces the residual stream before a pass through looped layers.

``ConcatLinear``: x <- W_in [x; x0] + step_t, x0 the embedding's output and step_t a learned vector for every pass.  The
product reads both in the activation type and leaves the new stream from its float32 sums.
"""

from __future__ import annotations

import torch

from .base import Entrance, register_part
from .linear import Linear

ROWS = "entrance.rows"  # [T, 2 width] of the step: what the product reads; its right half holds the embedding's output


class ConcatLinear(Entrance):
    def __init__(self, width: int, passes: int):
        super().__init__()
        if passes < 1:
            raise ValueError("a loop has at least one pass")
        self.width, self.passes = int(width), int(passes)
        self.proj = self.add_child("in", Linear(2 * width, width))
        self.declare("step", (passes, width), kind="scale")

    def begin(self, stream, batch, act_dtype) -> None:
        rows = torch.empty(stream.resid.shape[0], 2 * self.width, dtype=act_dtype, device=stream.resid.device)
        stream.rows_into(rows[:, self.width :])
        batch.shared[ROWS] = rows

    def enter(self, number: int, stream, batch, act_dtype) -> None:
        rows = batch.shared[ROWS]
        stream.rows_into(rows[:, : self.width])
        stream.replace(self.proj.forward(rows, out_dtype=torch.float32, bias=self.w["step"][number]))


register_part("entrance", "concat_linear", ConcatLinear)
