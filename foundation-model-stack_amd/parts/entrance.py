"""What replaces the residual stream before a pass through looped layers.

``AddEmbedding``: x <- x + x0 (from the second pass on) + step_t, in float32.
``ConcatLinear``: x <- W_in [x; x0] + step_t, x0 the embedding's output and step_t a learned vector for every pass.  The
product reads both in the activation type and leaves the new stream from its float32 sums.
"""

from __future__ import annotations

import torch

from ..kernels import ops
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


START = "entrance.start"  # the embedding's output of the step, float32 [T, width]


class AddEmbedding(Entrance):
    """The embedding's output x0 joins the stream again before every pass but the first, and a learned vector before each."""

    def __init__(self, width: int, passes: int, at_start: bool = False):
        """at_start: no layer runs before the first pass."""
        super().__init__()
        if passes < 1:
            raise ValueError("a loop has at least one pass")
        self.width, self.passes, self.at_start = int(width), int(passes), bool(at_start)
        self.declare("step", (passes, width), kind="scale")
        self._step = None

    def finalize(self, device, dtype) -> None:
        self._step = self.w["step"].to(torch.float32).contiguous()

    def begin(self, stream, batch, act_dtype) -> None:
        batch.shared[START] = stream.resid
        if not self.at_start:  # layers add to the stream in place: the ones before the first pass work on a copy
            stream.replace(ops.stream_enter(stream.resid))

    def enter(self, number: int, stream, batch, act_dtype) -> None:
        stream.advance(base=batch.shared[START] if number > 0 else None, shift=self._step[number])


register_part("entrance", "concat_linear", ConcatLinear)
register_part("entrance", "add_embedding", AddEmbedding)
