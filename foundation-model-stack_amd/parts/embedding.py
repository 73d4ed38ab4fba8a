"""Token embedding and output head.

fms/models/llama.py:185-187, 332: a table row per token, no scale.  The head is a
bias-free linear layer (fms/modules/head.py:89-95) whose logits leave in float32.
"""

from __future__ import annotations

import torch

from ..kernels import ops
from .base import Part, register_part


class TokenEmbedding(Part):
    def __init__(self, vocab: int, width: int, scale: float = 1.0):
        super().__init__()
        self.vocab, self.width, self.scale = vocab, width, float(scale)  # scale: a constant factor on every row
        self.declare("weight", (vocab, width))

    def forward(self, token_ids: torch.Tensor, batch=None) -> torch.Tensor:
        """int32 ids [T] -> the float32 residual stream [T, width].  `batch` is the step (positions, sequence of
        every token): an embedding that adds a learned vector per position reads it, this one does not."""
        return ops.embed(token_ids, self.w["weight"], self.scale)


class LinearHead(Part):
    def __init__(self, width: int, vocab: int, scale: float = 1.0, soft_cap: float = 0.0):
        """scale: a constant factor on every logit.  soft_cap: logits become soft_cap * tanh(logit / soft_cap) (0: no cap)."""
        super().__init__()
        self.vocab, self.width, self.scale, self.soft_cap = vocab, width, float(scale), float(soft_cap)
        if self.soft_cap < 0:
            raise ValueError(f"soft_cap {soft_cap} must be zero (none) or positive")
        self.declare("weight", (vocab, width))

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        logits = ops.linear(x, self.w["weight"], None, out_dtype=torch.float32)
        if self.scale != 1.0:
            logits = ops.scale_(logits, self.scale)
        return ops.soft_cap_(logits, self.soft_cap) if self.soft_cap else logits


register_part("embedding", "table", TokenEmbedding)
register_part("head", "linear", LinearHead)
