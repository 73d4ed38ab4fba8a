"""A linear layer y = x W^T (+ b) with the weight stored [out, in] as checkpoints store it
(fms/modules/linear.py:254-255: the reference's only linear type on this path is nn.Linear)."""

from __future__ import annotations

from typing import List, Optional

import torch

from ..kernels import ops
from .base import Part


class Linear(Part):
    def __init__(self, in_features: int, out_features: int, bias: bool = False):
        super().__init__()
        self.in_features, self.out_features, self.has_bias = in_features, out_features, bias
        self.declare("weight", (out_features, in_features))
        if bias:
            self.declare("bias", (out_features,), init="zeros")

    def forward(self, x: torch.Tensor, out_dtype: Optional[torch.dtype] = None, row_norm=None,
                bias: Optional[torch.Tensor] = None, activation: str = "identity") -> torch.Tensor:
        """bias: a vector to add in the place of the layer's own (a layer without one takes one that changes from call to call)."""
        return ops.linear(x, self.w["weight"], self.w.get("bias") if bias is None else bias, out_dtype=out_dtype, row_norm=row_norm,
                          activation=activation)

    def streams(self, rows: int, dtype: torch.dtype) -> bool:
        """True if a product of this shape runs in the weight-streaming kernel, which can take a deferred
        row norm on its input and add its output into the residual stream."""
        return dtype == torch.bfloat16 and self.w["weight"].dtype == torch.bfloat16 and rows <= ops.SKINNY_FAST_ROWS \
            and self.in_features % 8 == 0


class JointProjection(Linear):
    """Several linear layers with the same outputs as one: W_1 x_1 + W_2 x_2 + ... = [W_1 W_2 ...] [x_1; x_2; ...], with the
    bias of the one that has one.  It is no part of the model's tree: the layers keep their names, and their weights become
    views of the joint one (join, once they are bound)."""

    def __init__(self, layers: List[Linear]):
        super().__init__(sum(l.in_features for l in layers), layers[0].out_features)
        if any(l.out_features != self.out_features for l in layers) or sum(l.has_bias for l in layers) > 1:
            raise NotImplementedError("layers that join have the same outputs, and at most one of them a bias")
        self.layers = list(layers)
        self.has_bias = any(l.has_bias for l in layers)

    def join(self) -> None:
        joint = torch.cat([l.w["weight"] for l in self.layers], dim=1).contiguous()
        self.w["weight"] = joint
        at = 0
        for l in self.layers:
            l.w["weight"] = joint[:, at : at + l.in_features]
            at += l.in_features
            if l.has_bias:
                self.w["bias"] = l.w["bias"]

    def input_rows(self, rows: int, dtype: torch.dtype, device, batch, padding_written: bool) -> torch.Tensor:
        """Rows for the layers' inputs.  A decode step may hold padding rows, which the product reads: zeros, unless
        whoever writes the inputs writes those rows too."""
        x = torch.empty(rows, self.in_features, dtype=dtype, device=device)
        if batch.is_decode and not padding_written:
            x.zero_()
        return x
