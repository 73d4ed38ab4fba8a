"""The state-space recurrence of Mamba-2: a recurrent mixer whose memory is one matrix per head.

One projection of the mixer's input gives [z | x | B | C | dt]: a gate z and inputs x of heads * vdim channels, `groups`
rows B and C of `state` channels, and a step size per head.  x, B and C together pass a short causal convolution over
time on every channel (with a bias) and silu.  With dt <- softplus(dt + dt_bias) and head h in group h // (heads / groups),

    S <- exp(-exp(A_log) dt) S + dt x B^T;   y = S C + D x        (S: vdim x state, from zero)

and the mixer's output is W_o applied to y * silu(z), divided by its root mean square in `norm_groups` equal parts, times
a weight (the gate comes before the norm).

What a sequence carries from token to token is S (float32) and the last `conv - 1` inputs of the convolution; both are
fixed-size state of its slot.  Steps of single tokens walk the recurrence; longer ones run it in chunks of 64 tokens as
matrix products (float32), which starts from and leaves the same state and differs by rounding only.
"""

from __future__ import annotations

import torch

from ..cache import StateNeed
from ..kernels import ops
from .base import BranchOutput, Mixer, register_part
from .linear import Linear


class Mamba2(Mixer):
    def __init__(self, width: int, heads: int, vdim: int, state: int, groups: int = 1, conv: int = 4, norm_groups: int = 1, eps: float = 1e-6,
                 position_encoder=None):  # takes no positions: the recurrence knows the order of its tokens
        super().__init__()
        if heads <= 0 or groups <= 0 or heads % groups:
            raise ValueError(f"{heads} heads are no multiple of {groups} groups")
        if vdim <= 0 or not 0 < state <= ops.SSD_MAX_STATE:
            raise ValueError(f"{vdim} value channels and {state} state rows (1 to {ops.SSD_MAX_STATE})")
        if not 1 <= conv <= ops.CONV_MAX_TAPS:
            raise ValueError(f"a convolution of {conv} taps (1 to {ops.CONV_MAX_TAPS})")
        self.width, self.heads, self.vdim, self.state, self.groups = width, int(heads), int(vdim), int(state), int(groups)
        self.taps, self.norm_groups, self.eps = int(conv), int(norm_groups), float(eps)
        self.inner = self.heads * self.vdim
        if self.norm_groups <= 0 or self.inner % self.norm_groups:
            raise ValueError(f"{norm_groups} norm groups do not divide {self.inner} channels")
        self.channels = self.inner + 2 * self.groups * self.state  # what passes the convolution: x | B | C
        self.col_x = self.inner
        self.col_dt = self.inner + self.channels
        self.in_proj = self.add_child("in_proj", Linear(width, self.col_dt + self.heads))
        self.declare("conv.weight", (self.channels, self.taps))
        self.declare("conv.bias", (self.channels,), init="zeros")
        self.declare("A_log", (self.heads,), init="zeros", kind="scale")
        self.declare("dt_bias", (self.heads,), init="zeros", kind="scale")
        self.declare("D", (self.heads,), init="ones", kind="scale")
        self.declare("norm.weight", (self.inner,), init="ones", kind="scale")
        self.out = self.add_child("out", Linear(self.inner, width))
        self._a_log = self._dt_bias = self._skip = None

    def unfused_parameters(self) -> dict:
        GN = self.groups * self.state
        return {"in_proj": (("z", self.inner), ("x", self.inner), ("B", GN), ("C", GN), ("dt", self.heads))}

    def state_need(self) -> StateNeed:
        tensors = [("S", (self.heads, self.vdim, self.state), "float32")]
        if self.taps > 1:
            tensors.append(("conv", (self.taps - 1, self.channels), "float32"))
        return StateNeed(tuple(tensors))

    def output_projection(self) -> Linear:
        return self.out

    def finalize(self, device, dtype) -> None:
        self._a_log = self.w["A_log"].to(torch.float32).contiguous()
        self._dt_bias = self.w["dt_bias"].to(torch.float32).contiguous()
        self._skip = self.w["D"].to(torch.float32).contiguous()

    def forward(self, x: torch.Tensor, batch, cache) -> torch.Tensor:
        return self.forward_branch(x, batch, cache).value()

    def forward_branch(self, x: torch.Tensor, batch, cache) -> BranchOutput:
        state = cache.state
        # step sizes, decays, the gate and the recurrence are formed from the float32 sums of this product
        proj = self.in_proj.forward(x, out_dtype=torch.float32)
        z = proj[:, : self.inner]
        if batch.is_decode:
            # the convolution and the recurrence as one kernel; the convolution's state moves on beside the norm
            y = ops.ssd_step(proj, self.col_x, self.col_dt, self.w["conv.weight"], self.w["conv.bias"], state.get("conv"), self._a_log,
                             self._dt_bias, self._skip, state["S"], batch.seq_starts, batch.seq_of_token, batch.slot_ids, batch.n_seqs,
                             self.heads, self.vdim, self.groups, self.state)
            move = dict(conv_x=proj[:, self.col_x : self.col_dt], taps=self.taps, conv_state=state["conv"], slot_ids=batch.slot_ids) if self.taps > 1 else {}
            return BranchOutput(ops.gated_group_norm(y, z, self.w["norm.weight"], self.norm_groups, self.eps, x.dtype, batch.seq_of_token, **move),
                                self.out)
        xbc = ops.short_conv(proj, self.col_x, self.channels, self.w["conv.weight"], self.w["conv.bias"], state.get("conv"), batch.seq_of_token,
                             batch.slot_ids, torch.float32, activation="silu", seq_starts=batch.seq_starts, n_seqs=batch.n_seqs)
        y = ops.ssd(xbc, proj[:, self.col_dt :], self._a_log, self._dt_bias, self._skip, state["S"], batch.seq_starts, batch.seq_of_token,
                    batch.slot_ids, batch.n_seqs, self.heads, self.vdim, self.groups, self.state, longest=max(batch.q_lens))
        normed = ops.gated_group_norm(y, z, self.w["norm.weight"], self.norm_groups, self.eps, x.dtype, batch.seq_of_token)
        return BranchOutput(normed, self.out)


register_part("mixer", "mamba2", Mamba2)
