"""Linear attention with a decay: a recurrent mixer whose memory is one matrix per head instead of a cache of keys and
values, with neither a softmax nor a denominator.

With q, k (`dim` channels a head) and v (`vdim`) plain projections of the mixer's input h,

    S <- diag(a) S + k v^T,   o = S^T (dim^-1/2 q)

The decay a is a constant per head (`decay`, retention; q and k may be rotated by the token's position), or a factor per head
and key channel, a = sigmoid(W_2 W_1 h + b)^(1 / tau) through `decay_rank` numbers (gated linear attention).  Every head's o
is divided by its root mean square, times a weight shared by the heads if there is one, times silu(W_g h), and projected
back to the model's width.

What a sequence carries from token to token is S (float32), fixed-size state of its slot.  Decode steps and short portions
walk the recurrence; longer ones run it in chunks of 64 tokens as matrix products (float32), which starts from and leaves
the same state and differs by rounding only.  Everything behind the projections is float32.
"""

from __future__ import annotations

import math
from typing import List, Optional

import torch

from ..cache import StateNeed
from ..kernels import ops
from .base import BranchOutput, Mixer, register_part, split_normed
from .gated_delta import prefixed_state
from .linear import Linear
from .position import PositionEncoding


class LinearRecurrence(Mixer):
    writes_padding_rows = True

    def __init__(
        self,
        width: int,
        heads: int,
        dim: int,
        vdim: int,
        eps: float = 1e-6,
        decay: Optional[List[float]] = None,  # a constant per head ...
        decay_rank: int = 0,  # ... or a factor per head and key channel, through so many numbers
        tau: float = 1.0,
        norm_weight: bool = True,
        gate_activation: str = "silu",
        position_encoder: Optional[PositionEncoding] = None,  # rotates queries and keys
    ):
        super().__init__()
        if heads <= 0 or vdim <= 0 or not 0 < dim <= ops.LINEAR_MAX_DIM:
            raise ValueError(f"{heads} heads of {dim} key channels (1 to {ops.LINEAR_MAX_DIM}) and {vdim} value channels")
        if (decay is None) == (decay_rank <= 0):
            raise ValueError("the decay is either a constant per head or a projection through decay_rank numbers")
        if decay is not None and (len(decay) != heads or any(not 0 < d <= 1 for d in decay)):
            raise ValueError(f"{heads} heads need as many decays, each above zero and at most one")
        if tau <= 0:
            raise ValueError(f"tau {tau} must be positive")
        if gate_activation not in ops.ACTIVATIONS:
            raise ValueError(f"gate activation {gate_activation!r} is not one of {sorted(ops.ACTIVATIONS)}")
        self.width, self.heads, self.dim, self.vdim, self.eps = width, int(heads), int(dim), int(vdim), float(eps)
        self.decay = [float(d) for d in decay] if decay is not None else None
        self.decay_rank, self.tau, self.gate_activation = int(decay_rank), float(tau), gate_activation
        self.position_encoder = position_encoder
        # one product for everything that reads the mixer's input: [q | k | v | gate | the decay's low rank]
        HD, HV = self.heads * self.dim, self.heads * self.vdim
        self.cols = (0, HD, 2 * HD, 2 * HD + HV, 2 * HD + 2 * HV)
        self.in_proj = self.add_child("in_proj", Linear(width, self.cols[4] + self.decay_rank))
        if self.decay_rank:
            self.declare("decay_up.weight", (HD, self.decay_rank))
            self.declare("decay_up.bias", (HD,), init="zeros", kind="scale")
        self.has_norm_weight = bool(norm_weight)
        if norm_weight:
            self.declare("norm.weight", (self.vdim,), init="ones", kind="scale")
        self.out = self.add_child("out", Linear(HV, width))
        self._log_decay = self._up_t = self._up_bias = self._norm = None

    def unfused_parameters(self) -> dict:
        HD, HV = self.heads * self.dim, self.heads * self.vdim
        pieces = (("q", HD), ("k", HD), ("v", HV), ("g", HV))
        return {"in_proj": pieces + ((("a1", self.decay_rank),) if self.decay_rank else ())}

    def state_need(self) -> StateNeed:
        return StateNeed((("S", (self.heads, self.vdim, self.dim), "float32"),))  # transposed: a value channel's key channels lie together

    @property
    def graph_safe(self) -> bool:
        return getattr(self.position_encoder, "graph_safe", True)

    def check_step(self, max_position: int) -> None:
        if self.position_encoder is not None:
            self.position_encoder.check_positions(max_position)

    def output_projection(self) -> Linear:
        return self.out

    def finalize(self, device, dtype) -> None:
        """What the kernels read in float32: the heads' log decays, or the projection of the decays, transposed."""
        if self.decay is not None:
            self._log_decay = torch.tensor([math.log(d) for d in self.decay], dtype=torch.float32, device=device)
        else:
            self._up_t = self.w["decay_up.weight"].to(torch.float32).t().contiguous()
            self._up_bias = self.w["decay_up.bias"].to(torch.float32).contiguous()
        if self.has_norm_weight:
            self._norm = self.w["norm.weight"].to(torch.float32).contiguous()

    def accepts_normed_rows(self, rows: int, dtype, batch) -> bool:
        return self.in_proj.streams(rows, dtype)

    def forward(self, x: torch.Tensor, batch, cache) -> torch.Tensor:
        return self.forward_branch(x, batch, cache).value()

    def forward_branch(self, x, batch, cache, out: Optional[torch.Tensor] = None, out_scale: float = 1.0) -> BranchOutput:
        """out (rows [T, heads*vdim] of any stride) and out_scale: where the input of the output projection is written, and
        a factor on it, for a caller that runs this mixer beside another and projects both at once."""
        x, row_norm = split_normed(x)
        state = prefixed_state(cache.state, getattr(self, "state_prefix", ""))
        # decays, gate and recurrence are formed from the float32 sums of this product
        proj = self.in_proj.forward(x, out_dtype=torch.float32, row_norm=row_norm)
        rotation = self.position_encoder.tables_for_step(batch) if self.position_encoder is not None else None
        mixed = ops.linear_recurrence(
            proj, self.cols, self.heads, self.dim, self.vdim, state["S"], batch.seq_starts, batch.seq_of_token, batch.slot_ids, batch.n_seqs,
            1 if batch.is_decode else max(batch.q_lens), x.dtype, log_decay=self._log_decay, up_t=self._up_t, up_bias=self._up_bias,
            inv_tau=1.0 / self.tau, rotation=rotation, positions=batch.positions, q_scale=self.dim ** -0.5, norm_weight=self._norm,
            eps=self.eps, activation=self.gate_activation, scale=out_scale, out=out)
        return BranchOutput(mixed, self.out)


register_part("mixer", "linear_recurrence", LinearRecurrence)
