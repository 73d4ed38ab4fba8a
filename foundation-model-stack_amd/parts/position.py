"""Position encodings.

``RotaryEncoding`` is the reference's RoPE without complex numbers
(fms/modules/positions.py:269-464): adjacent pairs (x[2i], x[2i+1]) are rotated
by position * f_i, f_i = theta^(-2i/D), all in float32.  The frequencies are
computed with the reference's own expression; the cos/sin table is built once
on the device by a kernel and read by the fused rotate-and-store kernel.

The interface a position encoding offers to a mixer:
  * ``rotary_tables()``: (cos, sin, rotary size) for the fused kernel, or None;
    ``tables_for_step(batch)``: the same for one step, for encodings whose table depends on the step;
  * ``adjust_qk(qkv, batch, ...)``: transform queries and keys in place before
    they are cached, for encodings that are no plain rotation;
  * ``score_slopes(nheads)``: for encodings that act on the scores instead (the reference's
    ``adjusted_mask``, fms/modules/positions.py:9-36): a float32 slope per head, added to every score as
    slope * (key position - query position); None for encodings that leave the scores alone;
  * ``check_positions(max_position)``: raise if a position cannot be encoded.
"""

from __future__ import annotations

import math
from typing import Optional, Tuple

import torch

from ..kernels import ops
from .base import Part, register_part


def ntk_alpha(length: int, original_length: int) -> int:
    """fms/modules/positions.py:146-156: the power of two that stretches `original_length` over `length`."""
    ratio = max(1, -(-int(length) // int(original_length)))
    return 1 << (ratio - 1).bit_length()


def rope_frequencies(dim: int, theta: float, scaling: Optional[dict] = None, alpha: int = 1, exact: bool = False) -> torch.Tensor:
    """Float32 frequencies f_i, i < dim/2.

    regular: fms/modules/positions.py:124-132.  llama3: fms/modules/positions.py:171-196.
    ntk: fms/modules/positions.py:161-168, theta * alpha^(dim / (dim - 2)) for the power of two `alpha`.
    linear: every frequency divided by scaling["factor"].
    yarn: frequency i divided by the factor where its dimension turns fewer than `beta_slow` times over the original
    length, kept where it turns more than `beta_fast` times, and a straight line between the two in i in between.
    """
    scaling = dict(scaling or {})
    kind = scaling.get("rope_type", "regular")
    if kind == "ntk":
        theta = theta * alpha ** (dim / (dim - 2))
    if exact:
        # theta^(-2i/dim) formed in float64 and rounded once at the end (after any scaling), for models that define the
        # frequencies as real numbers
        freqs = torch.tensor([float(theta) ** (-2.0 * i / dim) for i in range(dim // 2)], dtype=torch.float64)
    else:
        freqs = 1.0 / (theta ** (torch.arange(0, dim, 2)[: dim // 2].float() / dim))
    if kind in ("regular", "ntk"):
        return freqs.to(torch.float32)
    if kind == "linear":  # positions counted in steps of 1 / factor: every frequency divided by the factor
        return (freqs / float(scaling["factor"])).to(torch.float32)
    if kind == "yarn":
        def dim_of(turns):  # the (real) index of the dimension pair that turns so many times over the original length
            return dim * math.log(scaling["original_max_position_embeddings"] / (2 * math.pi * turns)) / (2 * math.log(theta))

        lo = max(math.floor(dim_of(scaling["beta_fast"])), 0)
        hi = min(math.ceil(dim_of(scaling["beta_slow"])), dim - 1)
        ramp = ((torch.arange(dim // 2, dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
        return (freqs / float(scaling["factor"]) * ramp + freqs * (1 - ramp)).to(torch.float32)
    if kind == "llama3":
        factor = scaling["factor"]
        low_freq_factor = scaling["low_freq_factor"]
        high_freq_factor = scaling["high_freq_factor"]
        old_len = scaling["original_max_position_embeddings"]
        wavelen = 2 * math.pi / freqs
        scaled = torch.where(wavelen > old_len / low_freq_factor, freqs / factor, freqs)
        smooth = (old_len / wavelen - low_freq_factor) / (high_freq_factor - low_freq_factor)
        smoothed = (1 - smooth) * scaled / factor + smooth * scaled
        medium = ~(wavelen < old_len / high_freq_factor) * ~(wavelen > old_len / low_freq_factor)
        return torch.where(medium, smoothed, scaled).to(torch.float32)
    raise ValueError(f"rope_type {kind!r} is not supported (regular, linear, yarn, llama3, ntk)")


def rope_gain(scaling: Optional[dict]) -> float:
    """The factor on cosines and sines that goes with a scaling: 0.1 ln(factor) + 1 for yarn, else 1."""
    scaling = scaling or {}
    return 0.1 * math.log(scaling["factor"]) + 1.0 if scaling.get("rope_type") == "yarn" else 1.0


class PositionEncoding(Part):
    def rotary_tables(self) -> Optional[Tuple[torch.Tensor, torch.Tensor, int]]:
        return None

    def tables_for_step(self, batch) -> Optional[Tuple[torch.Tensor, torch.Tensor, int]]:
        """The tables for the tokens of one step; the same for every step unless the encoding says otherwise."""
        return self.rotary_tables()

    def adjust_qk(self, qkv: torch.Tensor, batch, nheads: int, kvheads: int, head_dim: int) -> None:
        """In-place transform of the query and key columns of qkv rows; default: none."""

    def score_slopes(self, nheads: int) -> Optional[torch.Tensor]:
        """float32 [nheads] on the device: a bias by distance that attention adds to its scores; default: none."""
        return None

    def check_positions(self, max_position: int) -> None:
        """Raise IndexError when `max_position` cannot be encoded."""


class RotaryEncoding(PositionEncoding):
    """max_seq_len: the length of the table (the reference's max_expected_seq_len).  With "ntk" scaling it is the
    length the frequencies were made for, and sequences may grow to `max_positions`: a step whose longest
    sequence holds n tokens rotates all its tokens with the table of alpha = ntk_alpha(n, max_seq_len), as
    the reference's call does (fms/modules/positions.py:311-355, 407-421: alpha from the call's longest
    sequence; keys cached by earlier calls keep the rotation they got).  Up to max_seq_len tokens alpha is 1 and
    the encoding is the regular one (tests/modules/test_positions.py:216-241)."""

    def __init__(self, dim: int, theta: float = 10_000.0, max_seq_len: int = 2048, scaling: Optional[dict] = None,
                 partial_rope: float = 1.0, max_positions: Optional[int] = None, exact_frequencies: bool = False,
                 rot_dim: Optional[int] = None):
        """rot_dim: the number of rotated dimensions of a head, for a model that gives it as a number (default:
        partial_rope times the head size)."""
        super().__init__()
        self.exact_frequencies = bool(exact_frequencies)
        self.head_dim = dim
        self.rot_dim = int(rot_dim) if rot_dim is not None else int(partial_rope * dim)
        if self.rot_dim % 2 or self.rot_dim <= 0 or self.rot_dim > dim:
            raise ValueError(f"rotary size {self.rot_dim} of head size {dim} must be even and within the head")
        self.theta, self.max_seq_len, self.scaling = float(theta), int(max_seq_len), dict(scaling or {})
        self.stretches = self.scaling.get("rope_type") == "ntk"
        self.max_positions = int(max_positions) if (max_positions and self.stretches) else self.max_seq_len
        if self.stretches and self.rot_dim <= 2:
            raise ValueError("ntk scaling needs a rotary size above 2")
        self.freqs = rope_frequencies(self.rot_dim, self.theta, self.scaling, exact=self.exact_frequencies)
        self.cos: Optional[torch.Tensor] = None
        self.sin: Optional[torch.Tensor] = None
        self.tables = {}  # alpha -> (cos, sin); alpha 1 only unless the encoding stretches

    @property
    def graph_safe(self) -> bool:
        """A captured step keeps the tables it was captured with; a stretching encoding changes them as sequences grow."""
        return self.max_positions <= self.max_seq_len

    def finalize(self, device, dtype) -> None:
        alpha = 1
        while True:
            length = min(self.max_seq_len * alpha, self.max_positions)
            freqs = rope_frequencies(self.rot_dim, self.theta, self.scaling, alpha, exact=self.exact_frequencies)
            self.tables[alpha] = ops.rope_table(freqs.to(device), length, rope_gain(self.scaling))
            if self.max_seq_len * alpha >= self.max_positions:
                break
            alpha *= 2
        self.cos, self.sin = self.tables[1]

    def rotary_tables(self):
        return self.cos, self.sin, self.rot_dim

    def tables_for_step(self, batch):
        if not self.stretches:
            return self.cos, self.sin, self.rot_dim
        cos, sin = self.tables[ntk_alpha(batch.max_context, self.max_seq_len)]
        return cos, sin, self.rot_dim

    def check_positions(self, max_position: int) -> None:
        # tests/modules/test_positions.py:156-168: a position beyond the table raises
        if max_position >= self.max_positions:
            raise IndexError(f"position {max_position} is beyond the rotary table of {self.max_positions} positions")


register_part("position", "rope", RotaryEncoding)
