"""Rotate-half rotary position encoding over the full head.

``inv_freq_i = theta^(-2i/d)`` for ``i = 0..d/2-1``, ``angle = position * inv_freq`` in 32-bit,
``x' = x*cos + rotate_half(x)*sin`` with ``rotate_half(x) = cat(-x[d/2:], x[:d/2])``
(utils/layers.py:140-177).  Positions are absolute token positions
(utils/batch.py:30,80).  The table of inverse frequencies is made once on the
host with the reference's expression (utils/layers.py:158); the rotation itself
happens inside the mixer's fused kernel, which gets the table and the positions of the step's
tokens, so a position depends on nothing but the token's own index.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Optional

import torch

from .base import PositionEncoding


@dataclasses.dataclass(frozen=True)
class YarnScaling:
    """Frequencies stretched for contexts longer than the ``original`` length: pairs that turn fast (more than ``fast`` times
    over that length) keep theirs, pairs that turn slowly (fewer than ``slow`` times) are divided by ``factor``, the pairs
    between are mixed, linearly in the pair's number; cosines and sines are multiplied by ``0.1 ln(factor) + 1``."""
    factor: float
    original: float
    fast: float
    slow: float

    def frequencies(self, plain, dims: int, base: float):
        def pair_that_turns(times):
            return dims * math.log(self.original / (2.0 * math.pi * times)) / (2.0 * math.log(base))

        first = max(math.floor(pair_that_turns(self.fast)), 0)
        last = min(math.ceil(pair_that_turns(self.slow)), dims - 1)
        width = max(last - first, 0.001)
        out = []
        for i, frequency in enumerate(plain):
            share = min(max((i - first) / width, 0.0), 1.0)
            out.append(frequency / self.factor * share + frequency * (1.0 - share))
        return out

    @property
    def amplitude(self) -> float:
        return 0.1 * math.log(self.factor) + 1.0


class RotaryPosition(PositionEncoding):
    """``rotary_dim`` may be smaller than the head it is applied to: dimension ``i`` then turns with ``i + rotary_dim / 2``
    and the dimensions behind ``rotary_dim`` pass unchanged (a mixer says whether its kernels do that).  ``precise``: the
    frequencies are formed in 64-bit and rounded to 32-bit once, instead of with the 32-bit expression above (``scaling``
    implies it)."""
    pairing = "halves"

    def __init__(self, rotary_dim: int, theta: float, precise: bool = False, scaling: Optional[YarnScaling] = None):
        if rotary_dim % 2:
            raise ValueError(f"rotary_dim must be even: {rotary_dim}")
        self.rotary_dim = rotary_dim
        self.theta = float(theta)
        self.scaling = scaling
        self.precise = bool(precise) or scaling is not None
        self._tables = {}

    def inverse_frequencies(self) -> torch.Tensor:
        if self.precise:
            plain = [self.theta ** (-2.0 * i / self.rotary_dim) for i in range(self.rotary_dim // 2)]
            if self.scaling is not None:
                plain = self.scaling.frequencies(plain, self.rotary_dim, self.theta)
            return torch.tensor(plain, dtype=torch.float32)
        indices = torch.arange(0, self.rotary_dim, 2, dtype=torch.long)
        return 1.0 / (self.theta ** (indices.to(torch.float32) / self.rotary_dim))

    def rotary_table(self, device):
        key = str(device)
        if key not in self._tables:
            self._tables[key] = self.inverse_frequencies().to(device=device, dtype=torch.float32).contiguous()
        return self._tables[key]

    def cos_sin(self, ctx):
        """cos and sin of the step's tokens, float32 ``[T, rotary_dim]``: computed once a step, whatever
        the number of layers that rotate with this encoding."""
        amplitude = {"amplitude": self.scaling.amplitude} if self.scaling is not None else {}
        return ctx.computed(("rotary", id(self)), lambda: ctx.ops.rotary_table(ctx.positions, self.rotary_table(ctx.device), **amplitude))


class PairedRotaryPosition(RotaryPosition):
    """The same angles, for mixers that turn neighbouring dimensions (2i, 2i+1) together instead of (i, i + d/2):
    ``(u, v) -> (u cos a - v sin a, v cos a + u sin a)`` with ``a = position * theta^(-2i/d)``.  ``rotary_dim`` may be
    smaller than the vector it is applied to; the dimensions behind it pass unchanged.  The frequencies are formed in
    64-bit and rounded to 32-bit once; angles, cosines and sines are 32-bit."""
    pairing = "neighbours"

    def inverse_frequencies(self) -> torch.Tensor:
        return torch.tensor([self.theta ** (-2.0 * i / self.rotary_dim) for i in range(self.rotary_dim // 2)], dtype=torch.float32)


class NoPosition(PositionEncoding):
    """Tokens enter the mixer unrotated."""
