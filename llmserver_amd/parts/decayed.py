"""Mixers that carry a matrix per head from token to token under one decay per head:
``S_t = a_t S_(t-1) + b_t k_t v_t^T``, ``o_t = S_t^T q_t``.  No softmax and no denominator; what differs between them is where
``a`` and ``b`` come from and what stands around the recurrence.  Both run on one kernel (``ops.decayed_recurrence``), which
takes portions of prompts in chunks, as matrix products, and single tokens one by one.

* :class:`Retention`: ``a`` is a constant per head, ``b`` is 1; queries and keys are rotated; each head's ``o`` is divided by
  its root mean square and multiplied by ``silu`` of a gate.
* :class:`StateSpaceDuality` (Mamba-2): ``b`` is a step size per head and token and ``a = exp(-exp(A_log) b)``; keys, values
  and queries pass a short convolution and silu, and groups of heads share keys and queries; a skip from the value, a gate
  and a norm in equal parts follow.

State per request: the matrices ``[heads, dim, vdim]`` in float32 and, behind them, the convolution's last ``taps - 1`` inputs,
oldest first; zeros before a sequence's first token.
"""
from __future__ import annotations

import dataclasses
import math
from typing import Sequence

import torch

from .base import VECTOR, Mixer, ParamSpec, PositionEncoding, StateSpec
from .linear import Linear


def run_recurrence(ctx, cache, q, k, v, log_keep, take, q_scale, heads, key_heads, dim, value_dim):
    """The recurrence over the step's tokens: float32 ``[T, heads * value_dim]``.  Scratch memory of the chunked form is
    given where the kernels ask for it."""
    ops, n = ctx.ops, v.shape[0]
    out = ctx.empty((n, heads * value_dim), dtype=torch.float32)
    chunks = ops.matrix_memory_chunks(n, ctx.row_len.shape[0])
    scratch = {}
    if chunks:
        scratch = {"sums": ctx.empty((chunks, heads, dim, value_dim), dtype=torch.float32),
                   "totals": ctx.empty((chunks, heads), dtype=torch.float32)}
    ops.decayed_recurrence(q, k, v, log_keep, take, q_scale, cache.state, ctx.state_slots, ctx.row_start, ctx.row_len, ctx.row_ctx, out,
                           heads, key_heads, dim, value_dim, **scratch)
    return out


@dataclasses.dataclass(frozen=True)
class RetentionNames:
    q: str = "q"
    k: str = "k"
    v: str = "v"
    gate: str = "g"
    out: str = "o"


class Retention(Mixer):
    """``q = rotate(W_q h)``, ``k = rotate(W_k h) * dim^-1/2``, ``v = W_v h``; ``S_t = decay_h S_(t-1) + k_t v_t^T``,
    ``o_t = S_t^T q_t``; each head's ``o`` divided by its root mean square, times ``silu(W_g h)``, then the output projection.
    Rotated rows, decays, state, read-outs and norms are 32-bit."""
    graph_safe = True

    def __init__(self, width: int, heads: int, dim: int, value_dim: int, decay: Sequence[float], position: PositionEncoding, norm_eps: float,
                 names: RetentionNames = RetentionNames()):
        if len(decay) != heads or not all(0.0 < d for d in decay):
            raise ValueError(f"{heads} heads take as many positive decays, got {list(decay)}")
        if position.rotary_dim is not None and (getattr(position, "pairing", None) != "halves" or position.rotary_dim > dim):
            raise ValueError("queries and keys turn as halves, on up to all dimensions of a head")
        self.width, self.heads, self.dim, self.value_dim = width, heads, dim, value_dim
        self.decay, self.position, self.norm_eps, self.names = tuple(float(d) for d in decay), position, float(norm_eps), names
        self.key_scale = float(dim) ** -0.5
        keys, values = heads * dim, heads * value_dim
        self.proj = Linear(width, (names.q, names.k, names.v, names.gate), (keys, keys, values, values), bare_names=True)
        self.o = Linear(values, (names.out,), (width,), bare_names=True)
        self.log_decay = None       # float32 [heads]

    def cache_spec(self):
        return StateSpec((self.heads * self.dim * self.value_dim,), "float32")

    def param_specs(self):
        return {**self.proj.param_specs(), **self.o.param_specs()}

    def assign(self, name, tensor):
        if self.o.owns(name):
            self.o.assign(name, tensor)
        elif self.proj.owns(name):
            self.proj.assign(name, tensor)
        else:
            raise KeyError(name)

    def finalize(self):
        self.proj.finalize()
        self.o.finalize()
        self.log_decay = torch.tensor([math.log(d) for d in self.decay], dtype=torch.float32, device=self.o.weight.device)

    def mixing_flops(self, new_tokens: int, context: int) -> float:
        """Per token, head and state element: the decay, the outer product's sum and the read-out."""
        return 6.0 * new_tokens * self.heads * self.dim * self.value_dim

    def forward(self, x, ctx, cache):
        ops, n = ctx.ops, x.shape[0]
        keys, values = self.heads * self.dim, self.heads * self.value_dim
        proj = self.proj.forward(x, ctx)
        q, k = ctx.empty((n, keys), dtype=torch.float32), ctx.empty((n, keys), dtype=torch.float32)
        ops.rotate_heads(proj[:, :keys], proj[:, keys:2 * keys], self.position.cos_sin(ctx), self.key_scale, q, k, self.heads)
        mixed = run_recurrence(ctx, cache, q, k, proj[:, 2 * keys:2 * keys + values], self.log_decay, None, 1.0, self.heads, self.heads,
                               self.dim, self.value_dim)
        gated = ctx.empty((n, values))
        ops.heads_norm_gate(mixed, None, False, self.norm_eps, proj[:, 2 * keys + values:], gated, self.heads, self.value_dim)
        return self.o.forward(gated, ctx)


@dataclasses.dataclass(frozen=True)
class StateSpaceNames:
    into: str = "in"
    conv: str = "conv"
    conv_bias: str = "conv.b"
    step_bias: str = "dt_bias"
    decay_scale: str = "A_log"
    skip: str = "D"
    norm: str = "norm"
    out: str = "o"


class StateSpaceDuality(Mixer):
    """``W_in h`` is ``[z | x | B | C | dt]`` with ``heads * value_dim`` gates and values, ``groups * state`` keys ``B`` and queries
    ``C`` each, and a step size a head.  ``x``, ``B`` and ``C`` pass a causal convolution with bias and silu;
    ``dt = softplus(dt + dt_bias)``; ``S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T``, ``y_t = S_t^T C_t + D x_t``, head ``h``
    reading group ``h // (heads / groups)``.  ``y * silu(z)`` is RMS-normed in ``norm_groups`` equal parts, times a weight per
    channel, then the output projection.  Step sizes, decays, state, read-outs and norms are 32-bit."""
    graph_safe = True

    def __init__(self, width: int, heads: int, value_dim: int, state: int, groups: int, taps: int, norm_groups: int, norm_eps: float,
                 names: StateSpaceNames = StateSpaceNames()):
        if heads % groups:
            raise ValueError(f"{heads} heads do not fall into {groups} equal groups")
        if (heads * value_dim) % norm_groups:
            raise ValueError(f"{heads * value_dim} channels do not fall into {norm_groups} equal parts")
        if taps < 1:
            raise ValueError(f"a convolution needs at least one tap, got {taps}")
        self.width, self.heads, self.value_dim, self.state, self.groups, self.taps = width, heads, value_dim, state, groups, int(taps)
        self.norm_groups, self.norm_eps, self.names = int(norm_groups), float(norm_eps), names
        self.inner, self.keys = heads * value_dim, groups * state
        self.channels = self.inner + 2 * self.keys              # what the convolution runs over: x | B | C
        self.matrix_size = heads * state * value_dim
        self.proj = Linear(width, (names.into,), (2 * self.inner + 2 * self.keys + heads,), bare_names=True)
        self.o = Linear(self.inner, (names.out,), (width,), bare_names=True)
        self.conv_weight = self.conv_bias = self.step_bias = self.decay_scale = self.skip = self.norm_weight = None

    def cache_spec(self):
        return StateSpec((self.matrix_size + (self.taps - 1) * self.channels,), "float32")

    def _vectors(self):
        n = self.names
        return {n.conv: ("conv_weight", ParamSpec((self.channels, self.taps), VECTOR, "normal")),
                n.conv_bias: ("conv_bias", ParamSpec((self.channels,), VECTOR, "bias")),
                n.step_bias: ("step_bias", ParamSpec((self.heads,), VECTOR, "bias")),
                n.decay_scale: ("decay_scale", ParamSpec((self.heads,), VECTOR, "bias")),
                n.skip: ("skip", ParamSpec((self.heads,), VECTOR, "norm")),
                n.norm: ("norm_weight", ParamSpec((self.inner,), VECTOR, "norm"))}

    def param_specs(self):
        return {**self.proj.param_specs(), **self.o.param_specs(), **{name: spec for name, (_, spec) in self._vectors().items()}}

    def assign(self, name, tensor):
        vectors = self._vectors()
        if name in vectors:
            setattr(self, vectors[name][0], tensor)
        elif self.o.owns(name):
            self.o.assign(name, tensor)
        elif self.proj.owns(name):
            self.proj.assign(name, tensor)
        else:
            raise KeyError(name)

    def finalize(self):
        self.proj.finalize()
        self.o.finalize()
        self.conv_weight = self.conv_weight.contiguous()

    def mixing_flops(self, new_tokens: int, context: int) -> float:
        """Per token, head and state element: the decay, the outer product's sum and the read-out."""
        return 6.0 * new_tokens * self.heads * self.state * self.value_dim

    def forward(self, x, ctx, cache):
        ops, n = ctx.ops, x.shape[0]
        inner, keys = self.inner, self.keys
        proj = self.proj.forward(x, ctx)
        through = proj[:, inner:inner + self.channels]
        single = ctx.n_tokens == ctx.n_rows         # one token a row: the thread that reads a row's last inputs also moves them on
        mixed = ctx.empty((n, self.channels))
        steps, log_keep = ctx.empty((n, self.heads), dtype=torch.float32), ctx.empty((n, self.heads), dtype=torch.float32)
        ops.ssd_prepare(through, self.conv_weight, self.conv_bias, cache.state, self.matrix_size, ctx.state_slots, ctx.token_row, ctx.positions,
                        ctx.row_start, mixed, proj[:, inner + self.channels:], self.step_bias, self.decay_scale, steps, log_keep, keep=single)
        if not single and self.taps > 1:
            ops.delta_conv_keep(through, self.channels, self.taps, cache.state, self.matrix_size, ctx.state_slots, ctx.row_start, ctx.row_len,
                                ctx.row_ctx)
        y = run_recurrence(ctx, cache, mixed[:, inner + keys:], mixed[:, inner:inner + keys], mixed[:, :inner], log_keep, steps, 1.0, self.heads,
                           self.groups, self.state, self.value_dim)
        normed = ctx.empty((n, inner))
        ops.gated_group_norm(y, mixed[:, :inner], self.skip, proj[:, :inner], self.norm_weight, self.norm_eps, normed, self.heads, self.norm_groups)
        return self.o.forward(normed, ctx)
