"""Routed experts: every token's feed-forward is a weighted sum of ``top`` of ``experts`` small gated feed-forwards.

Router logits ``z = R h`` (plus a bias per expert, where the checkpoint has one) in 32-bit.  ``scoring="softmax"``: the ``top`` largest logits are chosen (the first of equal
ones) and weighted by the softmax over the chosen logits only.  ``scoring="sigmoid"``: scores ``sigmoid(z)``; with
``groups=(count, keep)`` the experts form ``count`` equal groups of neighbours, a group's score is the sum of its two
largest scores, and only experts of the ``keep`` best groups can be chosen; the ``top`` largest scores are chosen and
are the weights as they are.  Expert: ``D (act(G h) * (U h))`` with ``act = silu``, or, with ``activation="clamped"``,
``g = min(G h, limit)``, ``u = clamp(U h, -limit, limit)``, ``D (g * sigmoid(1.702 g) * (u + 1))``; with ``activation="relu2"``
there is no gate: ``D max(U h, 0)^2``; no biases.
``scoring="softmax_all"``: scores are the softmax over all experts; the ``top`` largest of score + a correction per expert are
chosen; their scores, divided by their sum (+ 1e-20) and times a constant, are the weights.

``identity`` more choices behind the experts are identity experts: they have no matrices, their output is ``h`` itself.  A
:class:`SharedExpert` beside the routed ones runs for every token, times ``sigmoid(g . h)``, one number a token; its gate's
row stands behind the router's, so that one product makes both.  The experts' matrices
are stacked (``[experts, 2F, W]`` gate rows then up rows, ``[experts, W, F]``), and the kernels pick each token's from
the list of chosen experts on the device: nothing of the routing is read on the host.
"""
from __future__ import annotations

import dataclasses
from typing import Optional, Tuple

import torch

from .base import VECTOR, FeedForward, ParamSpec
from .linear import Linear


@dataclasses.dataclass(frozen=True)
class SharedExpert:
    """A feed-forward of the routed experts' form and of its own inner size that every token uses; names below ``prefix``
    (``pieces``: as the routed experts')."""
    intermediate: int
    prefix: str = "shared"
    pieces: Tuple[str, ...] = ("gate", "up", "down")
    gate: Optional[str] = "sg"      # the row [1, W] whose product's sigmoid multiplies the result (None: nothing does)


class RoutedExperts(FeedForward):
    reads_stream = True       # forward takes ``stream=``: the 32-bit rows that ``x`` was rounded from, for the router

    SCORINGS = ("softmax", "sigmoid", "softmax_all")
    ACTIVATIONS = ("silu", "clamped", "relu2")
    UNGATED = ("relu2",)            # experts of two matrices: ``pieces`` names the up and the down matrix

    def __init__(self, width: int, intermediate: int, experts: int, top: int, router: str = "router", expert: str = "e{}",
                 pieces=("gate", "up", "down"), scoring: str = "softmax", groups=None, activation: str = "silu", limit: float = 0.0,
                 reads_stream: bool = True, router_bias: str = None, correction: str = None, weight_scale: float = 1.0, identity: int = 0,
                 shared: SharedExpert = None):
        """``correction``: the name of a vector that joins the scores for the choice only, or None.  ``identity``: how many of
        the router's outputs, the last ones, are identity experts (``experts`` counts those with matrices)."""
        if not 1 <= top <= experts + identity or identity < 0:
            raise ValueError(f"a token uses {top} of {experts} experts and {identity} identity experts")
        if (correction is not None or weight_scale != 1.0) and scoring != "softmax_all":
            raise ValueError("a correction of the choice and a scale of the weights come with the softmax over all experts")
        if scoring not in self.SCORINGS or activation not in self.ACTIVATIONS:
            raise ValueError(f"scoring {scoring!r} / activation {activation!r}: built are {self.SCORINGS} and {self.ACTIVATIONS}")
        if groups is not None:
            count, keep = groups
            if scoring != "sigmoid" or experts % count or not 1 <= keep <= count or top > keep * (experts // count):
                raise ValueError(f"{experts} experts in {count} groups of which {keep} are kept, {top} chosen, scoring {scoring!r}")
        if shared is not None and activation == "clamped":
            raise ValueError("the shared expert's activation is silu or the square of the rectifier, as the routed experts' then is")
        self.gated = activation not in self.UNGATED
        if any(len(names) != (3 if self.gated else 2) for names in (pieces, *((shared.pieces,) if shared is not None else ()))):
            raise ValueError(f"an expert with the activation {activation!r} has {3 if self.gated else 2} matrices, named are {tuple(pieces)}")
        if activation == "clamped" and not limit > 0.0:
            raise ValueError("the clamped activation needs its limit")
        self.scoring, self.groups, self.activation, self.limit = scoring, tuple(groups) if groups is not None else None, activation, float(limit)
        self.reads_stream = reads_stream
        self.width, self.intermediate, self.experts, self.top = width, intermediate, experts, top
        self.router_name, self.expert_name, self.pieces = router, expert, tuple(pieces)
        self._parts = {}
        self.router_bias_name = router_bias       # the name of a vector that is added to the router's logits, or None
        self.router_bias = None   # float32 [experts]
        self.correction_name, self.correction = correction, None      # float32 [experts + identity]
        self.weight_scale, self.identity, self.shared = float(weight_scale), int(identity), shared
        self.choices = experts + self.identity
        self.router = None        # float32 [experts + identity (+ 1: the shared expert's gate), W]
        self.shared_gate = None
        self.shared_gate_up = self.shared_down = None
        if shared is not None:
            *ups, down = (f"{shared.prefix}.{piece}" for piece in shared.pieces)
            self.shared_gate_name = f"{shared.prefix}.{shared.gate}" if shared.gate is not None else None
            self.shared_gate_up = Linear(width, ups, (shared.intermediate,) * len(ups), bare_names=True)
            self.shared_down = Linear(shared.intermediate, (down,), (width,), bare_names=True)
        self.gate_up = None       # [experts, 2F, W]; without gates [experts, F, W]
        self.down = None          # [experts, W, F]

    def _names(self):
        """(names of the matrices that read the token, name of the one that writes) of every expert."""
        for index in range(self.experts):
            *ups, down = (f"{self.expert_name.format(index)}.{piece}" for piece in self.pieces)
            yield ups, down

    def param_specs(self):
        share = self.top / self.choices
        specs = {self.router_name: ParamSpec((self.choices, self.width), VECTOR, "normal")}
        if self.router_bias_name is not None:
            specs[self.router_bias_name] = ParamSpec((self.choices,), VECTOR, "bias")
        if self.correction_name is not None:
            specs[self.correction_name] = ParamSpec((self.choices,), VECTOR, "bias")
        if self.shared is not None:
            specs.update({**self.shared_gate_up.param_specs(), **self.shared_down.param_specs()})
            if self.shared_gate_name is not None:
                specs[self.shared_gate_name] = ParamSpec((1, self.width), VECTOR, "normal")
        for ups, down in self._names():
            for up in ups:
                specs[up] = ParamSpec((self.intermediate, self.width), share_per_token=share)
            specs[down] = ParamSpec((self.width, self.intermediate), share_per_token=share)
        return specs

    def assign(self, name, tensor):
        if name == self.router_name:
            self.router = tensor
        elif name == self.router_bias_name:
            self.router_bias = tensor
        elif name == self.correction_name:
            self.correction = tensor
        elif self.shared is not None and self.shared_gate_name is not None and name == self.shared_gate_name:
            self.shared_gate = tensor
        elif self.shared is not None and self.shared_gate_up.owns(name):
            self.shared_gate_up.assign(name, tensor)
        elif self.shared is not None and self.shared_down.owns(name):
            self.shared_down.assign(name, tensor)
        else:
            self._parts[name] = tensor

    def finalize(self):
        names = list(self._names())
        self.gate_up = torch.stack([torch.cat([self._parts[up] for up in ups], dim=0) for ups, _ in names]).contiguous()
        self.down = torch.stack([self._parts[down] for _, down in names]).contiguous()
        self._parts.clear()
        if self.shared is not None:
            self.shared_gate_up.finalize()
            self.shared_down.finalize()
            if self.shared_gate is not None:
                self.router = torch.cat([self.router, self.shared_gate], dim=0).contiguous()
                self.shared_gate = None

    def forward(self, x, ctx, stream=None):
        """``x [T, W]`` in the compute type -> float32 ``[T, W]``.  ``stream``: the same rows in 32-bit, if the caller
        has them (the router's logits are 32-bit either way; from these they need no widening first)."""
        ops = ctx.ops
        n = x.shape[0]
        chosen = ctx.empty((n, self.top), dtype=torch.int32)
        weights = ctx.empty((n, self.top), dtype=torch.float32)
        extra = {} if self.scoring == "softmax" else {"scoring": self.scoring, "groups": self.groups}
        if self.router_bias is not None:
            extra["bias"] = self.router_bias
        if self.scoring == "softmax_all":
            extra.update(correction=self.correction, weight_scale=self.weight_scale)
        shared_gate = None
        if self.shared is not None and self.shared.gate is not None:
            shared_gate = extra["gate_out"] = ctx.empty((n,), dtype=torch.float32)
        ops.route_experts(x if stream is None else stream, self.router, self.top, chosen, weights, **extra)
        out = ctx.empty((n, self.width), dtype=torch.float32)
        extra = {} if self.activation == "silu" else {"activation": self.activation, "limit": self.limit}
        beside = {"identity": self.identity} if self.identity else {}
        inside = self.shared is not None and ops.shared_expert_inside(n)     # few tokens: its products are made beside the routed experts'
        shared_y = {}
        if self.shared is not None and not inside:
            shared_y = {"shared_y": self.shared_down.forward(self._shared_hidden(x, ctx), ctx), "shared_gate": shared_gate}
        # many tokens: pairs sorted by expert
        if not inside and ops.experts_sorted(x, self.gate_up, self.down, chosen, weights, out, **extra, **beside, **shared_y):
            return out
        hidden = ctx.empty((n * self.top, self.intermediate))
        after = {"x": x} if self.identity else {}
        if inside:
            shared_hidden = ctx.empty((n, self.shared.intermediate))
            beside["shared"] = (self.shared_gate_up.weight, shared_hidden)
            after.update(shared=(self.shared_down.weight, shared_hidden), shared_gate=shared_gate)
        ops.experts_gate_up(x, self.gate_up, chosen, hidden, **extra, **beside)
        ops.experts_down(hidden, self.down, chosen, weights, out, **after, **shared_y)
        return out

    def _shared_hidden(self, x, ctx):
        """The shared expert's ``act(G h) * (U h)`` (or ``act(U h)``) as products of its own."""
        if not self.gated:
            return ctx.ops.linear_activated(x, self.shared_gate_up.weight, self.activation)
        hidden = ctx.ops.linear_gated(x, self.shared_gate_up.weight)
        if hidden is None:
            gate_up = self.shared_gate_up.forward(x, ctx)
            hidden = ctx.empty((x.shape[0], self.shared.intermediate))
            ctx.ops.swiglu(gate_up, hidden)
        return hidden
