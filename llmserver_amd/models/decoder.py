"""A decoder assembled from parts: embedding, blocks, the order they run in, final norm, head.

The order is data: ``order`` is a list of :class:`LayerCall`, each naming a block and the cache
it uses.  A block may be named twice (its weights are shared) and a call may read the cache that
another call writes.  The plain stacked model is ``[LayerCall(i, i) for i in range(L)]``
(utils/model.py:124-132).  Rows whose logits are wanted are selected before the
final norm and the head (utils/model.py:147-158).
"""
from __future__ import annotations

import dataclasses
from typing import Dict, Optional, Sequence

import torch

from ..parts.base import Block, Norm, ParamSpec, Part, StreamUpdate
from ..parts.embedding import TokenEmbedding
from ..parts.linear import Linear


@dataclasses.dataclass(frozen=True)
class LayerCall:
    block: int                  # index into ``blocks``
    cache: int                  # index of the cache this call uses
    writes_cache: bool = True   # False: read the cache another call has written
    entry: object = None        # what happens to the stream right before this call (``forward(resid, delta, ctx, following)``), or None


def joined(prefix: str, name: str) -> str:
    """``prefix.name``, or the prefix alone for a part whose own name is its tensor's."""
    return f"{prefix}.{name}" if name else prefix


class DecoderModel:
    """``names``: the checkpoint's names of the embedding, of the list of layers and of the final norm; layer ``i``'s
    tensors start with ``layer_name(i)`` (default: ``<layers>.<i>``).  ``extras``: parts with tensors that belong to no layer
    (vectors that calls of the order add to the stream), by the checkpoint's prefix."""

    def __init__(self, config, embedding: TokenEmbedding, blocks: Sequence[Block], final_norm: Norm, head: Linear,
                 tie_head: bool, order: Optional[Sequence[LayerCall]] = None,
                 names=("model.embed_tokens", "model.layers", "model.norm"), layer_name=None, extras: Optional[Dict[str, Part]] = None):
        self.config = config
        self.embedding = embedding
        self.blocks = list(blocks)
        self.final_norm = final_norm
        self.head = head
        self.tie_head = tie_head
        self.order = list(order) if order is not None else [LayerCall(i, i) for i in range(len(self.blocks))]
        self.embed_name, self.layers_name, self.norm_name = names
        self.layer_name = layer_name if layer_name is not None else (lambda index: f"{self.layers_name}.{index}")
        self.extras = dict(extras or {})
        self._owners = None
        self.after_call = None      # for whoever looks inside a step: called as (index in the order, residual, pending update) behind every call
        self.device = None
        self.dtype = None
        self._check_order()

    # -- structure ---------------------------------------------------------------------
    def _check_order(self):
        writers = {}
        for call in self.order:
            if not 0 <= call.block < len(self.blocks):
                raise ValueError(f"order names block {call.block}, the model has {len(self.blocks)}")
            if call.writes_cache:
                if call.cache in writers:
                    raise ValueError(f"cache {call.cache} is written by two calls of the order")
                writers[call.cache] = call.block
        for call in self.order:
            spec = self.blocks[call.block].cache_spec()
            if spec is None:
                continue
            if call.cache not in writers:
                raise ValueError(f"cache {call.cache} is read but never written")
            if self.blocks[writers[call.cache]].cache_spec() != spec:
                raise ValueError(f"cache {call.cache} is shared by mixers with different cache needs")

    def cache_specs(self) -> Dict[int, object]:
        """cache index -> what its writer stores."""
        specs = {}
        for call in self.order:
            spec = self.blocks[call.block].cache_spec()
            if spec is not None and call.writes_cache:
                specs[call.cache] = spec
        return specs

    # -- parameters --------------------------------------------------------------------
    def _named(self):
        """(checkpoint name, owning part, the part's own name of the tensor, spec) of every tensor."""
        for k, v in self.embedding.param_specs().items():
            yield joined(self.embed_name, k), self.embedding, k, v
        for prefix, part in self.extras.items():
            for k, v in part.param_specs().items():
                yield joined(prefix, k), part, k, v
        for i, block in enumerate(self.blocks):
            for k, v in block.param_specs().items():
                yield joined(self.layer_name(i), k), block, k, v
        for k, v in self.final_norm.param_specs().items():
            yield joined(self.norm_name, k), self.final_norm, k, v
        for k, v in self.head.param_specs().items():
            # Tied when the configuration says so or the checkpoint holds no head
            # (utils/model_loader.py:56-59).
            yield k, self.head, k, dataclasses.replace(v, optional=True)

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {name: spec for name, _, _, spec in self._named()}

    def ignored_names(self):
        """Checkpoint tensors that may be present but are not read."""
        return set(self.head.param_specs()) if self.tie_head else set()

    def assign(self, name: str, tensor: torch.Tensor) -> None:
        if self._owners is None:
            self._owners = {full: (part, own) for full, part, own, _ in self._named()}
        if name not in self._owners:
            raise KeyError(name)
        part, own = self._owners[name]
        part.assign(own, tensor)

    def finalize(self, assigned: Sequence[str], device, dtype) -> None:
        head_names = set(self.head.param_specs())
        if self.tie_head or not (head_names & set(assigned)):
            self.head.share_weight(self.embedding.weight)   # alias, not a copy
            self.tie_head = True
        for part in (self.embedding, *self.extras.values(), *self.blocks, self.final_norm, self.head):
            part.finalize()
        self.device, self.dtype = torch.device(device), dtype

    # -- the forward pass over one flat batch ----------------------------------------------
    def prepare(self, ctx) -> None:
        for call in self.order:
            self.blocks[call.block].mixer.prepare(ctx)

    def forward(self, ctx, caches) -> torch.Tensor:
        """Run the step's tokens through every call of the order; float32 logits ``[n_out, vocab]``."""
        resid = self.embedding.forward(ctx.token_ids, ctx)
        delta = None
        for index, call in enumerate(self.order):
            block = self.blocks[call.block]
            if call.entry is not None:
                resid, delta = call.entry.forward(resid, delta, ctx, block.entry_norm())
            after = self.order[index + 1] if index + 1 < len(self.order) else None
            if block.takes_following and after is not None and after.entry is None:
                # The block may add its last update itself and prepare the next block's first norm.
                following = self.blocks[after.block].entry_norm()
                resid, delta = block.forward(resid, delta, ctx, caches.view(call), following=following)
            else:
                resid, delta = block.forward(resid, delta, ctx, caches.view(call))
            if self.after_call is not None:
                self.after_call(index, delta.resid if isinstance(delta, StreamUpdate) else resid, delta)
        if isinstance(delta, StreamUpdate):
            resid, delta = delta.resid, None
        if ctx.n_out == 0:
            return torch.empty((0, self.head.out_features), device=resid.device, dtype=torch.float32)
        selected = self.final_norm.add_norm(resid, delta, ctx, rows=ctx.logit_idx)
        return self.head.forward(selected, ctx)
