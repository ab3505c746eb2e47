"""Setodra put together from parts, layer by layer, from its typed configuration.

The embedding row, times a constant, starts one residual stream in 32-bit.  Every layer is a pre-norm block
(:class:`~llmserver_amd.parts.block.MultiStreamBlock` with its one plain stream): a mixer and, unless the layer has none, routed
experts, each under an RMS norm.  A layer's mixer is attention over a shared latent whose rotated part is stretched by YaRN
(:class:`~llmserver_amd.parts.latent_attention.LatentAttention`), retention, or a state-space mixer (both
:mod:`~llmserver_amd.parts.decayed`).  The experts (:class:`~llmserver_amd.parts.experts.RoutedExperts`) are scored by a softmax
over all of them and chosen with a correction; the last choices are identity experts, and a gated shared expert runs for every
token.  A run of layers may be passed several times with the same weights: in front of every pass a vector of its own joins
the stream, in front of every pass but the first the embedding's output too (:class:`~llmserver_amd.parts.block.PassEntry`);
every pass keeps a cache or state of its own, so the order of calls names a block several times and a cache once.  Tensor
names: ``embed``, ``loop.step``, ``l<i>.<...>``, ``final.norm``, ``head``; every name is the tensor's whole name.
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.setodra import LatentSizes, RetentionSizes, SetodraConfig
from ..parts import (HyperConnection, LatentAttention, LatentAttentionNames, Linear, LoopSteps, MultiStreamBlock, NoPosition, PassEntry,
                     Retention, RotaryPosition, RoutedExperts, SharedExpert, StateSpaceDuality, StreamReadNorm, TokenEmbedding, YarnScaling)
from .decoder import DecoderModel, LayerCall

LATENT_NAMES = LatentAttentionNames(q="q", down="dkv", down_norm="dkv.norm", up_keys="uk", up_values="uv", out="o", sink=None, gate=None)
BLOCK_NAMES = ("norm1", "mix", "norm2", "mlp", "hc1", "hc2")     # (the connections are plain sums: no tensors)
MODEL_NAMES = ("embed", "l", "final.norm")
HEAD_NAME = "head"
LOOP_NAME, STEP_NAME = "loop", "step"
SCORING = "softmax_all"          # fixed by the design, as is the correction of the choice


def build_setodra(config: SetodraConfig) -> DecoderModel:
    eps, width = config.norm_eps, config.width

    def norm():
        return StreamReadNorm(width, eps, 1, tensor="")

    def connection():
        return HyperConnection(1, learned=False)

    positions = {}

    def position(rot):
        if not rot.dims:
            return NoPosition()
        if rot not in positions:
            scaling = YarnScaling(**rot.scaling.to_dict()) if rot.scaling is not None else None
            positions[rot] = RotaryPosition(rot.dims, rot.base, precise=True, scaling=scaling)
        return positions[rot]

    blocks = []
    for layer in config.layers:
        sizes = layer.mixer
        if isinstance(sizes, LatentSizes):
            mixer = LatentAttention(width, sizes.heads, sizes.dim, sizes.rot_dim, sizes.vdim, sizes.kv_rank, position(sizes.rot), sizes.scale, eps,
                                    names=LATENT_NAMES)
        elif isinstance(sizes, RetentionSizes):
            mixer = Retention(width, sizes.heads, sizes.dim, sizes.vdim, sizes.decay, position(sizes.rot), eps)
        else:
            mixer = StateSpaceDuality(width, sizes.heads, sizes.vdim, sizes.state, sizes.groups, sizes.conv, sizes.norm_groups, eps)
        feed = None
        if layer.mlp is not None:
            shared = SharedExpert(layer.mlp.shared_ff) if layer.mlp.shared_ff else None
            feed = RoutedExperts(width, layer.mlp.ff, layer.mlp.experts, layer.mlp.top, scoring=SCORING, correction="correction",
                                 weight_scale=layer.mlp.scale, identity=layer.mlp.identity, shared=shared, reads_stream=False)
        blocks.append(MultiStreamBlock(norm(), mixer, connection(), *((norm(), feed, connection()) if feed is not None else ()),
                                       names=BLOCK_NAMES))
    embedding = TokenEmbedding(config.vocab, width, tensor="", wide=True, scale=config.embedding_scale, streams=1)
    steps = LoopSteps(config.loop.times, width, tensor=STEP_NAME) if config.loop is not None else None
    # every run of a layer has a cache or state of its own; the weights are the block's
    order = [LayerCall(block, run, entry=PassEntry(steps, number, embedding) if number is not None else None)
             for run, (block, number) in enumerate(config.layer_runs())]
    head = Linear(width, (HEAD_NAME,), (config.vocab,), out_float32=True, bare_names=True)
    return DecoderModel(config, embedding, blocks, norm(), head, tie_head=False, order=order, names=MODEL_NAMES,
                        layer_name=lambda i: f"l{i}", extras={LOOP_NAME: steps} if steps is not None else None)


register_architecture(SetodraConfig.MODEL_TYPE, SetodraConfig, build_setodra, replace=True)
