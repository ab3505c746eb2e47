"""Mefurax put together from parts, layer by layer, from its typed configuration.

The embedding row starts a residual stream in 32-bit.  Every layer is a :class:`~llmserver_amd.parts.block.SumNormBlock`:
the sublayers read the stream itself, and the norm stands behind the sum of the scaled stream and a sublayer's result.  A
layer's mixer is attention (:class:`~llmserver_amd.parts.attention.GQAttention`) of one of two kinds: projections with biases that
pass short convolutions and are normed as a whole, no rotation, scores that fall with the distance, a window; or rotated
heads of unit root mean square, capped scores, chunks of the sequence, a gate a head.  In either kind a layer's values may
be mixed with those of the first layer that does so.  Its feed-forward is a gated one with the tanh form of GELU
(:class:`~llmserver_amd.parts.mlp.GatedMLP`), routed experts without gates beside a shared one
(:class:`~llmserver_amd.parts.experts.RoutedExperts`), or none.  All norms of the stream have weights stored around zero.
Tensor names: ``embed``, ``l<i>.<...>``, ``final.norm``, ``head``; every name is the tensor's whole name.
"""
from __future__ import annotations

from ..config.gogalix import DenseSizes
from ..config.mefurax import MefuraxConfig, SlopedAttentionSizes
from ..config.registry import register_architecture
from ..parts import (AttentionNames, GatedMLP, GatedMLPNames, GQAttention, Linear, NoPosition, PairedRotaryPosition, RMSNorm, RoutedExperts,
                     SharedExpert, SumNormBlock, TokenEmbedding, ValueMixing)
from .decoder import DecoderModel

ATTENTION_NAMES = AttentionNames(qkv=("q", "k", "v"), out="o", q_norm="q.norm", k_norm="k.norm", gate="g", conv_suffix=".conv")
MLP_NAMES = GatedMLPNames(gate_up=("gate", "up"), down="down")
BLOCK_NAMES = ("mix", "norm1", "mlp", "norm2")
MODEL_NAMES = ("embed", "l", "final.norm")
HEAD_NAME = "head"
BIAS_SUFFIX = ".b"
NORM_OFFSET = 1.0           # the stream's norms' stored weights lie around zero
DENSE_ACTIVATION, EXPERT_ACTIVATION = "gelu_tanh", "relu2"      # fixed by the design
EXPERT_PIECES = ("up", "down")


def build_mefurax(config: MefuraxConfig) -> DecoderModel:
    eps, width = config.norm_eps, config.width

    def norm():
        return RMSNorm(width, eps, offset=NORM_OFFSET, tensor="")

    positions = {}
    mixing = [index for index, layer in enumerate(config.layers) if layer.mixer.v_mix]
    blocks = []
    for index, layer in enumerate(config.layers):
        sizes = layer.mixer
        common = dict(qk_norm_eps=eps, scale=sizes.scale, names=ATTENTION_NAMES, value_dim=sizes.vdim, bare_names=True,
                      value_mixing=ValueMixing(first=index == mixing[0]) if sizes.v_mix else None)
        if isinstance(sizes, SlopedAttentionSizes):
            mixer = GQAttention(width, sizes.heads, sizes.kv_heads, sizes.dim, NoPosition(), bias=True, out_bias=False, window=sizes.window,
                                bias_suffix=BIAS_SUFFIX, norm_span="projection", distance_bias=True, conv_taps=sizes.taps, **common)
        else:
            key = (sizes.rot_dims, sizes.rot_base)
            if key not in positions:
                positions[key] = PairedRotaryPosition(sizes.rot_dims, sizes.rot_base) if sizes.rot_dims else NoPosition()
            mixer = GQAttention(width, sizes.heads, sizes.kv_heads, sizes.dim, positions[key], norm_weights=False, softcap=sizes.softcap,
                                chunk=sizes.chunk, head_gate=True, **common)
        if layer.mlp is None:
            blocks.append(SumNormBlock(mixer, norm(), alpha=config.alpha, names=BLOCK_NAMES))
            continue
        if isinstance(layer.mlp, DenseSizes):
            feed = GatedMLP(width, layer.mlp.ff, DENSE_ACTIVATION, names=MLP_NAMES, bare_names=True)
        else:
            shared = SharedExpert(layer.mlp.shared, pieces=EXPERT_PIECES, gate=None) if layer.mlp.shared is not None else None
            feed = RoutedExperts(width, layer.mlp.ff, layer.mlp.experts, layer.mlp.top, pieces=EXPERT_PIECES, activation=EXPERT_ACTIVATION,
                                 shared=shared)
        blocks.append(SumNormBlock(mixer, norm(), feed, norm(), alpha=config.alpha, names=BLOCK_NAMES))
    head = Linear(width, (HEAD_NAME,), (config.vocab,), out_float32=True, bare_names=True)
    return DecoderModel(config, TokenEmbedding(config.vocab, width, tensor="", wide=True), blocks, norm(), head, tie_head=False,
                        names=MODEL_NAMES, layer_name=lambda i: f"l{i}")


register_architecture(MefuraxConfig.MODEL_TYPE, MefuraxConfig, build_mefurax, replace=True)
