"""The Pizunex decoder put together from parts, and its entry in the registry.

Every layer is a pre-norm layer with RMSNorms (parts.PreNormBlock): x <- x + mixer(norm1(x)); x <- x + ff(norm2(x)), the
second half only where the layer has a feed-forward.  The mixer is one of three, chosen by the layer's type: "delta": the
delta rule with one decay a head behind short convolutions (parts.HeadDeltaMixer); "attention": grouped-query attention
over a sliding window whose values are the keys as projected, with norms over the whole query and key projections, a
temperature on the queries that grows with the position, a soft cap and then a linear distance bias on the scores
(parts.GatedWindowAttention); "latent_attention": keys and values of all heads from one normed latent a token beside one
turned key part, queries through a normed latent of their own, a rotation in pairs whose long waves are stretched
(parts.LatentAttention).  The feed-forward squares the relu of one product (parts.UngatedMlp).  A layer may run with the
tensors of another one: it is then a second run of that layer's block on a cache of its own.
Tensor names: embed; l<i>.norm1|norm2; l<i>.mix.*; l<i>.mlp.up|down; final.norm; head.
"""
from __future__ import annotations

from ..config.pizunex import PizunexConfig
from ..config.registry import register_architecture
from ..parts import (RmsNorm, NoPosition, RotaryScaledInterleaved, LinearDistanceBias, HeadDeltaMixer, GatedWindowAttention,
                     LatentAttention, UngatedMlp, PreNormBlock)
from .decoder import DecoderModel, LayerRun, TokenEmbedding, OutputHead

DEFAULT_POSITIONS = 1 << 16      # rows of the rotation's tables when the caller names no longest sequence


def _rotation(rot, capacity):
    if rot.dims == 0:
        return NoPosition()
    sc = rot.scaling
    return RotaryScaledInterleaved(rot.base, rot.dims, capacity,
                                   **({} if sc is None else dict(factor=sc.factor, original=sc.original, fast=sc.fast,
                                                                 slow=sc.slow)))


def _mixer(layer, p, W, eps, capacity):
    m = layer.mixer
    if layer.type == "delta":
        return HeadDeltaMixer(p, W, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, norm_eps=eps)
    if layer.type == "latent_attention":
        return LatentAttention(p, W, m.heads, m.dim, m.rot_dim, m.vdim, m.kv_rank, position=_rotation(m.rot, capacity),
                               norm_eps=eps, scale=m.scale, q_rank=m.q_rank)
    return GatedWindowAttention(p, W, m.heads, m.kv_heads, m.dim, position=LinearDistanceBias(), qk_norm_eps=eps,
                                qk_norm_whole=True, values_are_keys=True, scale=m.scale, score_softcap=m.softcap,
                                window=m.window, q_temp=None if m.q_temp is None else (m.q_temp.coef, m.q_temp.every))


def build_pizunex(cfg: PizunexConfig, max_positions: int | None = None) -> DecoderModel:
    W, eps = cfg.width, cfg.eps_f32
    capacity = max_positions or DEFAULT_POSITIONS
    blocks, block_of = [], {}
    for i, layer in enumerate(cfg.layers):
        if layer.weights_of is not None:
            continue
        p = f"l{i}."
        norm2 = ff = None
        if layer.mlp is not None:
            norm2, ff = RmsNorm(p + "norm2", W, eps), UngatedMlp(p + "mlp.", W, layer.mlp.ff, "relu_squared")
        block_of[i] = len(blocks)
        blocks.append(PreNormBlock(RmsNorm(p + "norm1", W, eps), _mixer(layer, p + "mix.", W, eps, capacity), norm2, ff))
    schedule = [LayerRun(block_of[cfg.weight_source(i)], i) for i in range(len(cfg.layers))]
    embedding = TokenEmbedding("embed", cfg.vocab, W)
    return DecoderModel(cfg, embedding, blocks, schedule, RmsNorm("final.norm", W, eps), OutputHead("head", cfg.vocab, W))


PIZUNEX = register_architecture("Pizunex", PizunexConfig, build_pizunex, model_types=("pizunex",))
