"""The Sunosun decoder put together from parts, and its entry in the registry.

Every layer is a pre-norm layer with RMSNorms (parts.PreNormBlock): x <- x + mixer(norm1(x)); x <- x + ff(norm2(x)), the
second half only where the layer has a feed-forward.  The mixer is one of two, chosen by the layer's type: "gla": gated
linear attention with a decay for every key channel (parts.GatedLinearAttention); "parallel": the scaled sum of
grouped-query attention over all earlier keys, with biases, without positions and with one added to the softmax's denominator
(parts.GatedWindowAttention), and of gated linear attention, which share their input and output products
(parts.ParallelMixers).  The feed-forward is silu-gated (parts.GatedMlp) or a mixture of experts that square the relu of one
product, behind a router that scores every expert by itself, picks within the groups whose two best experts score best and
divides the weights by their sum, beside one expert that every token passes through a gate of its own (parts.RoutedExperts).
Some layers in a row may run several times with the same weights, each pass on caches and states of its own; before a pass a
vector of its own and, but for the first, the embedding's output are added to the residual (models.decoder.LoopInputs).
The embedding is scaled and gets sinusoidal positions; RMSNorm, the embedding table as the output matrix, and a soft cap on
the logits at the end.
Tensor names: embed; loop.step; l<i>.norm1|norm2; l<i>.mix.*, in parallel layers l<i>.mix.left.*, l<i>.mix.right.*;
l<i>.mlp.gate|up|down; l<i>.mlp.e<j>.up|down, l<i>.mlp.router|correction, l<i>.mlp.shared.up|down|sg; final.norm.
"""
from __future__ import annotations

from ..config.registry import register_architecture
from ..config.sunosun import SunosunConfig
from ..parts import (RmsNorm, GatedWindowAttention, GatedLinearAttention, ParallelMixers, GatedMlp, UngatedMlp, RoutedExperts,
                     PreNormBlock)
from .decoder import DecoderModel, LayerRun, LoopInputs, TokenEmbedding, OutputHead

SINUSOID_BASE = 10000.0
WEIGHTS_EPS = 1e-20            # beside the sum that the chosen experts' scores are divided by


def _gla(p, W, m, eps, rank):
    mixer = GatedLinearAttention(p, W, m.heads, m.dim, m.vdim, m.tau, norm_eps=eps)
    if rank is not None:
        mixer.set_rank(rank)
    return mixer


def _mixer(layer, p, W, eps, rank):
    m = layer.mixer
    if layer.type == "gla":
        return _gla(p, W, m, eps, rank)
    a = m.left
    left = GatedWindowAttention(p + "left.", W, a.heads, a.kv_heads, a.dim, a.vdim, scale=a.scale, sink_one=True, bias=True)
    return ParallelMixers([left, _gla(p + "right.", W, m.right, eps, rank)], [m.left_scale, m.right_scale])


def _feed_forward(p, W, c):
    if c.kind == "dense":
        return GatedMlp(p, W, c.ff, "silu", names=("gate", "up", "down"))
    shared = None if c.shared_ff is None else UngatedMlp(p + "shared.", W, c.shared_ff, "relu_squared")
    return RoutedExperts(p, W, c.ff, c.experts, c.top, "relu_squared", router="scores", score="sigmoid", group_score="two",
                         n_groups=c.groups, keep_groups=c.keep_groups, renorm=True, renorm_eps=WEIGHTS_EPS,
                         route_scale=c.route_scale, shared=shared, shared_gate=None if shared is None else "shared.sg")


def build_sunosun(cfg: SunosunConfig, max_positions: int | None = None) -> DecoderModel:
    W, eps = cfg.width, cfg.eps_f32
    blocks = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        norm2 = ff = None
        if layer.mlp is not None:
            norm2, ff = RmsNorm(p + "norm2", W, eps), _feed_forward(p + "mlp.", W, layer.mlp)
        blocks.append(PreNormBlock(RmsNorm(p + "norm1", W, eps), _mixer(layer, p + "mix.", W, eps, cfg.middle_rank), norm2, ff))
    schedule = [LayerRun(i, c, opens) for c, (i, opens) in enumerate(cfg.runs())]
    loop = None if cfg.loop is None else LoopInputs("loop.step", cfg.loop.times, W)
    embedding = TokenEmbedding("embed", cfg.vocab, W, scale=cfg.embedding_scale, sinusoid_base=SINUSOID_BASE)
    head = OutputHead("head", cfg.vocab, W, tied_to=embedding, softcap=cfg.logit_softcap)
    return DecoderModel(cfg, embedding, blocks, schedule, RmsNorm("final.norm", W, eps), head, loop=loop)


SUNOSUN = register_architecture("Sunosun", SunosunConfig, build_sunosun, model_types=("sunosun",))
