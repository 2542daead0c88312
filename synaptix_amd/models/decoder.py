"""A decoder as data: an embedding, a list of blocks, the order in which they run, a final norm
and an output head.

The order is a list of LayerRun(block, cache): it may name a block twice (its weights are then
used twice, each run with a cache of its own), or give two runs the same cache index (the first
run that names a cache writes it, the later ones only read it).  Which mixer, feed-forward and
norm a block has is decided layer by layer by whoever builds the list of blocks.

Forward of one step, as crates/synaptix-models/llm/common/src/model.rs:1052-1105,1160-1262:
embedding (no scale), the runs in order, final norm on the wanted rows only, output product in
float.  The reference norms every row and keeps the last (1068-1074); gathering first is the
same arithmetic on fewer rows.
"""
from __future__ import annotations

import math
from dataclasses import dataclass

import torch

from ..kernels import ops
from ..parts.base import Part
from ..parts.linear import Matrix, linear, as_delta, as_rows, InjectedDelta
from ..weights.source import TensorSpec


@dataclass(frozen=True)
class LayerRun:
    block: int     # index into DecoderModel.blocks
    cache: int     # index of the cache layer it uses
    opens: int | None = None     # the pass of the looped layers (LoopInputs) that this run opens


class TokenEmbedding(Part):
    """x[n, :] = scale * E[id[n], :] (crates/synaptix-ops/src/embed/token_embed.rs:4-15; the reference has no scale).
    sinusoid_base: a sinusoidal vector of the token's position p is added, with f_i = base^(-2 i / hidden) sin(p f_i) at
    column 2 i and cos(p f_i) at column 2 i + 1 (None: none)."""
    capturable = True

    def __init__(self, name: str, vocab: int, hidden: int, scale: float = 1.0, sinusoid_base: float | None = None):
        self.name, self.vocab, self.hidden, self.scale = name, vocab, hidden, float(scale)
        self.sinusoid_base = sinusoid_base
        self.table = self.rates = None

    def tensor_specs(self):
        return {self.name: TensorSpec((self.vocab, self.hidden), "table")}

    def load(self, get):
        self.table = Matrix(get(self.name))       # (a tied output head multiplies with the same matrix)
        if self.sinusoid_base is not None:
            i = torch.arange((self.hidden + 1) // 2, dtype=torch.float64)
            # (in turns a position)
            self.rates = (float(self.sinusoid_base) ** (-2.0 * i / self.hidden) / (2.0 * math.pi)).to(self.table.device)

    def forward(self, ids, positions=None, keep=None):
        """positions [N] int32: of the rows' tokens (read with sinusoid_base); keep [N, hidden] float: gets the rows too."""
        resid = torch.empty((ids.shape[0], self.hidden), dtype=torch.float32, device=ids.device)
        if self.rates is not None or keep is not None:
            ops.embed(self.table.data, ids, resid, self.scale,
                      sinusoid=None if self.rates is None else (self.rates, positions), keep=keep)
        elif self.scale == 1.0:
            ops.embed(self.table.data, ids, resid)
        else:
            ops.embed(self.table.data, ids, resid, self.scale)
        return resid


class LoopInputs(Part):
    """What layers that run several times in a row get before each pass t = 0, 1, ...: the vector `name`[t] ([times, hidden]),
    and before every pass but the first the embedding's output once more.  A run of the schedule that opens a pass says so
    (LayerRun.opens); its first norm adds both (parts.linear.InjectedDelta)."""
    capturable = True

    def __init__(self, name: str, times: int, hidden: int):
        self.name, self.times, self.hidden = name, int(times), hidden
        self.steps = None

    def tensor_specs(self):
        return {self.name: TensorSpec((self.times, self.hidden), "bias")}

    def load(self, get):
        self.steps = get(self.name).float().contiguous()

    def add_to(self, pending, t, resid, embedded):
        return InjectedDelta(pending, embedded if t > 0 else None, self.steps[t], resid.shape)


class OutputHead(Part):
    """logits = h . W^T in float; tied: W is the embedding table
    (crates/synaptix-models/llm/common/src/model.rs:757-764).  softcap: logits <- cap tanh(logits / cap)."""
    capturable = True

    def __init__(self, name: str, vocab: int, hidden: int, tied_to: TokenEmbedding | None = None,
                 softcap: float | None = None):
        self.point = ("softcap", float(softcap)) if softcap else None
        self.name, self.vocab, self.hidden, self.tied_to = name, vocab, hidden, tied_to
        self.weight = None

    def tensor_specs(self):
        return {} if self.tied_to is not None else {self.name: TensorSpec((self.vocab, self.hidden))}

    def ignored_tensors(self):
        # a tied checkpoint may still carry the matrix; it is not read
        return [self.name] if self.tied_to is not None else []

    def load(self, get):
        self.weight = self.tied_to.table if self.tied_to is not None else Matrix(get(self.name))

    def forward(self, h):
        return linear(h, self.weight, torch.float32, point=self.point)


class DecoderModel:
    def __init__(self, config, embedding: TokenEmbedding, blocks: list, schedule: list, final_norm, head: OutputHead,
                 streams: int | None = None, loop: LoopInputs | None = None):
        """loop: what the runs that open a pass of looped layers add to the residual.  streams: the residual runs in this many copies [N, streams, hidden] that all start as the embedding
        (blocks that read and write them: parts.HyperConnectionBlock; the final norm gets their sum); None: one
        plain residual [N, hidden]."""
        self.config = config
        self.streams, self.loop = streams, loop
        self.embedding, self.blocks, self.schedule = embedding, list(blocks), list(schedule)
        self.final_norm, self.head = final_norm, head
        self.vocab, self.hidden = embedding.vocab, embedding.hidden
        self.act_dtype = None
        self.device = None
        for run in self.schedule:
            if not (0 <= run.block < len(self.blocks)):
                raise ValueError(f"schedule names block {run.block}; there are {len(self.blocks)}")
            if run.opens is not None and (loop is None or streams is not None or not 0 <= run.opens < loop.times):
                raise ValueError(f"a run that opens pass {run.opens} of looped layers without inputs for it")
        # the first run that names a cache owns (writes) it
        seen, self._owner = set(), []
        for run in self.schedule:
            self._owner.append(run.cache not in seen)
            seen.add(run.cache)
        if seen and seen != set(range(len(seen))):
            raise ValueError("cache indices of the schedule must be 0 .. n-1 without gaps")
        self.n_caches = len(seen)

    # ------------------------------------------------------------------ weights
    def _parts(self):
        return [self.embedding] + self.blocks + [self.final_norm, self.head] + ([] if self.loop is None else [self.loop])

    def tensor_specs(self) -> dict:
        specs = {}
        for p in self._parts():
            for n, s in p.tensor_specs().items():
                if n in specs and specs[n] != s:
                    raise ValueError(f"tensor {n} is declared twice with different shapes")
                specs[n] = s
        return specs

    def ignored_tensors(self) -> list:
        return self.head.ignored_tensors()

    def load(self, get) -> None:
        for p in self._parts():
            p.load(get)
        self.device = self.embedding.table.device

    def check(self, dtype) -> None:
        """Every part is asked whether its kernels take its sizes in `dtype`."""
        for p in self._parts():
            p.check(dtype)

    def capturable(self) -> bool:
        """Whether a step of this model may be captured into a graph: every part says so of itself."""
        return all(getattr(p, "capturable", False) for p in self._parts())

    # ------------------------------------------------------------------ cache
    def cache_needs(self) -> list:
        """Need of each cache layer, from the mixer of the run that owns it."""
        needs = [None] * self.n_caches
        for run, owner in zip(self.schedule, self._owner):
            need = self.blocks[run.block].mixer.cache_need()
            if owner:
                needs[run.cache] = need
            elif needs[run.cache] != need:
                raise ValueError(f"block {run.block} reads cache {run.cache} but needs {need}, "
                                 f"its owner keeps {needs[run.cache]}")
        return needs

    # ------------------------------------------------------------------ one step
    def forward(self, ctx, tokens, want_rows, cache) -> torch.Tensor:
        """tokens [N] int32 and want_rows [n] int32 (or None) on the device; returns logits [n, vocab] float."""
        with ops.stream_scope():     # one stream for the whole pass, asked for once
            embedded = None
            if any(run.opens for run in self.schedule):       # (a pass behind the first: the embedding's output once more)
                embedded = torch.empty((tokens.shape[0], self.hidden), dtype=torch.float32, device=tokens.device)
            if embedded is None and getattr(self.embedding, "rates", None) is None:
                resid = self.embedding.forward(tokens)
            else:
                resid = self.embedding.forward(tokens, ctx.tok_pos, embedded)
            if self.streams is not None:
                x0, resid = resid, torch.empty((tokens.shape[0], self.streams, self.hidden), dtype=torch.float32,
                                               device=tokens.device)
                ops.streams_start(x0, resid)
            pending = None
            for run, owner in zip(self.schedule, self._owner):
                block = self.blocks[run.block]
                if run.opens is not None:
                    pending = self.loop.add_to(pending, run.opens, resid, embedded)
                if not block.takes_deferred_product:
                    pending = as_delta(pending)      # a product that the last block left for a norm to take in
                pending = block.forward(resid, pending, ctx, cache.layer_view(run.cache), owner)
            if want_rows is None:
                return None          # nothing is asked for: the cache has been written, that is all
            if not getattr(self.final_norm, "takes_deferred_product", False):
                pending = as_delta(pending)
            h = self.final_norm.add_apply(resid, pending, ctx.act_dtype, rows=want_rows)
            return self.head.forward(as_rows(h))
