"""Typed configuration of the Sunosun decoder, read from config.json's own keys.

    {"architecture": "Sunosun", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s}, "logit_softcap": c,
     "loop": {"start": a, "stop": b, "times": n},
     "layers": [{"type": "gla" | "parallel", "mixer": {...}, "mlp": {...} | null}, ...]}

    mixer of "gla":       heads, dim, vdim, tau
    mixer of "parallel":  left: {heads, kv_heads, dim, vdim, scale}, right: the keys of "gla", left_scale, right_scale
    mlp:  {"kind": "dense", "ff"}  or
          {"kind": "moe", "expert": {"ff"}, "router": {"experts", "top", "scale", "groups": {"count", "keep"}}, "shared": {"ff"}}

Every layer carries its own sizes; the list's order is the order in which the layers run, and the layers a .. b - 1 of `loop`
run n times in a row.  Keys that a model may do without: loop (every layer runs once), embedding (a scale of 1),
logit_softcap (logits as they are), left.scale (dim^-1/2), left_scale and right_scale (1), router.scale (1), router.groups (one
group), shared (no expert that every token passes).
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Optional

import numpy as np

from .errors import ConfigError
from .fields import obj as _obj, integer as _int, number as _num

LAYER_TYPES = ("gla", "parallel")


def _or(d, key, where, default):
    return _num(d, key, where) if d.get(key) is not None else default


@dataclass(frozen=True)
class GlaConfig:
    heads: int
    dim: int
    vdim: int
    tau: float                     # decays are sigmoid(z)^(1 / tau)

    @classmethod
    def from_dict(cls, d, where):
        c = cls(_int(d, "heads", where), _int(d, "dim", where), _int(d, "vdim", where), _num(d, "tau", where))
        if not c.tau > 0.0:
            raise ConfigError(f"{where}: tau {c.tau} must be positive")
        return c

    def to_dict(self):
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float

    @classmethod
    def from_dict(cls, d, where):
        heads, kv, dim = _int(d, "heads", where), _int(d, "kv_heads", where), _int(d, "dim", where)
        if heads % kv:
            raise ConfigError(f"{where}: {heads} heads do not divide into {kv} kv heads")
        return cls(heads, kv, dim, _int(d, "vdim", where), _or(d, "scale", where, float(dim) ** -0.5))

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}


@dataclass(frozen=True)
class ParallelConfig:
    left: AttentionConfig
    right: GlaConfig
    left_scale: float
    right_scale: float

    @classmethod
    def from_dict(cls, d, where):
        return cls(AttentionConfig.from_dict(_obj(d, "left", where), where + ".left"),
                   GlaConfig.from_dict(_obj(d, "right", where), where + ".right"),
                   _or(d, "left_scale", where, 1.0), _or(d, "right_scale", where, 1.0))

    def to_dict(self):
        return {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                "right_scale": self.right_scale}


MIXER_CONFIGS = {"gla": GlaConfig, "parallel": ParallelConfig}


@dataclass(frozen=True)
class DenseConfig:
    ff: int

    kind = "dense"

    @classmethod
    def from_dict(cls, d, where):
        return cls(_int(d, "ff", where))

    def to_dict(self):
        return {"kind": self.kind, "ff": self.ff}


@dataclass(frozen=True)
class MoeConfig:
    ff: int                        # of each routed expert
    experts: int
    top: int
    groups: int
    keep_groups: int
    route_scale: float
    shared_ff: Optional[int]       # None: no expert that every token passes

    kind = "moe"

    @classmethod
    def from_dict(cls, d, where):
        router, at = _obj(d, "router", where), where + ".router"
        count = keep = 1
        if router.get("groups") is not None:
            groups = _obj(router, "groups", at)
            count, keep = _int(groups, "count", at + ".groups"), _int(groups, "keep", at + ".groups")
        c = cls(_int(_obj(d, "expert", where), "ff", where + ".expert"), _int(router, "experts", at), _int(router, "top", at),
                count, keep, _or(router, "scale", at, 1.0),
                _int(_obj(d, "shared", where), "ff", where + ".shared") if d.get("shared") is not None else None)
        if c.experts % c.groups or c.keep_groups > c.groups:
            raise ConfigError(f"{at}: {c.experts} experts in {c.groups} groups of which {c.keep_groups} stay")
        if c.top > c.keep_groups * (c.experts // c.groups):
            raise ConfigError(f"{at}: top {c.top} of {c.keep_groups} groups of {c.experts // c.groups}")
        return c

    def to_dict(self):
        d = {"kind": self.kind, "expert": {"ff": self.ff},
             "router": {"experts": self.experts, "top": self.top, "scale": self.route_scale,
                        "groups": {"count": self.groups, "keep": self.keep_groups}}}
        if self.shared_ff is not None:
            d["shared"] = {"ff": self.shared_ff}
        return d


MLP_CONFIGS = {"dense": DenseConfig, "moe": MoeConfig}


@dataclass(frozen=True)
class SunosunLayerConfig:
    type: str
    mixer: object
    mlp: object                    # DenseConfig, MoeConfig or None

    @classmethod
    def from_dict(cls, d, where):
        kind = d.get("type") if isinstance(d, dict) else None
        if kind not in LAYER_TYPES:
            raise ConfigError(f"{where}: layer type {kind!r} (this decoder has {', '.join(LAYER_TYPES)})")
        mlp = None
        if d.get("mlp") is not None:
            m = _obj(d, "mlp", where)
            if m.get("kind") not in MLP_CONFIGS:
                raise ConfigError(f"{where}.mlp: kind {m.get('kind')!r} (one of {', '.join(MLP_CONFIGS)})")
            mlp = MLP_CONFIGS[m["kind"]].from_dict(m, where + ".mlp")
        return cls(kind, MIXER_CONFIGS[kind].from_dict(_obj(d, "mixer", where), where + ".mixer"), mlp)

    def to_dict(self):
        return {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}


@dataclass(frozen=True)
class LoopConfig:
    start: int
    stop: int
    times: int

    @classmethod
    def from_dict(cls, d, where, n_layers):
        c = cls(_int(d, "start", where, 0), _int(d, "stop", where), _int(d, "times", where))
        if not c.start < c.stop <= n_layers:
            raise ConfigError(f"{where}: layers {c.start} .. {c.stop - 1} of {n_layers}")
        return c

    def to_dict(self):
        return {"start": self.start, "stop": self.stop, "times": self.times}


@dataclass(frozen=True)
class SunosunConfig:
    vocab: int
    width: int
    layers: tuple
    norm_eps: float
    embedding_scale: float = 1.0
    logit_softcap: Optional[float] = None     # None: logits as they are
    loop: Optional[LoopConfig] = None
    # size of the narrow middle in front of the decays for random weights (stored weights bring their own, and no key of
    # config.json names it); written out only when it was set
    middle_rank: Optional[int] = None

    architecture = "Sunosun"
    max_position_embeddings = None    # positions enter by a formula: any number of them
    eos_token_id = None

    @classmethod
    def from_dict(cls, d: dict) -> "SunosunConfig":
        if not isinstance(d.get("layers"), list) or not d["layers"]:
            raise ConfigError("config key 'layers' must be a list with at least one layer")
        layers = tuple(SunosunLayerConfig.from_dict(l, f"layers[{i}]") for i, l in enumerate(d["layers"]))
        scale = 1.0
        if d.get("embedding") is not None:
            scale = _or(_obj(d, "embedding", "config"), "scale", "config.embedding", 1.0)
        cap = _or(d, "logit_softcap", "config", None)
        if cap is not None and not cap > 0.0:
            raise ConfigError(f"logit_softcap {cap} must be positive")
        loop = LoopConfig.from_dict(_obj(d, "loop", "config"), "config.loop", len(layers)) if d.get("loop") is not None else None
        cfg = cls(_int(d, "vocab", "config"), _int(d, "width", "config"), layers,
                  _num(_obj(d, "norm", "config"), "eps", "config.norm"), scale, cap, loop,
                  _int(d, "middle_rank", "config") if d.get("middle_rank") is not None else None)
        if not cfg.norm_eps > 0.0:
            raise ConfigError(f"norm.eps {cfg.norm_eps} must be positive")
        return cfg

    def runs(self) -> list:
        """The layers in the order they run, as (layer, opens): `opens` is the number of the looped layers' pass that the run
        opens, or None."""
        n, loop = len(self.layers), self.loop
        if loop is None:
            return [(i, None) for i in range(n)]
        looped = [(i, t if i == loop.start else None) for t in range(loop.times) for i in range(loop.start, loop.stop)]
        return [(i, None) for i in range(loop.start)] + looped + [(i, None) for i in range(loop.stop, n)]

    @classmethod
    def from_json(cls, path: str) -> "SunosunConfig":
        if os.path.isdir(path):
            path = os.path.join(path, "config.json")
        try:
            with open(path) as f:
                d = json.load(f)
        except OSError as e:
            raise ConfigError(f"read {path}: {e}") from None
        except json.JSONDecodeError as e:
            raise ConfigError(f"parse {path}: {e}") from None
        if not isinstance(d, dict):
            raise ConfigError(f"parse {path}: top level is not an object")
        return cls.from_dict(d)

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
             "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.norm_eps},
             "embedding": {"scale": self.embedding_scale}}
        if self.logit_softcap is not None:
            d["logit_softcap"] = self.logit_softcap
        if self.loop is not None:
            d["loop"] = self.loop.to_dict()
        if self.middle_rank is not None:
            d["middle_rank"] = self.middle_rank
        return d

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def eps_f32(self) -> float:
        return float(np.float32(self.norm_eps))

    @property
    def stop_token_ids(self) -> tuple:
        return ()
