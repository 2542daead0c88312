"""Typed configuration of the Pizunex decoder, read from config.json's own keys.

    {"architecture": "Pizunex", "vocab": V, "width": W, "norm": {"eps": e},
     "layers": [{"type": "delta" | "attention" | "latent_attention", "mixer": {...}, "mlp": {...} | null,
                 "weights_of": j}, ...]}

    mixer of "delta":             heads, kv_heads, dim, vdim, conv
    mixer of "attention":         heads, kv_heads, dim, vdim (= dim), scale, softcap, mask: {size}, q_temp: {coef, every}
    mixer of "latent_attention":  heads, dim, rot_dim, vdim, kv_rank, q_rank, scale,
                                  rot: {base, dims, scaling: {factor, original, fast, slow}}
    mlp:  {"kind": "dense", "ff"}

Every layer carries its own sizes; the list's order is the order in which the layers run.  A layer with `weights_of` has
no tensors of its own: it runs with those of the layer it names (whose entry is otherwise the same), on a cache or state
of its own.  Keys that a layer may do without: mask (every earlier key is seen), softcap (scores are not bounded), q_temp
(queries as they are), rot (nothing is turned), rot.scaling (the plain rates), q_rank (queries straight from the input).
"""
from __future__ import annotations

import json
import os
from dataclasses import dataclass
from typing import Optional

import numpy as np

from .errors import ConfigError
from .fields import obj as _obj, integer as _int, number as _num

LAYER_TYPES = ("delta", "attention", "latent_attention")


def _heads(d, where):
    heads, kv = _int(d, "heads", where), _int(d, "kv_heads", where)
    if heads % kv:
        raise ConfigError(f"{where}: {heads} heads do not divide into {kv} kv heads")
    return heads, kv


def _scale(d, where, size):
    return _num(d, "scale", where) if d.get("scale") is not None else float(size) ** -0.5


@dataclass(frozen=True)
class DeltaConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    conv: int                      # taps of the short convolutions

    @classmethod
    def from_dict(cls, d, where):
        heads, kv = _heads(d, where)
        return cls(heads, kv, _int(d, "dim", where), _int(d, "vdim", where), _int(d, "conv", where))

    def to_dict(self):
        return {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "conv": self.conv}


@dataclass(frozen=True)
class QueryTemperature:
    coef: float
    every: int

    @classmethod
    def from_dict(cls, d, where):
        return cls(_num(d, "coef", where), _int(d, "every", where))

    def to_dict(self):
        return {"coef": self.coef, "every": self.every}


@dataclass(frozen=True)
class AttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    scale: float
    softcap: Optional[float]
    window: Optional[int]          # mask.size; None: every earlier key
    q_temp: Optional[QueryTemperature]

    @property
    def vdim(self):
        return self.dim            # (the values are the keys as projected)

    @classmethod
    def from_dict(cls, d, where):
        heads, kv = _heads(d, where)
        dim = _int(d, "dim", where)
        if d.get("vdim") is not None and _int(d, "vdim", where) != dim:
            raise ConfigError(f"{where}: vdim {d['vdim']} for values that are the keys of {dim}")
        softcap = _num(d, "softcap", where) if d.get("softcap") is not None else None
        if softcap is not None and not softcap > 0.0:
            raise ConfigError(f"{where}: softcap {softcap} must be positive")
        return cls(heads, kv, dim, _scale(d, where, dim), softcap,
                   _int(_obj(d, "mask", where), "size", where + ".mask") if d.get("mask") is not None else None,
                   QueryTemperature.from_dict(_obj(d, "q_temp", where), where + ".q_temp") if d.get("q_temp") is not None else None)

    def to_dict(self):
        d = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.dim, "scale": self.scale}
        if self.softcap is not None:
            d["softcap"] = self.softcap
        if self.window is not None:
            d["mask"] = {"size": self.window}
        if self.q_temp is not None:
            d["q_temp"] = self.q_temp.to_dict()
        return d


@dataclass(frozen=True)
class RotationScaling:
    factor: float
    original: float
    fast: float
    slow: float

    @classmethod
    def from_dict(cls, d, where):
        c = cls(_num(d, "factor", where), _num(d, "original", where), _num(d, "fast", where), _num(d, "slow", where))
        if not (c.factor > 0.0 and c.original > 0.0 and c.fast > 0.0 and c.slow > 0.0):
            raise ConfigError(f"{where}: factor, original, fast and slow must be positive")
        return c

    def to_dict(self):
        return {"factor": self.factor, "original": self.original, "fast": self.fast, "slow": self.slow}


@dataclass(frozen=True)
class Rotation:
    base: float
    dims: int                      # 0: nothing is turned
    scaling: Optional[RotationScaling] = None

    @classmethod
    def from_dict(cls, d, where, most):
        if d.get("rot") is None:
            return cls(10000.0, 0)
        rot, at = _obj(d, "rot", where), where + ".rot"
        scaling = None
        if rot.get("scaling") is not None:
            scaling = RotationScaling.from_dict(_obj(rot, "scaling", at), at + ".scaling")
        c = cls(_num(rot, "base", at), _int(rot, "dims", at, 0), scaling)
        if c.dims % 2 or c.dims > most:
            raise ConfigError(f"{at}: dims {c.dims} must be even and at most {most}")
        if not c.base > 1.0:
            raise ConfigError(f"{at}: base {c.base} must be larger than 1")
        return c

    def to_dict(self):
        d = {"base": self.base, "dims": self.dims}
        if self.scaling is not None:
            d["scaling"] = self.scaling.to_dict()
        return d


@dataclass(frozen=True)
class LatentAttentionConfig:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    q_rank: Optional[int]          # None: queries straight from the mixer's input
    scale: float
    rot: Rotation

    @classmethod
    def from_dict(cls, d, where):
        dim, rot_dim = _int(d, "dim", where), _int(d, "rot_dim", where, 0)
        return cls(_int(d, "heads", where), dim, rot_dim, _int(d, "vdim", where), _int(d, "kv_rank", where),
                   _int(d, "q_rank", where) if d.get("q_rank") is not None else None, _scale(d, where, dim + rot_dim),
                   Rotation.from_dict(d, where, rot_dim))

    def to_dict(self):
        d = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "kv_rank": self.kv_rank,
             "scale": self.scale, "rot": self.rot.to_dict()}
        if self.q_rank is not None:
            d["q_rank"] = self.q_rank
        return d


MIXER_CONFIGS = {"delta": DeltaConfig, "attention": AttentionConfig, "latent_attention": LatentAttentionConfig}


@dataclass(frozen=True)
class DenseConfig:
    ff: int

    kind = "dense"

    @classmethod
    def from_dict(cls, d, where):
        if d.get("kind") != cls.kind:
            raise ConfigError(f"{where}: kind {d.get('kind')!r} (this decoder's feed-forwards are {cls.kind!r})")
        return cls(_int(d, "ff", where))

    def to_dict(self):
        return {"kind": self.kind, "ff": self.ff}


@dataclass(frozen=True)
class PizunexLayerConfig:
    type: str
    mixer: object
    mlp: Optional[DenseConfig]
    weights_of: Optional[int] = None     # the layer whose tensors this one runs with; None: its own

    @classmethod
    def from_dict(cls, d, where):
        kind = d.get("type") if isinstance(d, dict) else None
        if kind not in LAYER_TYPES:
            raise ConfigError(f"{where}: layer type {kind!r} (this decoder has {', '.join(LAYER_TYPES)})")
        mlp = DenseConfig.from_dict(_obj(d, "mlp", where), where + ".mlp") if d.get("mlp") is not None else None
        return cls(kind, MIXER_CONFIGS[kind].from_dict(_obj(d, "mixer", where), where + ".mixer"), mlp,
                   _int(d, "weights_of", where, 0) if d.get("weights_of") is not None else None)

    def to_dict(self):
        d = {"type": self.type, "mixer": self.mixer.to_dict(), "mlp": None if self.mlp is None else self.mlp.to_dict()}
        if self.weights_of is not None:
            d["weights_of"] = self.weights_of
        return d


@dataclass(frozen=True)
class PizunexConfig:
    vocab: int
    width: int
    layers: tuple
    norm_eps: float

    architecture = "Pizunex"
    max_position_embeddings = None    # the rotation's table bounds the positions (the mixers' position parts say how far)
    eos_token_id = None

    @classmethod
    def from_dict(cls, d: dict) -> "PizunexConfig":
        if not isinstance(d.get("layers"), list) or not d["layers"]:
            raise ConfigError("config key 'layers' must be a list with at least one layer")
        cfg = cls(_int(d, "vocab", "config"), _int(d, "width", "config"),
                  tuple(PizunexLayerConfig.from_dict(l, f"layers[{i}]") for i, l in enumerate(d["layers"])),
                  _num(_obj(d, "norm", "config"), "eps", "config.norm"))
        if not cfg.norm_eps > 0.0:
            raise ConfigError(f"norm.eps {cfg.norm_eps} must be positive")
        for i in range(len(cfg.layers)):
            cfg.weight_source(i)
        return cfg

    def weight_source(self, i: int) -> int:
        """The layer whose tensors layer i runs with: itself, or where its chain of `weights_of` ends.  Both entries name
        the same mixer and feed-forward."""
        at, seen = i, set()
        while self.layers[at].weights_of is not None:
            seen.add(at)
            src = self.layers[at].weights_of
            if not 0 <= src < len(self.layers) or src in seen:
                raise ConfigError(f"layers[{at}]: weights_of {src} must name another layer with tensors of its own")
            at = src
        a, b = self.layers[i], self.layers[at]
        if (a.type, a.mixer, a.mlp) != (b.type, b.mixer, b.mlp):
            raise ConfigError(f"layers[{i}]: weights_of {at} names a layer with another mixer or feed-forward")
        return at

    @classmethod
    def from_json(cls, path: str) -> "PizunexConfig":
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
        return {"architecture": self.architecture, "vocab": self.vocab, "width": self.width,
                "layers": [l.to_dict() for l in self.layers], "norm": {"eps": self.norm_eps}}

    @property
    def vocab_size(self) -> int:
        return self.vocab

    @property
    def eps_f32(self) -> float:
        return float(np.float32(self.norm_eps))

    @property
    def stop_token_ids(self) -> tuple:
        return ()
