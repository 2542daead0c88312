"""Small Pizunex configurations for the tests, their model folders (random weights), and the plain model's logits."""
from __future__ import annotations

import copy
import os
import tempfile

import torch

from synaptix_amd.config import PizunexConfig
from synaptix_amd import write_random_model
from plain_pizunex import PlainPizunex


def delta(heads, kv_heads, dim, vdim, conv):
    return "delta", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def attention(heads, kv_heads, dim, window=None, softcap=None, q_temp=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale if scale is not None else 4.0 * dim ** -0.5}
    if window is not None:
        m["mask"] = {"size": window}
    if softcap is not None:
        m["softcap"] = softcap
    if q_temp is not None:
        m["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return "attention", m


def latent(heads, dim, rot_dim, vdim, rank, q_rank=None, base=10000.0, scaling=None, scale=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank,
         "scale": scale if scale is not None else 6.0 * (dim + rot_dim) ** -0.5, "rot": {"base": base, "dims": rot_dim}}
    if q_rank is not None:
        m["q_rank"] = q_rank
    if scaling is not None:
        m["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return "latent_attention", m


def config(vocab, width, layers, eps=1e-6):
    """layers: (mixer, feed-forward's width or None), or the index of the earlier or later layer whose tensors it uses."""
    out = []
    for l in layers:
        if isinstance(l, int):
            out.append(l)
        else:
            (kind, m), ff = l
            out.append({"type": kind, "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff}})
    for i, l in enumerate(out):
        if isinstance(l, int):
            src = out[l]
            while isinstance(src, int):
                src = out[src]
            out[i] = dict(copy.deepcopy({k: src[k] for k in ("type", "mixer", "mlp")}), weights_of=l)
    return {"architecture": "Pizunex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": out}


# P: the three mixers in an order of their own, a window shorter than a page, value heads that share key heads, a
#    temperature that steps inside every test sequence, a cap that bites, stretched long waves, layers with and without a
#    feed-forward, and second runs of an attention layer, a delta layer and the latent layer, each on a cache of its own.
# Q: sizes that are multiples of nothing (a width of 72, keys of 10 and 12, a latent of 20 beside 6 turned values, an odd
#    vocabulary), one key head, no window, no cap, no temperature, plain rates, queries without a latent, one tap, a query
#    latent wider than the width.
# R: sizes at which the products and prompts' attention run on the matrix cores; a window of a page and a token, a window
#    that no test sequence outgrows; as many key heads as heads; two layers that run three times.
# S: one head everywhere, windows of one and of two, a temperature that steps at every position, a chain of three layers
#    that share tensors (one names a layer that comes later).
# T: delta layers alone: a model without keys and values.
# U: windows and delta layers only, so that every cache group gives its pages back.
CONFIGS = {
    "P": config(300, 64, [(attention(4, 2, 16, window=20, softcap=8.0, q_temp=(0.5, 16)), 48),
                          (delta(6, 2, 16, 24, 4), None),
                          (latent(4, 8, 8, 12, 32, q_rank=24, base=500.0, scaling=(4.0, 64, 8.0, 1.0)), 80),
                          0, 1, 2,
                          (delta(3, 3, 8, 20, 3), 36)]),
    "Q": config(257, 72, [(delta(4, 1, 12, 18, 1), 50),
                          (attention(3, 1, 10), 30),
                          (latent(5, 6, 2, 4, 9), None),
                          (latent(3, 10, 6, 14, 20, q_rank=90, base=300.0), 44),
                          (attention(2, 2, 14, window=65, q_temp=(1.5, 50)), None),
                          (delta(5, 5, 7, 6, 6), None), 5], eps=1e-5),
    "R": config(512, 128, [(delta(8, 4, 32, 64, 4), None),
                           (attention(8, 8, 64, window=65, softcap=30.0, q_temp=(0.3, 32)), 256),
                           (latent(4, 32, 16, 32, 64, q_rank=128, base=1e6, scaling=(8.0, 128, 16.0, 1.0)), 256),
                           (attention(4, 1, 48, window=4096, softcap=12.0), 128),
                           1, (delta(4, 4, 64, 32, 5), 128), 0, 1]),
    "S": config(101, 40, [(attention(1, 1, 8, window=1, q_temp=(2.0, 1)), 16),
                          3,
                          (latent(1, 4, 2, 6, 5, q_rank=3), 24),
                          (delta(1, 1, 6, 5, 2), None),
                          1, (attention(1, 1, 6, window=2, softcap=1.0, q_temp=(0.7, 3)), None)]),
    "T": config(160, 96, [(delta(4, 2, 24, 32, 4), 64), (delta(2, 1, 40, 16, 7), None), 0]),
    "U": config(200, 64, [(attention(4, 2, 16, window=70, softcap=20.0, q_temp=(0.2, 100)), 32),
                          (delta(2, 2, 16, 16, 4), None), (attention(2, 1, 32, window=9), None), 0]),
}
SEEDS = {"P": 51, "Q": 52, "R": 53, "S": 54, "T": 55, "U": 56}

_tmp = None
_folders, _plain, _logits = {}, {}, {}


def _extra(cfg, g):
    """Decays between 0.9 and 0.999 a token, so that what was written a hundred tokens ago still counts."""
    extra = {}
    for i, l in enumerate(cfg.layers):
        if l.type == "delta" and l.weights_of is None:
            extra[f"l{i}.mix.A_log"] = (-4.0 + torch.randn(l.mixer.heads, generator=g)).to(torch.bfloat16)
    return extra


def _write(folder, cfg, seed, std):
    g = torch.Generator().manual_seed(700 + seed)
    write_random_model(folder, cfg, seed, std=std, gain_std=0.3, extra_tensors=_extra(cfg, g))


def _temporary():
    global _tmp
    if _tmp is None:
        _tmp = tempfile.TemporaryDirectory(prefix="synaptix_amd_pizunex_")
    return _tmp.name


def model_folder(name: str) -> str:
    """Random bf16 weights, drawn wide enough that every branch carries weight; the configurations' scales make the
    attention peaked, so that a lost or wrong key moves the logits."""
    if name not in _folders:
        folder = os.path.join(_temporary(), name)
        _write(folder, PizunexConfig.from_dict(copy.deepcopy(CONFIGS[name])), SEEDS[name], 0.08)
        _folders[name] = folder
    return _folders[name]


def plain_model(name: str) -> PlainPizunex:
    if name not in _plain:
        _plain[name] = PlainPizunex.from_folder(model_folder(name))
    return _plain[name]


def plain_logits(name: str, tokens) -> torch.Tensor:
    key = (name, tuple(tokens))
    if key not in _logits:
        _logits[key] = plain_model(name).logits(list(tokens))
    return _logits[key]


def tokens_for(name: str, n: int, seed: int) -> list:
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


def random_config(seed: int) -> dict:
    """A configuration drawn from a seed: layer kinds in any order, head counts, sizes (multiples of sixteen and not),
    windows from one position to none, every optional mechanism on or off, layers with other layers' tensors."""
    import random
    rng = random.Random(seed)
    width, vocab = rng.choice([64, 96, 128, 192, 256, 80]), rng.choice([200, 384, 512, 1000, 333])
    layers, owners = [], []
    for i in range(rng.randint(2, 7)):
        if owners and rng.random() < 0.35:
            layers.append(rng.choice(owners))
            continue
        owners.append(i)
        kind = rng.choice(["delta", "attention", "latent"])
        heads = rng.choice([1, 2, 3, 4, 6, 8, 12])
        kv = rng.choice([h for h in (1, 2, 3, 4, 6, 8, 12) if heads % h == 0])
        if kind == "delta":
            mixer = delta(heads, kv, rng.choice([8, 16, 24, 32, 48, 64, 96, 128]), rng.choice([8, 16, 24, 32, 64, 96, 128, 40]),
                          rng.choice([1, 2, 3, 4, 5, 8]))
        elif kind == "attention":
            dim = rng.choice([16, 32, 48, 64, 96, 128, 160, 24, 40])
            mixer = attention(heads, kv, dim, window=rng.choice([None, 1, 7, 16, 31, 64, 65, 100, 128, 200]),
                              softcap=rng.choice([None, 5.0, 15.0, 50.0]), scale=2.0 * dim ** -0.5,
                              q_temp=rng.choice([None, (0.1, 64), (0.5, 20), (1.0, 7), (0.3, 1000)]))
        else:
            rot, nope = rng.choice([2, 8, 16, 32, 64]), rng.choice([8, 16, 32, 64, 24])
            mixer = latent(heads, nope, rot, rng.choice([16, 32, 48, 64, 40]), rng.choice([16, 32, 64, 128, 96, 40, 256]),
                           q_rank=rng.choice([None, 24, 48, 64, 128, 160]), base=rng.choice([1e4, 5e5, 100.0]),
                           scaling=rng.choice([None, (4.0, 64, 32.0, 1.0), (2.0, 4096, 32.0, 1.0), (40.0, 1000, 8.0, 2.0)]),
                           scale=3.0 * (nope + rot) ** -0.5)
        layers.append((mixer, rng.choice([None, 32, 64, 100, 256, 512])))
    return config(vocab, width, layers, eps=rng.choice([1e-6, 1e-5]))


def random_model(seed: int):
    """(typed configuration, model folder, plain model) of random_config(seed)."""
    cfg = PizunexConfig.from_dict(random_config(seed))
    folder = os.path.join(_temporary(), f"random{seed}")
    if not os.path.isdir(folder):
        _write(folder, cfg, seed, 0.06)
    return cfg, folder, PlainPizunex.from_folder(folder)
