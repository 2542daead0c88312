"""Small Sunosun configurations for the tests, their model folders (random weights), and the plain model's logits."""
from __future__ import annotations

import copy
import os
import tempfile

import torch

from synaptix_amd.config import SunosunConfig
from synaptix_amd import write_random_model
from plain_sunosun import PlainSunosun


def linear(heads, dim, vdim, tau=16.0):
    return {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}


def gla(heads, dim, vdim, tau=16.0):
    return "gla", linear(heads, dim, vdim, tau)


def parallel(left, right, left_scale=0.7, right_scale=1.2):
    """left: (heads, kv heads, key size, value size)."""
    h, kv, d, e = left
    return "parallel", {"left": {"heads": h, "kv_heads": kv, "dim": d, "vdim": e, "scale": 4.0 * d ** -0.5},
                        "right": linear(*right), "left_scale": left_scale, "right_scale": right_scale}


def moe(ff, experts, top, groups=None, scale=None, shared=None):
    router = {"experts": experts, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    if scale is not None:
        router["scale"] = scale
    m = {"kind": "moe", "expert": {"ff": ff}, "router": router}
    if shared is not None:
        m["shared"] = {"ff": shared}
    return m


def dense(ff):
    return {"kind": "dense", "ff": ff}


def config(vocab, width, layers, rank, loop=None, scale=None, cap=None, eps=1e-6):
    d = {"architecture": "Sunosun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "middle_rank": rank,
         "layers": [{"type": k, "mixer": m, "mlp": f} for (k, m), f in layers]}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    if scale is not None:
        d["embedding"] = {"scale": scale}
    if cap is not None:
        d["logit_softcap"] = cap
    return d


# P: both mixers, all kinds of feed-forward and none, layers 1 and 2 three times, groups whose best two decide, choice scores
#    that are all negative, a cap that bites.
# Q: sizes that are multiples of nothing (a width of 72, keys of 10 and 12, values of 14 and 18, a middle of 5, an odd
#    vocabulary), one key head, tau 4; no loop, cap, groups, shared expert, factors.
# R: sizes at which the products and prompts' attention run on the matrix cores; the whole stack twice.
# S: one head everywhere, values and keys of one value, groups of one expert, one expert chosen, tau 1, a loop of one pass.
# T: gated linear layers alone: a model without keys and values; the first layer four times.
# U: a parallel layer that runs three times, each on keys and a state of its own, with the last layer the loop's last.
CONFIGS = {
    "P": config(300, 64, [(parallel((4, 2, 16, 24), (3, 8, 12)), dense(48)),
                          (gla(4, 16, 20), moe(40, 12, 3, (4, 2), 1.7, 24)),
                          (gla(2, 24, 32, 8.0), None),
                          (gla(3, 8, 16), moe(24, 6, 3, (2, 1), 2.5, 32))], 6, (1, 3, 3), 9.0, 1.5),
    "Q": config(257, 72, [(gla(4, 12, 18, 4.0), dense(50)),
                          (parallel((3, 1, 10, 14), (5, 10, 6, 4.0), 1.0, 1.0), moe(30, 7, 3)),
                          (gla(5, 7, 6), None)], 5, eps=1e-5),
    "R": config(512, 128, [(gla(4, 32, 64), dense(256)),
                           (parallel((8, 2, 64, 32), (2, 64, 32)), moe(64, 16, 4, (4, 2), 2.0, 128)),
                           (gla(2, 64, 128), moe(96, 8, 8, (2, 2), 1.0, 64))], 16, (0, 3, 2), 8.0, 30.0),
    "S": config(101, 40, [(parallel((1, 1, 8, 1), (1, 1, 5, 1.0), -0.5, 0.8), moe(9, 4, 1, (4, 2), 3.0, 5)),
                          (gla(1, 6, 1, 1.0), dense(16))], 1, (1, 2, 1), 6.0, 4.0),
    "T": config(160, 96, [(gla(4, 24, 32), dense(64)), (gla(2, 40, 16, 64.0), moe(32, 8, 2, (2, 1), 1.5))], 12, (0, 1, 4), 7.0),
    "U": config(200, 256, [(gla(2, 16, 16), None),
                           (parallel((4, 4, 32, 48), (4, 48, 24)), dense(128))], 16, (1, 2, 3), 12.0, 2.0),
}
SEEDS = {"P": 61, "Q": 62, "R": 63, "S": 64, "T": 65, "U": 66}

_tmp = None
_folders, _plain, _logits = {}, {}, {}


def _extra(cfg, g):
    """Decays between 0.95 and 0.999 a token in most channels, so that what was written a hundred tokens ago still counts;
    choice scores that are negative; routers whose scores lie apart."""
    extra = {}
    for i, l in enumerate(cfg.layers):
        p = f"l{i}.mix." + ("right." if l.type == "parallel" else "")
        m = l.mixer.right if l.type == "parallel" else l.mixer
        extra[p + "a2.b"] = (3.0 + 1.5 * torch.randn(m.heads * m.dim, generator=g)).to(torch.bfloat16)
        if l.mlp is not None and l.mlp.kind == "moe":
            n = l.mlp.experts
            extra[f"l{i}.mlp.correction"] = (-1.2 + 0.3 * torch.randn(n, generator=g)).to(torch.bfloat16)
            extra[f"l{i}.mlp.router"] = (2.0 * cfg.width ** -0.5 * torch.randn(n, cfg.width, generator=g)).to(torch.bfloat16)
    return extra


def _write(folder, cfg, seed, std):
    g = torch.Generator().manual_seed(700 + seed)
    write_random_model(folder, cfg, seed, std=std, gain_std=0.3, extra_tensors=_extra(cfg, g))


def _temporary():
    global _tmp
    if _tmp is None:
        _tmp = tempfile.TemporaryDirectory(prefix="synaptix_amd_sunosun_")
    return _tmp.name


def model_folder(name: str) -> str:
    """Random bf16 weights, drawn wide enough that every branch carries weight; the attention's scales make it peaked, so
    that a lost or wrong key moves the logits."""
    if name not in _folders:
        folder = os.path.join(_temporary(), name)
        _write(folder, SunosunConfig.from_dict(copy.deepcopy(CONFIGS[name])), SEEDS[name], 0.08)
        _folders[name] = folder
    return _folders[name]


def plain_model(name: str) -> PlainSunosun:
    if name not in _plain:
        _plain[name] = PlainSunosun.from_folder(model_folder(name))
    return _plain[name]


def plain_logits(name: str, tokens) -> torch.Tensor:
    key = (name, tuple(tokens))
    if key not in _logits:
        _logits[key] = plain_model(name).logits(list(tokens))
    return _logits[key]


def tokens_for(name: str, n: int, seed: int) -> list:
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, CONFIGS[name]["vocab"], (n,), generator=g).tolist()


def routing_margins(plain: PlainSunosun, tokens) -> torch.Tensor:
    """[T]: how far each token is from another choice of experts anywhere in the model: the smallest gap between the last
    chosen and the best that was left (experts, and groups) over all runs of layers with experts; infinite without experts.
    Rounding in bfloat16 may turn a close call, and the token's logits are then another function of the weights."""
    import plain_sunosun
    least, route = torch.full((len(tokens),), float("inf"), dtype=torch.float64), plain_sunosun.route

    def spy(z, correction, top, groups, keep, scale):
        nonlocal least
        T, E = z.shape
        choice, per = torch.sigmoid(z) + correction, E // groups
        two = choice.view(T, groups, per).topk(min(2, per), -1).values.sum(-1).sort(-1, descending=True)
        if keep < groups:
            least = torch.minimum(least, two.values[:, keep - 1] - two.values[:, keep])
        on = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, two.indices[:, :keep], True)
        left = choice.masked_fill(~on[:, :, None].expand(T, groups, per).reshape(T, E), -1e9).sort(-1, descending=True).values
        if top < E:
            least = torch.minimum(least, left[:, top - 1] - left[:, top])
        return route(z, correction, top, groups, keep, scale)

    plain_sunosun.route = spy
    try:
        plain.residuals(tokens)
    finally:
        plain_sunosun.route = route
    return least


def random_config(seed: int) -> dict:
    """A configuration drawn from a seed: layer kinds in any order, head counts, sizes (multiples of sixteen and not),
    groups, loops, every optional mechanism on or off."""
    import random
    rng = random.Random(seed)
    width, vocab = rng.choice([64, 96, 128, 192, 256, 80]), rng.choice([200, 384, 512, 1000, 333])

    def one_linear():
        return (rng.choice([1, 2, 3, 4, 6]), rng.choice([8, 16, 24, 32, 48, 64, 96, 20]), rng.choice([8, 16, 32, 64, 96, 40]),
                rng.choice([1.0, 4.0, 16.0, 32.0]))

    layers = []
    n = rng.randint(2, 5)
    for _ in range(n):
        if rng.random() < 0.45:
            heads = rng.choice([1, 2, 3, 4, 6, 8, 12])
            kv = rng.choice([h for h in (1, 2, 3, 4, 6, 8, 12) if heads % h == 0])
            mixer = parallel((heads, kv, rng.choice([16, 32, 48, 64, 96, 128, 24]), rng.choice([16, 32, 48, 64, 40])), one_linear(),
                             rng.choice([0.5, 1.0, 1.5]), rng.choice([0.6, 1.0, 1.3]))
        else:
            mixer = gla(*one_linear())
        kind = rng.random()
        if kind < 0.45:
            count = rng.choice([1, 2, 4])
            experts = count * rng.choice([1, 2, 3, 4])
            keep = rng.randint(1, count)
            mlp = moe(rng.choice([32, 64, 48, 20]), experts, rng.randint(1, min(6, keep * experts // count)),
                      (count, keep) if count > 1 else None, rng.choice([None, 1.5, 2.5]), rng.choice([None, 32, 64, 30]))
        else:
            mlp = dense(rng.choice([32, 64, 100, 256])) if kind < 0.85 else None
        layers.append((mixer, mlp))
    loop = None
    if rng.random() < 0.7:
        a = rng.randint(0, n - 1)
        loop = (a, rng.randint(a + 1, n), rng.randint(1, 3))
    return config(vocab, width, layers, rng.choice([1, 4, 8, 16, 20]), loop, rng.choice([None, 4.0, 12.0]),
                  rng.choice([None, 2.0, 20.0]), eps=rng.choice([1e-6, 1e-5]))


def random_model(seed: int):
    """(typed configuration, model folder, plain model) of random_config(seed)."""
    cfg = SunosunConfig.from_dict(random_config(seed))
    folder = os.path.join(_temporary(), f"random{seed}")
    if not os.path.isdir(folder):
        _write(folder, cfg, seed, 0.06)
    return cfg, folder, PlainSunosun.from_folder(folder)
