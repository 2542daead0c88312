"""A plain, slow statement of the Pizunex decoder in float64 on the CPU: one function for each mechanism, whole
sequences only (no cache, no batches, no portions; attention is a full score matrix with a mask, the recurrence a loop
over tokens).  The oracle of the GPU tests; it shares no code with the package.

Notation: T tokens, W the width; positions count from 0; a weight [out, in] meets a row x as x @ w.T.
"""
from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


def over_rms(x, eps):
    return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)


def rms_norm(x, gain, eps):
    return over_rms(x, eps) * gain


def silu(z):
    return z * torch.sigmoid(z)


# ---------------------------------------------------------------- the delta rule with one decay a head
def short_conv(u, taps):
    """u [T, C], taps [C, n]: y_t = sum_j taps[:, j] u_(t - n + 1 + j), zeros before the first token."""
    T, C = u.shape
    n = taps.shape[1]
    padded = torch.cat([torch.zeros(n - 1, C, dtype=u.dtype), u], 0)
    y = torch.zeros_like(u)
    for j in range(n):
        y = y + padded[j:j + T] * taps[:, j]
    return y


def unit(x):
    return x / torch.sqrt(x.pow(2).sum(-1, keepdim=True) + 1e-6)


def delta_cell(q, k, v, beta, decay, state=None):
    """q, k [T, H, D], v [T, H, E], beta and decay [T, H] -> (o [T, H, E], the state [H, D, E] after the last token).
    For each token:  S <- decay S;  u = beta (v - S^T k);  S <- S + k u^T;  o = S^T q."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if state is None else state.clone()
    out = []
    for t in range(T):
        S = S * decay[t][:, None, None]
        u = beta[t][:, None] * (v[t] - (S * k[t][:, :, None]).sum(1))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append((S * q[t][:, :, None]).sum(1))
    return torch.stack(out), S


def delta_mixer(h, w, p, c, eps):
    T = h.shape[0]
    H, K, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q, k, v = (silu(short_conv(h @ w[p + n].T, w[p + n + ".conv"])) for n in ("q", "k", "v"))
    rep = H // K                                    # head h reads key head h // rep
    q = (unit(q.view(T, K, D)) * D ** -0.5).repeat_interleave(rep, 1)
    k = unit(k.view(T, K, D)).repeat_interleave(rep, 1)
    beta = torch.sigmoid(h @ w[p + "b"].T)
    decay = torch.exp(-torch.exp(w[p + "A_log"]) * torch.nn.functional.softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    o, _ = delta_cell(q, k, v.view(T, H, E), beta, decay)
    o = over_rms(o, eps) * w[p + "norm"] * silu((h @ w[p + "g"].T).view(T, H, E))
    return o.reshape(T, H * E) @ w[p + "o"].T


# ---------------------------------------------------------------- attention
def window_mask(T, size):
    """[T, T] bool: query i sees key j iff 0 <= i - j < size (size None: every earlier key)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    m = j <= i
    return m if size is None else m & (i - j < size)


def linear_slopes(H):
    return torch.tensor([2.0 ** (-8.0 * (h + 1) / H) for h in range(H)], dtype=F64)


def temperature(T, coef, every):
    """One factor a position: 1 + coef ln(floor((p + 1) / every) + 1)."""
    return torch.tensor([1.0 + coef * math.log((p + 1) // every + 1) for p in range(T)], dtype=F64)


def attend(q, k, v, scale, mask, softcap=None, slopes=None):
    """q [T, H, D], k [T, G, D], v [T, G, E], mask [T, T] bool -> [T, H, E].  Head h reads kv head h // (H / G).
    score = scale q.k, then softcap tanh(score / softcap), then - slope_h (i - j); softmax over the visible keys."""
    T, H, _ = q.shape
    G = k.shape[1]
    dist = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(F64)
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * scale
        if softcap is not None:
            s = softcap * torch.tanh(s / softcap)
        if slopes is not None:
            s = s - slopes[h] * dist
        out[:, h] = torch.softmax(s.masked_fill(~mask, -math.inf), -1) @ v[:, g]
    return out


def attention(h, w, p, c, eps):
    """Values are the keys as projected; q and k are normed over the whole projection; no rotation."""
    T = h.shape[0]
    H, G, D = c["heads"], c["kv_heads"], c["dim"]
    raw = h @ w[p + "k"].T
    q = rms_norm(h @ w[p + "q"].T, w[p + "q.norm"], eps).view(T, H, D)
    k = rms_norm(raw, w[p + "k.norm"], eps).view(T, G, D)
    if c.get("q_temp") is not None:
        q = q * temperature(T, c["q_temp"]["coef"], c["q_temp"]["every"])[:, None, None]
    mask = window_mask(T, c["mask"]["size"] if c.get("mask") else None)
    o = attend(q, k, raw.view(T, G, D), c["scale"], mask, c.get("softcap"), linear_slopes(H))
    return o.reshape(T, H * D) @ w[p + "o"].T


# ---------------------------------------------------------------- latent attention
def rates(base, dims, scaling=None):
    """(f_i, the factor on cos and sin): f_i = base^(-2i / dims), with `scaling` blended towards f_i / factor by a ramp
    over i between the places where a wave turns `fast` and `slow` times over the original context."""
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=F64)
    if scaling is None:
        return f, 1.0

    def place(turns):
        return dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo = max(math.floor(place(scaling["fast"])), 0)
    hi = min(math.ceil(place(scaling["slow"])), dims - 1)
    for i in range(dims // 2):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        f[i] = f[i] / scaling["factor"] * r + f[i] * (1.0 - r)
    return f, 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_pairs(x, f, mult=1.0, first=0):
    """x [T, ..., D]: the pairs (2i, 2i + 1), i < len(f), turned by position * f_i and multiplied by `mult`; the token at
    row t has position first + t."""
    T, n = x.shape[0], f.shape[0]
    ang = torch.arange(first, first + T, dtype=F64)[:, None] * f[None, :]
    shape = [T] + [1] * (x.dim() - 2) + [n]
    c, s = (torch.cos(ang) * mult).view(shape), (torch.sin(ang) * mult).view(shape)
    out = x.clone()
    u, v = x[..., 0:2 * n:2], x[..., 1:2 * n:2]
    out[..., 0:2 * n:2] = u * c - v * s
    out[..., 1:2 * n:2] = v * c + u * s
    return out


def latent_attention(h, w, p, c, eps):
    """Queries through a normed latent of their own (or straight from h: no q_rank); per-head keys and values from one normed latent a token, and one
    turned key part for all heads."""
    T = h.shape[0]
    H, D, R, E, C = c["heads"], c["dim"], c["rot_dim"], c["vdim"], c["kv_rank"]
    f, mult = rates(c["rot"]["base"], c["rot"]["dims"], c["rot"].get("scaling"))
    if c.get("q_rank") is not None:
        q = rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], eps) @ w[p + "uq"].T
    else:
        q = h @ w[p + "q"].T
    q = q.view(T, H, D + R)
    q = torch.cat([q[..., :D], rotate_pairs(q[..., D:], f, mult)], -1)
    down = h @ w[p + "dkv"].T
    lat = rms_norm(down[:, :C], w[p + "dkv.norm"], eps)
    k_rot = rotate_pairs(down[:, C:].view(T, 1, R), f, mult)
    k = torch.cat([(lat @ w[p + "uk"].T).view(T, H, D), k_rot.expand(T, H, R)], -1)
    v = (lat @ w[p + "uv"].T).view(T, H, E)
    return attend(q, k, v, c["scale"], window_mask(T, None)).reshape(T, H * E) @ w[p + "o"].T


# ---------------------------------------------------------------- feed-forward
def squared_relu_mlp(h, w, p):
    return torch.relu(h @ w[p + "up"].T).pow(2) @ w[p + "down"].T


# ---------------------------------------------------------------- the model
MIXERS = {"delta": delta_mixer, "attention": attention, "latent_attention": latent_attention}


class PlainPizunex:
    def __init__(self, config: dict, weights: dict):
        self.c = config
        self.w = {k: v.to(F64) for k, v in weights.items()}

    @classmethod
    def from_folder(cls, folder):
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            config = json.load(f)
        return cls(config, load_file(os.path.join(folder, "model.safetensors")))

    def tensors_of(self, i):
        """The layer whose tensors layer i runs with: its own, or where its chain of `weights_of` ends."""
        while self.c["layers"][i].get("weights_of") is not None:
            i = self.c["layers"][i]["weights_of"]
        return i

    def residuals(self, tokens):
        """[layers, T, W]: the residual after each layer."""
        c, w = self.c, self.w
        eps = c["norm"]["eps"]
        x = w["embed"][torch.tensor(tokens)]
        out = []
        for i, layer in enumerate(c["layers"]):
            p = f"l{self.tensors_of(i)}."
            x = x + MIXERS[layer["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
            if layer.get("mlp") is not None:
                x = x + squared_relu_mlp(rms_norm(x, w[p + "norm2"], eps), w, p + "mlp.")
            out.append(x)
        return torch.stack(out)

    def logits(self, tokens):
        x = self.residuals(tokens)[-1]
        return rms_norm(x, self.w["final.norm"], self.c["norm"]["eps"]) @ self.w["head"].T
