"""A plain, slow statement of the Sunosun decoder in float64 on the CPU: one function for each mechanism, whole
sequences only (no cache, no batches, no portions; the recurrence is a loop over tokens, attention a full score matrix
with a mask).  The oracle of the GPU tests; it shares no code with the package.

Notation: T tokens, W the width; positions count from 0; a weight [out, in] meets a row x as x @ w.T.
"""
from __future__ import annotations

import json
import math
import os

import torch

F64 = torch.float64


def rms_norm(x, gain, eps):
    y = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    return y if gain is None else y * gain


# ---------------------------------------------------------------- the embedding
def sinusoid(T, W):
    """[T, W]: row p holds sin(p f_i) in place 2i and cos(p f_i) in place 2i + 1, f_i = 10000^(-2i / W)."""
    out = torch.zeros(T, W, dtype=F64)
    for c in range(W):
        f = 10000.0 ** (-2.0 * (c // 2) / W)
        ang = torch.arange(T, dtype=F64) * f
        out[:, c] = torch.sin(ang) if c % 2 == 0 else torch.cos(ang)
    return out


def embed(table, tokens, scale):
    x = table[torch.tensor(tokens)] * scale
    return x + sinusoid(x.shape[0], x.shape[1])


# ---------------------------------------------------------------- mixers
def softmax_one(s, mask):
    """exp(s) / (1 + sum exp(s)) over the places that the mask leaves."""
    s = s.masked_fill(~mask, -math.inf)
    m = torch.clamp(s.max(-1, keepdim=True).values, min=0.0)
    e = torch.exp(s - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention(h, w, p, c):
    """Grouped-query attention with biases, no positions, every earlier key, one added to the softmax's denominator."""
    T = h.shape[0]
    H, G, D, E = c["heads"], c["kv_heads"], c["dim"], c["vdim"]
    q = (h @ w[p + "q"].T + w[p + "q.b"]).view(T, H, D)
    k = (h @ w[p + "k"].T + w[p + "k.b"]).view(T, G, D)
    v = (h @ w[p + "v"].T + w[p + "v.b"]).view(T, G, E)
    mask = torch.arange(T)[None, :] <= torch.arange(T)[:, None]
    out = torch.zeros(T, H, E, dtype=F64)
    for i in range(H):
        g = i // (H // G)
        out[:, i] = softmax_one((q[:, i] @ k[:, g].T) * c["scale"], mask) @ v[:, g]
    return out.reshape(T, H * E) @ w[p + "o"].T


def decays(z, tau):
    """sigmoid(z)^(1 / tau)."""
    return torch.exp(torch.nn.functional.logsigmoid(z) / tau)


def gla_cell(q, k, v, alpha, S=None):
    """q, k, alpha [T, H, D], v [T, H, E]: S <- diag(alpha_t) S + k_t v_t^T, o_t = S^T q_t.  Returns (o [T, H, E], S)."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=F64) if S is None else S.clone()
    o = torch.zeros_like(v)
    for t in range(T):
        S = alpha[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        o[t] = (S * q[t][:, :, None]).sum(1)
    return o, S


def gla(h, w, p, c, eps):
    """Gated linear attention; each head's read-out normed, then gated by silu(W_g h)."""
    T = h.shape[0]
    H, D, E = c["heads"], c["dim"], c["vdim"]
    q = (h @ w[p + "q"].T).view(T, H, D) * D ** -0.5
    k = (h @ w[p + "k"].T).view(T, H, D)
    v = (h @ w[p + "v"].T).view(T, H, E)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    o, _ = gla_cell(q, k, v, decays(z, c["tau"]).view(T, H, D))
    o = rms_norm(o, w[p + "norm"], eps).reshape(T, H * E)
    g = h @ w[p + "g"].T
    return (o * g * torch.sigmoid(g)) @ w[p + "o"].T


def parallel(h, w, p, c, eps):
    return (c["left_scale"] * attention(h, w, p + "left.", c["left"])
            + c["right_scale"] * gla(h, w, p + "right.", c["right"], eps))


# ---------------------------------------------------------------- feed-forwards
def dense(h, w, p):
    z = h @ w[p + "gate"].T
    return (z * torch.sigmoid(z) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def expert(h, w, p):
    return torch.clamp(h @ w[p + "up"].T, min=0.0).pow(2) @ w[p + "down"].T


def route(z, correction, top, groups, keep, scale):
    """z [T, E] router outputs -> (ids [T, top], weights [T, top]).  The choice is made on sigmoid(z) + correction among
    the members of the `keep` groups whose two largest choice scores have the largest sum; the weights are the chosen
    sigmoids over their sum, times `scale`."""
    T, E = z.shape
    s = torch.sigmoid(z)
    choice = s + correction
    per = E // groups
    two = choice.view(T, groups, per).topk(min(2, per), -1).values.sum(-1)
    kept = two.topk(keep, -1).indices
    on = torch.zeros(T, groups, dtype=torch.bool).scatter_(1, kept, True)
    allowed = on[:, :, None].expand(T, groups, per).reshape(T, E)
    ids = choice.masked_fill(~allowed, -math.inf).topk(top, -1).indices
    wt = s.gather(1, ids)
    return ids, wt / (wt.sum(-1, keepdim=True) + 1e-20) * scale


def experts(h, w, p, c):
    r = c["router"]
    g = r.get("groups") or {"count": 1, "keep": 1}
    ids, wt = route(h @ w[p + "router"].T, w[p + "correction"], r["top"], g["count"], g["keep"], r.get("scale", 1.0))
    y = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for e, a in zip(ids[t].tolist(), wt[t].tolist()):
            y[t] += a * expert(h[t:t + 1], w, f"{p}e{e}.")[0]
    if c.get("shared") is not None:
        y = y + expert(h, w, p + "shared.") * torch.sigmoid(h @ w[p + "shared.sg"].T)
    return y


# ---------------------------------------------------------------- the model
def layer_runs(config):
    """The layers in the order they run, each as (layer, pass): pass is the number of the looped layers' pass that the
    run opens, or None."""
    n, loop = len(config["layers"]), config.get("loop")
    if loop is None:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    runs = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        runs += [(i, t if i == a else None) for i in range(a, b)]
    return runs + [(i, None) for i in range(b, n)]


class PlainSunosun:
    def __init__(self, config: dict, weights: dict):
        self.c = config
        self.w = {k: v.to(F64) for k, v in weights.items()}

    @classmethod
    def from_folder(cls, folder):
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            config = json.load(f)
        return cls(config, load_file(os.path.join(folder, "model.safetensors")))

    def residuals(self, tokens):
        """[layer runs, T, W]: the residual after each run of a layer."""
        c, w = self.c, self.w
        eps = c["norm"]["eps"]
        x0 = embed(w["embed"], tokens, (c.get("embedding") or {}).get("scale", 1.0))
        x, out = x0, []
        for i, t in layer_runs(c):
            layer, p = c["layers"][i], f"l{i}."
            if t is not None:
                if t > 0:
                    x = x + x0
                x = x + w["loop.step"][t]
            mix = {"gla": gla, "parallel": parallel}[layer["type"]]
            x = x + mix(rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
            f = layer.get("mlp")
            if f is not None:
                h = rms_norm(x, w[p + "norm2"], eps)
                x = x + (dense(h, w, p + "mlp.") if f["kind"] == "dense" else experts(h, w, p + "mlp.", f))
            out.append(x)
        return torch.stack(out)

    def logits(self, tokens):
        x = self.residuals(tokens)[-1]
        y = rms_norm(x, self.w["final.norm"], self.c["norm"]["eps"]) @ self.w["embed"].T
        cap = self.c.get("logit_softcap")
        return y if cap is None else cap * torch.tanh(y / cap)
