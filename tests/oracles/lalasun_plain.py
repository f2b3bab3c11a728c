"""A plain, slow Lalasun forward: one function per mechanism, written token by token from the design's equations.

It is the oracle the framework's Lalasun path is tested against and shares no code with it.  Everything is computed in
float64 from whatever weights it is given (a dict name -> tensor with the checkpoint's tensor names, and the parsed
config.json dict).  Sequences are processed one token at a time; caches and states are plain Python lists and tensors.
"""
from __future__ import annotations

import math

import torch

F = torch.float64


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def dynamic_tanh(x, W, name):
    """The stream's norm: no statistic, a squashing per element."""
    return torch.tanh(W[name + ".alpha"] * x) * W[name] + W[name + ".b"]


def poly_norm(z, abcd, eps):
    """a N(z) + b N(z^2) + c N(z^3) + e, N = division by the vector's root mean square."""
    a, b, c, e = (abcd[i] for i in range(4))
    return a * rms_unit(z, eps) + b * rms_unit(z ** 2, eps) + c * rms_unit(z ** 3, eps) + e


def rotate(x, pos, base, dims, interleaved):
    """Rotary position on the first ``dims`` entries of a vector."""
    y = x.clone()
    for i in range(dims // 2):
        a = pos * base ** (-2.0 * i / dims)
        m, n = (2 * i, 2 * i + 1) if interleaved else (i, i + dims // 2)
        u, v = float(x[m]), float(x[n])
        y[m] = u * math.cos(a) - v * math.sin(a)
        y[n] = v * math.cos(a) + u * math.sin(a)
    return y


def window_visible(i, j, size):
    return j <= i and (not size or i - j < size)


def chunk_visible(i, j, size):
    return j <= i and (not size or i // size == j // size)


def latent_token(h, W, p, mx, eps, pos, cache):
    """One token of the latent attention.  cache: list of (latent c, rotated key part) of ALL earlier tokens."""
    H, D, R, Dv, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    base, dims = (mx["rot"]["base"], mx["rot"]["dims"]) if mx.get("rot") else (1.0, 0)
    q = (W[p + "q"] @ h).view(H, D + R)
    dkv = W[p + "dkv"] @ h
    c = rms_unit(dkv[:rank], eps) * W[p + "dkv.norm"]
    cache.append((c, rotate(dkv[rank:], pos, base, dims, True)))
    size = (mx.get("mask") or {}).get("size", 0)
    js = [j for j in range(pos + 1) if window_visible(pos, j, size)]
    cs = torch.stack([cache[j][0] for j in js])
    kr = torch.stack([cache[j][1] for j in js])
    uk, uv = W[p + "uk"].view(H, D, rank), W[p + "uv"].view(H, Dv, rank)
    out = torch.zeros(H, Dv, dtype=F)
    for hd in range(H):
        keys, vals = cs @ uk[hd].t(), cs @ uv[hd].t()
        sc = (keys @ q[hd, :D] + kr @ rotate(q[hd, D:], pos, base, dims, True)) * mx["scale"]
        a = torch.exp(sc - sc.max())
        out[hd] = (a / a.sum()) @ vals
    return W[p + "o"] @ (out.reshape(-1) * sigmoid(W[p + "g"] @ h))


def attention_token(h, W, p, mx, pos, cache):
    """One token of the chunked attention with one added to the softmax denominator.  cache: list of (k [G, D],
    v [G, Dv]) of ALL earlier tokens."""
    H, G, D, Dv = mx["heads"], mx.get("kv_heads", mx["heads"]), mx["dim"], mx["vdim"]
    base, dims = (mx["rot"]["base"], mx["rot"]["dims"]) if mx.get("rot") else (1.0, 0)
    q = (W[p + "q"] @ h + W[p + "q.b"]).view(H, D)
    k = (W[p + "k"] @ h + W[p + "k.b"]).view(G, D)
    v = (W[p + "v"] @ h + W[p + "v.b"]).view(G, Dv)
    cache.append((torch.stack([rotate(k[g], pos, base, dims, False) for g in range(G)]), v))
    size = (mx.get("mask") or {}).get("size", 0)
    js = [j for j in range(pos + 1) if chunk_visible(pos, j, size)]
    keys = torch.stack([cache[j][0] for j in js])
    vals = torch.stack([cache[j][1] for j in js])
    out = torch.zeros(H, Dv, dtype=F)
    for hd in range(H):
        g = hd // (H // G)
        sc = (keys[:, g] @ rotate(q[hd], pos, base, dims, False)) * mx["scale"]
        top = max(float(sc.max()), 0.0)
        a = torch.exp(sc - top)
        out[hd] = (a / (math.exp(-top) + a.sum())) @ vals[:, g]
    return W[p + "o"] @ out.reshape(-1) + W[p + "o.b"]


def gla_token(h, W, p, mx, eps, state):
    """One token of the gated linear attention.  state: dict with 'S' [heads, dim, vdim]."""
    H, D, Dv = mx["heads"], mx["dim"], mx["vdim"]
    q = (W[p + "q"] @ h).view(H, D) * D ** -0.5
    k = (W[p + "k"] @ h).view(H, D)
    v = (W[p + "v"] @ h).view(H, Dv)
    z = W[p + "a2"] @ (W[p + "a1"] @ h) + W[p + "a2.b"]
    alpha = (sigmoid(z) ** (1.0 / mx["tau"])).view(H, D)
    out = torch.zeros(H, Dv, dtype=F)
    for hd in range(H):
        state["S"][hd] = alpha[hd][:, None] * state["S"][hd] + torch.outer(k[hd], v[hd])
        out[hd] = rms_unit(state["S"][hd].t() @ q[hd], eps) * W[p + "norm"]
    return W[p + "o"] @ (out.reshape(-1) * silu(W[p + "g"] @ h))


def feed_forward(h, W, p, eps):
    return W[p + "down"] @ poly_norm(W[p + "up"] @ h, W[p + "act"], eps)


def gated(y, h, W, name):
    """A sublayer's result times the gate made of what the sublayer read."""
    return y * sigmoid(W[name] @ h + W[name + ".b"])


class PlainLalasun:
    """Token-by-token forward of one sequence.  ``step(token)`` returns (logits, [stream after every layer])."""

    def __init__(self, cfg: dict, tensors: dict):
        self.cfg = cfg
        self.W = {k: v.to(F) for k, v in tensors.items() if v.is_floating_point()}
        self.pos = 0
        self.state = []
        for l in cfg["layers"]:
            mx = l["mixer"]
            if l["type"] == "gla":
                self.state.append({"S": torch.zeros(mx["heads"], mx["dim"], mx["vdim"], dtype=F)})
            elif l["type"] in ("attention", "latent_attention"):
                self.state.append([])
            else:
                raise ValueError(l["type"])

    def step(self, token: int):
        cfg, W = self.cfg, self.W
        eps, m = cfg["norm"]["eps"], cfg["residual_mult"]
        x = W["embed"][token].clone()
        history = [x.clone()]                       # X_0 ... X_i: embedding output and the layers' own results
        streams = []
        for i, l in enumerate(cfg["layers"]):
            p = f"l{i}."
            h = dynamic_tanh(x, W, p + "norm1")
            if l["type"] == "attention":
                y = attention_token(h, W, p + "mix.", l["mixer"], self.pos, self.state[i])
            elif l["type"] == "latent_attention":
                y = latent_token(h, W, p + "mix.", l["mixer"], eps, self.pos, self.state[i])
            else:
                y = gla_token(h, W, p + "mix.", l["mixer"], eps, self.state[i])
            x = x + m * gated(y, h, W, p + "rg1")
            if l.get("mlp"):
                h = dynamic_tanh(x, W, p + "norm2")
                x = x + m * gated(feed_forward(h, W, p + "mlp.", eps), h, W, p + "rg2")
            history.append(x.clone())
            x = sum(W[p + "dwa"][j] * history[j] for j in range(i + 2))
            streams.append(x.clone())
        self.pos += 1
        return W["head"] @ dynamic_tanh(x, W, "final.norm"), streams


def run(cfg: dict, tensors: dict, tokens):
    """Logits of every token [n, vocab] and the stream after every layer [layers][n, width]."""
    m = PlainLalasun(cfg, tensors)
    logits, per = [], [[] for _ in cfg["layers"]]
    for t in tokens:
        lg, streams = m.step(int(t))
        logits.append(lg)
        for r, x in enumerate(streams):
            per[r].append(x)
    return torch.stack(logits), [torch.stack(v) for v in per]
