"""A plain, slow Nubodra forward: one function per mechanism, written token by token from the design's equations.

It is the oracle the framework's Nubodra path is tested against and shares no code with it.  Everything is computed in
float64 from whatever weights it is given (a dict name -> tensor with the checkpoint's tensor names, and the parsed
config.json dict).  Sequences are processed one token at a time; caches and histories are plain Python lists.
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


def layer_norm(x, W, name, eps):
    mean = x.mean()
    dev = x - mean
    return dev / torch.sqrt((dev * dev).mean() + eps) * W[name] + W[name + ".b"]


def query_temperature(pos, temp):
    """Factor on the query at position pos: 1 + coef ln(floor((pos + 1) / every) + 1); 1 without a temperature."""
    if not temp:
        return 1.0
    return 1.0 + temp["coef"] * math.log(math.floor((pos + 1) / temp["every"]) + 1)


def conv_token(u, taps, earlier):
    """Causal convolution per channel of the newest projection u; ``earlier``: every projection before it, oldest
    first (a list that grows by u).  taps [channels, K], the last column for the newest one."""
    earlier.append(u)
    K = taps.shape[1]
    y = torch.zeros_like(u)
    for j in range(K):
        back = K - 1 - j
        if back < len(earlier):
            y = y + taps[:, j] * earlier[-1 - back]
    return y


def frequencies(rot):
    """Rotation frequencies per pair and the factor on cosine and sine."""
    base, dims = rot["base"], rot["dims"]
    f = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def turns_at(t):
        return dims * math.log(s["original"] / (2 * math.pi * t)) / (2 * math.log(base))

    lo = max(math.floor(turns_at(s["fast"])), 0)
    hi = min(math.ceil(turns_at(s["slow"])), dims - 1)
    out = []
    for i, fi in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(fi / s["factor"] * r + fi * (1.0 - r))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate(x, pos, rot):
    """Rotary position on neighbouring pairs of the vector's first rot.dims entries."""
    if not rot:
        return x
    y = x.clone()
    fs, mag = frequencies(rot)
    for i, f in enumerate(fs):
        u, v, c, s = float(x[2 * i]), float(x[2 * i + 1]), math.cos(pos * f) * mag, math.sin(pos * f) * mag
        y[2 * i] = u * c - v * s
        y[2 * i + 1] = v * c + u * s
    return y


def attention_token(h, W, p, mx, eps, pos, state):
    """One token of the attention whose values are its keys before the norm.  state: dict of the projections so far
    (q, k) and the cached (normed key, value) of ALL earlier tokens."""
    H, G, D = mx["heads"], mx.get("kv_heads", mx["heads"]), mx["dim"]
    q = conv_token(W[p + "q"] @ h, W[p + "q.conv"], state["q"]).view(H, D)
    k = conv_token(W[p + "k"] @ h, W[p + "k.conv"], state["k"]).view(G, D)
    state["kv"].append((rms_unit(k, eps), k))
    q = rms_unit(q, eps) * query_temperature(pos, mx.get("q_temp"))
    keys = torch.stack([e[0] for e in state["kv"]])
    vals = torch.stack([e[1] for e in state["kv"]])
    g = sigmoid(W[p + "g"] @ h)
    out = torch.zeros(H, D, dtype=F)
    for hd in range(H):
        kv = hd // (H // G)
        sc = (keys[:, kv] @ q[hd]) * mx["scale"]
        a = torch.exp(sc - sc.max())
        out[hd] = (a / a.sum()) @ vals[:, kv] * g[hd]
    return W[p + "o"] @ out.reshape(-1)


def latent_token(h, W, p, mx, eps, pos, cache, own):
    """One token of the latent attention with a sink.  cache: list of (latent, rotated key part) of ALL tokens; ``own``:
    this layer adds the newest token's pair (otherwise another layer has)."""
    H, D, R, Dv, rank = mx["heads"], mx["dim"], mx["rot_dim"], mx["vdim"], mx["kv_rank"]
    rot = mx.get("rot")
    q = (W[p + "uq"] @ (rms_unit(W[p + "dq"] @ h, eps) * W[p + "dq.norm"])).view(H, D + R)
    if own:
        dkv = W[p + "dkv"] @ h
        cache.append((rms_unit(dkv[:rank], eps) * W[p + "dkv.norm"], rotate(dkv[rank:], pos, rot)))
    cs = torch.stack([e[0] for e in cache])
    kr = torch.stack([e[1] for e in cache])
    uk, uv = W[p + "uk"].view(H, D, rank), W[p + "uv"].view(H, Dv, rank)
    out = torch.zeros(H, Dv, dtype=F)
    for hd in range(H):
        sc = (cs @ (uk[hd].t() @ q[hd, :D]) + kr @ rotate(q[hd, D:], pos, rot)) * mx["scale"]
        sink = float(W[p + "sink"][hd])
        top = max(float(sc.max()), sink)
        a = torch.exp(sc - top)
        out[hd] = uv[hd] @ ((a / (a.sum() + math.exp(sink - top))) @ cs)
    return W[p + "o"] @ out.reshape(-1)


def feed_forward(h, W, p):
    return W[p + "down"] @ (silu(W[p + "gate"] @ h) * (W[p + "up"] @ h))


class PlainNubodra:
    """Token-by-token forward of one sequence.  ``step(token)`` returns (logits, [stream after every layer])."""

    def __init__(self, cfg: dict, tensors: dict):
        self.cfg = cfg
        self.W = {k: v.to(F) for k, v in tensors.items() if v.is_floating_point()}
        self.pos = 0
        self.state = []
        for l in cfg["layers"]:
            if l["type"] == "attention":
                self.state.append(dict(q=[], k=[], kv=[]))
            elif l["type"] == "latent_attention":
                src = l["mixer"].get("kv_from")
                self.state.append([] if src is None else self.state[src])
            else:
                raise ValueError(l["type"])

    def step(self, token: int):
        cfg, W, eps = self.cfg, self.W, self.cfg["norm"]["eps"]
        x = W["embed"][token] * cfg["embedding"]["scale"]
        streams = []
        for i, l in enumerate(cfg["layers"]):
            p, mx = f"l{i}.", l["mixer"]
            h = layer_norm(x, W, p + "norm1", eps)
            if l["type"] == "attention":
                y = attention_token(h, W, p + "mix.", mx, eps, self.pos, self.state[i])
            else:
                y = latent_token(h, W, p + "mix.", mx, eps, self.pos, self.state[i], mx.get("kv_from") is None)
            if l.get("mlp"):
                y = y + feed_forward(h, W, p + "mlp.")
            x = x + y
            streams.append(x.clone())
        self.pos += 1
        return W["head"] @ layer_norm(x, W, "final.norm", eps), streams


def run(cfg: dict, tensors: dict, tokens):
    """Logits of every token [n, vocab] and the stream after every layer [layers][n, width]."""
    m = PlainNubodra(cfg, tensors)
    logits, per = [], [[] for _ in cfg["layers"]]
    for t in tokens:
        lg, streams = m.step(int(t))
        logits.append(lg)
        for r, x in enumerate(streams):
            per[r].append(x)
    return torch.stack(logits), [torch.stack(v) for v in per]
