"""Lalasun: a hybrid decoder on a pre-norm residual stream without norm statistics (every norm is Dynamic Tanh,
tanh(alpha x) w + b).  What a sublayer adds is gated element by element by sigmoid of a projection of the sublayer's
own input and multiplied by one constant, and after every layer the stream becomes a weighted sum of the embedding
output and all layers' results so far.  Its layers mix tokens with chunked grouped-query attention (biased projections,
rotated queries and keys, one added to the softmax denominator), with latent attention through a sliding window
(interleaved rotation, a sigmoid output gate per column) or with gated linear attention, and feed forward through a
dense unit with the PolyNorm activation.

This module is the design's reader: ``config.json`` -> :class:`chronos.models.hybrid.HybridConfig`, the checkpoint's
tensor names -> the packed weights the hybrid kernels take, and random weights of the same shapes for benchmarks and
tests.  Everything computed lives in :mod:`chronos.models.hybrid` and :mod:`chronos.ops.hybrid`.

config.json:  architecture "Lalasun"; vocab, width, residual_mult, norm.eps; layers[i] = {type, mixer{...}, mlp|null}
  type "attention":         mixer {heads, kv_heads, dim, vdim, scale, mask{size}, rot{base, dims}}
  type "latent_attention":  mixer {heads, dim, rot_dim, vdim, kv_rank, scale, mask{size}, rot{base, dims}}
  type "gla":               mixer {heads, dim, vdim, tau}   (the decay projection's rank is the shape of mix.a1)
  mlp {kind "dense", ff}
tensors (bfloat16, [out, in]):  embed, head, final.norm (+ .alpha, .b), l<i>.norm1 / .norm2 (+ .alpha, .b),
                                l<i>.rg1 / .rg2 (+ .b), l<i>.dwa, l<i>.mix.*, l<i>.mlp.up / .down / .act
"""
from __future__ import annotations

import json
import os

import torch

from .hybrid import (FEED_FORWARDS, MIXERS, GLASpec, HybridConfig, HybridDecoder, HybridLayerWeights, HybridWeights,
                     LatentAttentionSpec, LayerSpec, PolyFFSpec, WindowAttentionSpec)
from .zokunex import _SafetensorsDir

ARCHITECTURE = "Lalasun"
DEFAULT_GLA_RANK = 16
SINK_SCORE = 0.0   # one added to the softmax denominator: a sink of score 0 in every head


def config_from_dict(c: dict, name: str = "lalasun", max_position: int = 8192, gla_ranks: dict | None = None) -> HybridConfig:
    """``gla_ranks``: layer index -> rank of that layer's decay projection (a checkpoint's ``mix.a1`` has that many
    rows; config.json may also carry it as mixer.rank)."""
    layers = []
    for i, l in enumerate(c["layers"]):
        mx = l["mixer"]
        rot, size = mx.get("rot") or {}, int((mx.get("mask") or {}).get("size", 0))
        if l["type"] == "attention":
            heads = int(mx["heads"])
            mixer = WindowAttentionSpec(heads, int(mx.get("kv_heads", heads)), int(mx["dim"]), int(mx["vdim"]),
                                        float(mx["scale"]), rope_base=float(rot.get("base", 10000.0)),
                                        rope_dims=int(rot.get("dims", mx["dim"] if rot else 0)), chunk=size,
                                        qk_norm=False, sink=True, sink_fixed=SINK_SCORE, gate=False, bias=True,
                                        bias_o=True)
            if mixer.heads % mixer.kv_heads:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
            if mixer.rope_dims % 2 or mixer.rope_dims > mixer.dim:
                raise ValueError(f"layer {i}: rot.dims must be even and at most dim")
        elif l["type"] == "latent_attention":
            mixer = LatentAttentionSpec(int(mx["heads"]), int(mx["dim"]), int(mx["rot_dim"]), int(mx["vdim"]),
                                        int(mx["kv_rank"]), float(mx["scale"]), float(rot.get("base", 10000.0)),
                                        int(rot.get("dims", mx["rot_dim"] if rot else 0)), window=size,
                                        rope_interleaved=True, gate_wide=True, two_term=True)
            if mixer.rope_dims % 2 or mixer.rope_dims > mixer.rot_dim:
                raise ValueError(f"layer {i}: rot.dims must be even and at most rot_dim")
        elif l["type"] == "gla":
            rank = int((gla_ranks or {}).get(i, mx.get("rank", DEFAULT_GLA_RANK)))
            mixer = GLASpec(int(mx["heads"]), int(mx["dim"]), int(mx["vdim"]), float(mx["tau"]), rank)
        else:
            raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
        mlp = l.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
        layers.append(LayerSpec(mixer, PolyFFSpec(int(mlp["ff"])) if mlp is not None else None))
    return HybridConfig(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
                        norm_eps=float(c["norm"]["eps"]), max_position=max_position, architecture=ARCHITECTURE,
                        residual="pre_norm", norm="tanh", residual_mult=float(c.get("residual_mult", 1.0)),
                        residual_gate=True, depth_average=True)


def config_to_dict(cfg: HybridConfig) -> dict:
    """The config.json form of a configuration (what :func:`config_from_dict` reads)."""
    layers = []
    for l in cfg.layers:
        m = l.mixer
        if m.kind == "window_attention":
            mixer, typ, size = dict(heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim, scale=m.scale), \
                "attention", m.chunk
        elif m.kind == "latent_attention":
            mixer, typ, size = dict(heads=m.heads, dim=m.dim, rot_dim=m.rot_dim, vdim=m.vdim, kv_rank=m.kv_rank,
                                    scale=m.scale), "latent_attention", m.window
        else:
            mixer, typ, size = dict(heads=m.heads, dim=m.dim, vdim=m.vdim, tau=m.tau, rank=m.rank), "gla", 0
        if size:
            mixer["mask"] = dict(size=size)
        if typ != "gla" and m.rope_dims:
            mixer["rot"] = dict(base=m.rope_base, dims=m.rope_dims)
        layers.append(dict(type=typ, mixer=mixer, mlp=dict(kind="dense", ff=l.ff.ff) if l.ff is not None else None))
    return dict(architecture=ARCHITECTURE, vocab=cfg.vocab_size, width=cfg.hidden_size, residual_mult=cfg.residual_mult,
                norm=dict(eps=cfg.norm_eps), layers=layers)


def tensor_shapes(cfg: HybridConfig) -> dict:
    """Checkpoint tensor name -> shape."""
    d, V = cfg.hidden_size, cfg.vocab_size
    norm = lambda p: {p: (d,), p + ".b": (d,), p + ".alpha": ()}  # noqa: E731
    out = {"embed": (V, d)}
    for i, l in enumerate(cfg.layers):
        m, p = l.mixer, f"l{i}."
        out.update(norm(p + "norm1"))
        if l.ff is not None:
            out.update(norm(p + "norm2"))
        if m.kind == "window_attention":
            hq, gk, gv = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
            out.update({p + "mix.q": (hq, d), p + "mix.q.b": (hq,), p + "mix.k": (gk, d), p + "mix.k.b": (gk,),
                        p + "mix.v": (gv, d), p + "mix.v.b": (gv,), p + "mix.o": (d, m.heads * m.vdim), p + "mix.o.b": (d,)})
        elif m.kind == "latent_attention":
            hv = m.heads * m.vdim
            out.update({p + "mix.q": (m.heads * (m.dim + m.rot_dim), d), p + "mix.dkv": (m.kv_rank + m.rot_dim, d),
                        p + "mix.dkv.norm": (m.kv_rank,), p + "mix.uk": (m.heads * m.dim, m.kv_rank),
                        p + "mix.uv": (hv, m.kv_rank), p + "mix.g": (hv, d), p + "mix.o": (d, hv)})
        else:
            hd, hv = m.heads * m.dim, m.heads * m.vdim
            out.update({p + "mix.q": (hd, d), p + "mix.k": (hd, d), p + "mix.v": (hv, d), p + "mix.g": (hv, d),
                        p + "mix.o": (d, hv), p + "mix.norm": (m.vdim,), p + "mix.a1": (m.rank, d),
                        p + "mix.a2": (hd, m.rank), p + "mix.a2.b": (hd,)})
        out.update({p + "rg1": (d, d), p + "rg1.b": (d,)})
        if l.ff is not None:
            out.update({p + "mlp.up": (l.ff.ff, d), p + "mlp.down": (d, l.ff.ff), p + "mlp.act": (4,),
                        p + "rg2": (d, d), p + "rg2.b": (d,)})
        out[p + "dwa"] = (i + 2,)
    out.update(norm("final.norm"))
    out["head"] = (V, d)
    return out


def random_tensors(cfg: HybridConfig, seed: int = 0, device="cpu", std: float | None = None) -> dict:
    """Checkpoint-named random bfloat16 tensors: norm weights and slopes near one, biases small, depth averages that lean
    on the newest result, decay-logit biases positive so the linear-attention state mostly persists."""
    gen = torch.Generator(device="cpu")
    gen.manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        rn = lambda s=1.0: torch.randn(shape, generator=gen) * s  # noqa: E731
        if name.endswith(".alpha"):
            t = rn(0.1) + 0.7
        elif name.endswith(".dwa"):
            t = rn(0.15)
            t[-1] += 0.8
        elif name.endswith("mlp.act"):
            t = rn(0.3) + torch.tensor([0.6, -0.3, 0.2, 0.1])
        elif name.endswith("a2.b"):
            t = rn(0.5) + 2.0
        elif "norm" in name and not name.endswith(".b"):
            t = rn(0.1) + 1.0
        elif len(shape) == 1:
            t = rn(0.2)
        elif name == "embed":
            t = rn()
        else:
            t = rn(std if std is not None else shape[1] ** -0.5)
        out[name] = t.to(torch.bfloat16).to(device)
    return out


def pack_weights(cfg: HybridConfig, tensors, device, act_dtype) -> HybridWeights:
    """``tensors``: a mapping (or any object with ``__getitem__``) from checkpoint names to tensors.  The rows of a
    sublayer's residual gate join the sublayer's own first projection (they read the same input)."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    shapes = tensor_shapes(cfg)

    def get(name):
        t = tensors[name]
        if tuple(t.shape) != tuple(shapes[name]):
            raise ValueError(f"tensor {name}: shape {tuple(t.shape)}, the configuration says {tuple(shapes[name])}")
        return t

    norm = lambda n: f(torch.cat([get(n), get(n + ".b"), get(n + ".alpha").reshape(1)]))  # noqa: E731

    def sub(p, kinds, spec, gate):
        names = [n[len(p):] for n in shapes if n.startswith(p)]
        return kinds[spec.kind][1](spec, {**{n: get(p + n) for n in names}, "rg": get(gate)}, device, act_dtype)

    layers = []
    for i, l in enumerate(cfg.layers):
        lw = HybridLayerWeights(norm(f"l{i}.norm1"), sub(f"l{i}.mix.", MIXERS, l.mixer, f"l{i}.rg1"),
                                gate1=dict(b=f(get(f"l{i}.rg1.b"))), dwa=f(get(f"l{i}.dwa")))
        if l.ff is not None:
            lw.norm2, lw.ff = norm(f"l{i}.norm2"), sub(f"l{i}.mlp.", FEED_FORWARDS, l.ff, f"l{i}.rg2")
            lw.gate2 = dict(b=f(get(f"l{i}.rg2.b")))
        layers.append(lw)
    return HybridWeights(a(get("embed")), layers, norm("final.norm"), a(get("head")))


def is_checkpoint(path: str) -> bool:
    cj = os.path.join(path, "config.json")
    if not os.path.exists(cj):
        return False
    with open(cj) as fh:
        return json.load(fh).get("architecture") == ARCHITECTURE


def load(path: str, device="cpu", act_dtype=torch.bfloat16, max_position: int | None = None) -> HybridDecoder:
    with open(os.path.join(path, "config.json")) as fh:
        c = json.load(fh)
    tensors = _SafetensorsDir(path)
    ranks = {i: int(tensors.shape(f"l{i}.mix.a1")[0]) for i, l in enumerate(c["layers"]) if l["type"] == "gla"}
    cfg = config_from_dict(c, name=os.path.basename(path.rstrip("/")) or "lalasun",
                           max_position=max_position or 8192, gla_ranks=ranks)
    return HybridDecoder(cfg, pack_weights(cfg, tensors, device, act_dtype), device, max_position, act_dtype)


def save(cfg: HybridConfig, tensors: dict, path: str) -> None:
    """Write config.json + model.safetensors (bfloat16) — the layout :func:`load` reads."""
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(config_to_dict(cfg), fh, indent=1)
    save_file({k: v.to(torch.bfloat16).cpu().contiguous() for k, v in tensors.items()},
              os.path.join(path, "model.safetensors"))


def _preset(width, vocab, pattern, heads, kv_heads, dim, chunk, latent, window, gla, ff) -> dict:
    """pattern: one letter per layer — a = chunked attention, l = latent attention, g = gated linear attention; upper
    case = no feed-forward.  latent: (heads, dim, rot_dim, vdim, kv_rank); gla: (heads, dim, vdim)."""
    layers = []
    for ch in pattern:
        k = ch.lower()
        if k == "a":
            mixer, typ = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, scale=dim ** -0.5, mask=dict(size=chunk),
                              rot=dict(base=500000.0, dims=dim)), "attention"
        elif k == "l":
            lh, ld, lr, lv, rank = latent
            mixer, typ = dict(heads=lh, dim=ld, rot_dim=lr, vdim=lv, kv_rank=rank, scale=(ld + lr) ** -0.5,
                              mask=dict(size=window), rot=dict(base=100000.0, dims=lr)), "latent_attention"
        else:
            mixer, typ = dict(heads=gla[0], dim=gla[1], vdim=gla[2], tau=16.0, rank=16), "gla"
        layers.append(dict(type=typ, mixer=mixer, mlp=None if ch.isupper() else dict(kind="dense", ff=ff)))
    return dict(architecture=ARCHITECTURE, vocab=vocab, width=width, residual_mult=0.4, norm=dict(eps=1e-6), layers=layers)


# random-init presets (benchmarks, smoke runs); sizes in the range of real models' layers
PRESETS = {
    "lalasun-tiny": _preset(128, 512, "galG", 4, 2, 32, 40, (3, 32, 16, 32, 64), 24, (2, 32, 48), 320),
    "lalasun-1b": _preset(2048, 32768, "aglgaglg", 16, 4, 128, 1024, (16, 128, 64, 128, 512), 1024, (8, 128, 256), 8192),
    "lalasun-8b-layers": _preset(4096, 128256, "aglg", 32, 8, 128, 4096, (32, 128, 64, 128, 512), 4096, (16, 128, 256),
                                 14336),
}


def build(name_or_path: str, device="cpu", seed: int = 0, act_dtype=torch.bfloat16,
          max_position: int | None = None) -> HybridDecoder:
    if os.path.isdir(name_or_path):
        return load(name_or_path, device, act_dtype, max_position)
    cfg = config_from_dict(PRESETS[name_or_path], name=name_or_path, max_position=max_position or 8192)
    w = pack_weights(cfg, random_tensors(cfg, seed), device, act_dtype)
    return HybridDecoder(cfg, w, device, max_position, act_dtype)
