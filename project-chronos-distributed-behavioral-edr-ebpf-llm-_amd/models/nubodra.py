"""Nubodra: a hybrid decoder on a parallel residual stream: every layer has one layer norm (weight and bias), and its
mixer and its feed-forward both read that norm's output, x <- x + mixer(h) + ff(h).  Its layers mix tokens with full
causal grouped-query attention without rotation (queries and keys pass a short causal convolution, the values are the
convolved keys before their norm, queries and keys are scaled to unit RMS per head without weights, queries carry a
temperature that grows with the position, heads are gated by one sigmoid each) or with latent attention (queries through
a latent of their own, interleaved rotation with a scaled frequency ramp, a learned softmax sink per head), where a
layer may read the latents that an earlier one has cached.  The feed-forward is a gated unit with SiLU.

This module is the design's reader: ``config.json`` -> :class:`chronos.models.hybrid.HybridConfig`, the checkpoint's
tensor names -> the packed weights the hybrid kernels take, and random weights of the same shapes for benchmarks and
tests.  Everything computed lives in :mod:`chronos.models.hybrid` and :mod:`chronos.ops.hybrid`.

config.json:  architecture "Nubodra"; vocab, width, embedding.scale, norm.eps; layers[i] = {type, mixer{...}, mlp|null}
  type "attention":         mixer {heads, kv_heads, dim, vdim, conv, scale, q_temp{coef, every}}
  type "latent_attention":  mixer {heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, kv_from?,
                                   rot{base, dims, scaling{factor, original, fast, slow}}}
  mlp {kind "dense", ff}
(conv taps and q_rank may be left out: the stored tensors have them as a dimension)
tensors (bfloat16, [out, in]):  embed, head, final.norm (+ .b), l<i>.norm1 (+ .b), l<i>.mix.*, l<i>.mlp.gate / .up / .down
"""
from __future__ import annotations

import json
import os

import torch

from .hybrid import (FEED_FORWARDS, MIXERS, GluFFSpec, HybridConfig, HybridDecoder, HybridLayerWeights, HybridWeights,
                     LatentAttentionSpec, LayerSpec, WindowAttentionSpec, ff_rides_along)
from .zokunex import _SafetensorsDir

ARCHITECTURE = "Nubodra"


def config_from_dict(c: dict, name: str = "nubodra", max_position: int = 8192, dims: dict | None = None) -> HybridConfig:
    """``dims``: layer index -> the size config.json may leave out (an attention layer's convolution taps, a latent
    layer's q_rank), as a checkpoint's tensors have it."""
    layers = []
    for i, l in enumerate(c["layers"]):
        mx = l["mixer"]
        if l["type"] == "attention":
            heads, temp = int(mx["heads"]), mx.get("q_temp")
            mixer = WindowAttentionSpec(heads, int(mx.get("kv_heads", heads)), int(mx["dim"]), int(mx.get("vdim", mx["dim"])),
                                        float(mx["scale"]), sink=False, v_from_k=True, qk_norm_weight=False,
                                        conv=int(mx.get("conv", (dims or {}).get(i, 0))),
                                        q_temp=(float(temp["coef"]), float(temp["every"])) if temp else None)
            if mixer.heads % mixer.kv_heads:
                raise ValueError(f"layer {i}: heads must be a multiple of kv_heads")
            if mixer.vdim != mixer.dim:
                raise ValueError(f"layer {i}: the values are the keys, vdim must equal dim")
            if mixer.conv < 1:
                raise ValueError(f"layer {i}: the convolution needs its number of taps")
        elif l["type"] == "latent_attention":
            rot, src = mx.get("rot") or {}, mx.get("kv_from")
            sc = rot.get("scaling")
            mixer = LatentAttentionSpec(int(mx["heads"]), int(mx["dim"]), int(mx["rot_dim"]), int(mx["vdim"]),
                                        int(mx["kv_rank"]), float(mx["scale"]), float(rot.get("base", 10000.0)),
                                        int(rot.get("dims", mx["rot_dim"] if rot else 0)), rope_interleaved=True, two_term=True,
                                        gate=False, q_rank=int(mx.get("q_rank", (dims or {}).get(i, 0))), sink=True,
                                        kv_from=None if src is None else int(src),
                                        rope_scaling=("ramp", *(float(sc[k]) for k in ("factor", "original", "fast", "slow")))
                                        if sc else None)
            if mixer.rope_dims % 2 or mixer.rope_dims > mixer.rot_dim:
                raise ValueError(f"layer {i}: rot.dims must be even and at most rot_dim")
            if mixer.q_rank < 1:
                raise ValueError(f"layer {i}: the queries' latent needs its size")
        else:
            raise ValueError(f"layer {i}: unknown mixer type {l['type']!r}")
        mlp = l.get("mlp")
        if mlp is not None and mlp.get("kind", "dense") != "dense":
            raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
        layers.append(LayerSpec(mixer, GluFFSpec(int(mlp["ff"]), float("inf"), 1.0, 0.0) if mlp is not None else None))
    return HybridConfig(name=name, vocab_size=int(c["vocab"]), hidden_size=int(c["width"]), layers=layers,
                        norm_eps=float(c["norm"]["eps"]), max_position=max_position, architecture=ARCHITECTURE,
                        residual="parallel", norm="layer", embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)))


def config_to_dict(cfg: HybridConfig) -> dict:
    """The config.json form of a configuration (what :func:`config_from_dict` reads)."""
    layers = []
    for l in cfg.layers:
        m = l.mixer
        if m.kind == "window_attention":
            typ, mixer = "attention", dict(heads=m.heads, kv_heads=m.kv_heads, dim=m.dim, vdim=m.vdim, conv=m.conv, scale=m.scale)
            if m.q_temp:
                mixer["q_temp"] = dict(coef=m.q_temp[0], every=m.q_temp[1])
        else:
            typ, mixer = "latent_attention", dict(heads=m.heads, dim=m.dim, rot_dim=m.rot_dim, vdim=m.vdim, kv_rank=m.kv_rank,
                                                  q_rank=m.q_rank, scale=m.scale)
            if m.rope_dims:
                mixer["rot"] = dict(base=m.rope_base, dims=m.rope_dims)
            if m.rope_scaling:
                mixer["rot"]["scaling"] = dict(zip(("factor", "original", "fast", "slow"), m.rope_scaling[1:]))
            if m.kv_from is not None:
                mixer["kv_from"] = m.kv_from
        layers.append(dict(type=typ, mixer=mixer, mlp=dict(kind="dense", ff=l.ff.ff) if l.ff is not None else None))
    return dict(architecture=ARCHITECTURE, vocab=cfg.vocab_size, width=cfg.hidden_size, embedding=dict(scale=cfg.embed_scale),
                norm=dict(eps=cfg.norm_eps), layers=layers)


def tensor_shapes(cfg: HybridConfig) -> dict:
    """Checkpoint tensor name -> shape."""
    d, V = cfg.hidden_size, cfg.vocab_size
    norm = lambda p: {p: (d,), p + ".b": (d,)}  # noqa: E731
    out = {"embed": (V, d)}
    for i, l in enumerate(cfg.layers):
        m, p = l.mixer, f"l{i}."
        out.update(norm(p + "norm1"))
        hv = m.heads * m.vdim
        if m.kind == "window_attention":
            hq, gk = m.heads * m.dim, m.kv_heads * m.dim
            out.update({p + "mix.q": (hq, d), p + "mix.k": (gk, d), p + "mix.q.conv": (hq, m.conv), p + "mix.k.conv": (gk, m.conv),
                        p + "mix.g": (m.heads, d), p + "mix.o": (d, hv)})
        else:
            out.update({p + "mix.dq": (m.q_rank, d), p + "mix.dq.norm": (m.q_rank,),
                        p + "mix.uq": (m.heads * (m.dim + m.rot_dim), m.q_rank)})
            if m.kv_from is None:
                out.update({p + "mix.dkv": (m.kv_rank + m.rot_dim, d), p + "mix.dkv.norm": (m.kv_rank,)})
            out.update({p + "mix.uk": (m.heads * m.dim, m.kv_rank), p + "mix.uv": (hv, m.kv_rank), p + "mix.sink": (m.heads,),
                        p + "mix.o": (d, hv)})
        if l.ff is not None:
            out.update({p + "mlp.gate": (l.ff.ff, d), p + "mlp.up": (l.ff.ff, d), p + "mlp.down": (d, l.ff.ff)})
    out.update(norm("final.norm"))
    out["head"] = (V, d)
    return out


def random_tensors(cfg: HybridConfig, seed: int = 0, device="cpu", std: float | None = None) -> dict:
    """Checkpoint-named random bfloat16 tensors: norm weights near one, biases and sinks around zero, convolutions that
    lean on the newest token."""
    gen = torch.Generator(device="cpu")
    gen.manual_seed(seed)
    out = {}
    for name, shape in tensor_shapes(cfg).items():
        rn = lambda s=1.0: torch.randn(shape, generator=gen) * s  # noqa: E731
        if name.endswith(".conv"):
            t = rn(0.4)
            t[:, -1] += 0.8
        elif name.endswith(".sink"):
            t = rn(1.0)
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
    """``tensors``: a mapping (or any object with ``__getitem__``) from checkpoint names to tensors.  The feed-forward's
    two products join the mixer's first and last (they read the same norm and are added to the same stream)."""
    a = lambda x: x.to(device=device, dtype=act_dtype).contiguous()  # noqa: E731
    f = lambda x: x.to(device=device, dtype=torch.float32).contiguous()  # noqa: E731
    shapes = tensor_shapes(cfg)

    def get(name):
        t = tensors[name]
        if tuple(t.shape) != tuple(shapes[name]):
            raise ValueError(f"tensor {name}: shape {tuple(t.shape)}, the configuration says {tuple(shapes[name])}")
        return t

    norm = lambda n: f(torch.cat([get(n), get(n + ".b")]))  # noqa: E731
    sub = lambda p: {n[len(p):]: get(n) for n in shapes if n.startswith(p)}  # noqa: E731
    layers = []
    for i, l in enumerate(cfg.layers):
        mix, ff = sub(f"l{i}.mix."), sub(f"l{i}.mlp.")
        rides = ff_rides_along(l.mixer, l.ff)
        if rides:
            mix["ff"] = (l.ff, torch.cat([ff["gate"], ff["up"]], 0), ff["down"])
        lw = HybridLayerWeights(norm(f"l{i}.norm1"), MIXERS[l.mixer.kind][1](l.mixer, mix, device, act_dtype))
        if l.ff is not None and not rides:
            lw.ff = FEED_FORWARDS[l.ff.kind][1](l.ff, ff, device, act_dtype)
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
    dims = {i: int(tensors.shape(f"l{i}.mix.q.conv")[1] if l["type"] == "attention" else tensors.shape(f"l{i}.mix.dq")[0])
            for i, l in enumerate(c["layers"])}
    cfg = config_from_dict(c, name=os.path.basename(path.rstrip("/")) or "nubodra",
                           max_position=max_position or 8192, dims=dims)
    return HybridDecoder(cfg, pack_weights(cfg, tensors, device, act_dtype), device, max_position, act_dtype)


def save(cfg: HybridConfig, tensors: dict, path: str) -> None:
    """Write config.json + model.safetensors (bfloat16) — the layout :func:`load` reads."""
    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as fh:
        json.dump(config_to_dict(cfg), fh, indent=1)
    save_file({k: v.to(torch.bfloat16).cpu().contiguous() for k, v in tensors.items()},
              os.path.join(path, "model.safetensors"))


def _preset(width, vocab, pattern, heads, kv_heads, dim, latent, ff) -> dict:
    """pattern: one letter per layer — a = attention, l = latent attention, s = latent attention on the latents of the
    newest layer of kind l; upper case = no feed-forward.  latent: (heads, dim, rot_dim, vdim, kv_rank, q_rank)."""
    layers, own = [], 0
    for i, ch in enumerate(pattern):
        k = ch.lower()
        if k == "a":
            mixer, typ = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, conv=4, scale=dim ** -0.5,
                              q_temp=dict(coef=0.1, every=1024)), "attention"
        else:
            lh, ld, lr, lv, rank, qr = latent
            mixer, typ = dict(heads=lh, dim=ld, rot_dim=lr, vdim=lv, kv_rank=rank, q_rank=qr, scale=(ld + lr) ** -0.5,
                              rot=dict(base=500000.0, dims=lr,
                                       scaling=dict(factor=4.0, original=4096, fast=32.0, slow=1.0))), "latent_attention"
            if k == "s":
                mixer["kv_from"] = own
            else:
                own = i
        layers.append(dict(type=typ, mixer=mixer, mlp=None if ch.isupper() else dict(kind="dense", ff=ff)))
    return dict(architecture=ARCHITECTURE, vocab=vocab, width=width, embedding=dict(scale=2.0), norm=dict(eps=1e-5),
                layers=layers)


# random-init presets (benchmarks, smoke runs); sizes in the range of real models' layers
PRESETS = {
    "nubodra-tiny": _preset(128, 512, "alAs", 4, 2, 32, (3, 32, 16, 32, 64, 48), 320),
    "nubodra-1b": _preset(2048, 32768, "aalaasaa", 16, 4, 128, (16, 128, 64, 128, 512, 768), 5632),
    "nubodra-8b-layers": _preset(4096, 128256, "alas", 32, 8, 128, (32, 128, 64, 128, 512, 1536), 14336),
}


def build(name_or_path: str, device="cpu", seed: int = 0, act_dtype=torch.bfloat16,
          max_position: int | None = None) -> HybridDecoder:
    if os.path.isdir(name_or_path):
        return load(name_or_path, device, act_dtype, max_position)
    cfg = config_from_dict(PRESETS[name_or_path], name=name_or_path, max_position=max_position or 8192)
    w = pack_weights(cfg, random_tensors(cfg, seed), device, act_dtype)
    return HybridDecoder(cfg, w, device, max_position, act_dtype)
