"""Throughput of a hybrid design (Zokunex, Kalesun, Tugovik, Vogerax, Lalasun, Nubodra) beside the framework's other models at equal width and depth:
whole-model prefill and decode steps, and each of the design's kernels beside its closest existing kernel with the
fraction of its roofline it reaches.

``python bench.py --design-compare [--design zokunex|kalesun|tugovik|vogerax|lalasun|nubodra] [--design-sizes 1k,2k,4k]`` prints one JSON line
(the default benchmark and its output line are untouched).  Zokunex stands beside Llama; Kalesun beside Zokunex (the
closest family: recurrent layers, attention and mixtures of experts on a float32 stream) and Llama; Tugovik beside
Kalesun (masked grouped-query attention over paged keys and values, linear-state scans behind a short convolution,
gated experts, RMS norms on the stream) and Llama; Vogerax beside Kalesun too (windowed and causal sink attention on
the same kernels, a linear-state scan, RMS norms joined to a float32 stream) and Llama; Lalasun beside Kalesun (masked
sink attention, gated linear attention, dense feed-forwards), Zokunex (latent attention) and Llama; Nubodra beside
Kalesun (grouped-query attention over pages, short convolution, gated feed-forwards), Zokunex (causal latent attention)
and Llama.  Weights are random; every number is measured on the GPU this
process runs on.

Rooflines: HBM 8 TB/s for kernels bound by the bytes they must move, 2.5 PFLOP/s dense bf16 for the matrix-shaped
ones (the attention kernels over a long context are priced by their FLOPs in prefill and by their cache bytes in
decode, like the Llama kernels they stand beside).
"""
from __future__ import annotations

import json
import math
import sys
import time

import torch

HBM_BPS = 8.0e12
BF16_FLOPS = 2.5e15

# width -> (mlstm heads, dim, vdim | latent heads, dim, rot, vdim, rank | dense ff | experts, identity, top, expert ff)
SIZES = {
    "1k": dict(width=1024, m=(4, 128, 256), a=(8, 64, 32, 64, 256), ff=4096, moe=(8, 2, 2, 512)),
    "2k": dict(width=2048, m=(4, 256, 512), a=(16, 128, 64, 128, 512), ff=8192, moe=(16, 2, 4, 1408)),
    "4k": dict(width=4096, m=(8, 256, 512), a=(32, 128, 64, 128, 512), ff=14336, moe=(32, 2, 4, 2048)),
}
LAYERS = 4
VOCAB = 32768


def zokunex_config(size: dict) -> dict:
    mh, md, mv = size["m"]
    ah, ad, ar, av, rank = size["a"]
    ne, ni, top, eff = size["moe"]
    mix_m = dict(type="mlstm", mixer=dict(heads=mh, dim=md, vdim=mv, gate_cap=10.0))
    mix_a = dict(type="latent_attention", mixer=dict(heads=ah, dim=ad, rot_dim=ar, vdim=av, kv_rank=rank,
                                                     scale=(ad + ar) ** -0.5, rot=dict(base=10000.0, dims=ar)))
    dense = dict(kind="dense", ff=size["ff"])
    moe = dict(kind="moe", expert=dict(ff=eff), router=dict(experts=ne, identity=ni, top=top))
    layers = [dict(mix_m, mlp=dense), dict(mix_a, mlp=moe), dict(mix_m, mlp=moe), dict(mix_a, mlp=dense)][:LAYERS]
    return dict(architecture="Zokunex", vocab=VOCAB, width=size["width"], logit_scale=1.0, norm=dict(eps=1e-5),
                layers=layers)


# Kalesun: width -> (attention heads, kv heads, dim, vdim, window, kept | delta heads, qk heads, dim, vdim |
#                    gla heads, dim, vdim | dense ff | experts, top, expert ff)
KALESUN_SIZES = {
    "1k": dict(width=1024, a=(8, 2, 128, 128, 512, 4), d=(8, 4, 128, 128), g=(4, 128, 256), ff=2816, moe=(8, 2, 512)),
    "2k": dict(width=2048, a=(16, 4, 128, 128, 1024, 4), d=(16, 8, 128, 128), g=(8, 128, 256), ff=5632, moe=(16, 4, 1024)),
    "4k": dict(width=4096, a=(32, 8, 128, 128, 1024, 4), d=(32, 16, 128, 128), g=(16, 128, 256), ff=11008, moe=(32, 4, 1536)),
}


def kalesun_config(size: dict) -> dict:
    ah, ag, ad, av, win, keep = size["a"]
    dh, dk, dd, dv = size["d"]
    gh, gd, gv = size["g"]
    ne, top, eff = size["moe"]
    mix_a = dict(type="attention", mixer=dict(heads=ah, kv_heads=ag, dim=ad, vdim=av, scale=ad ** -0.5, v_mix=True,
                                              mask=dict(size=win, keep_first=keep),
                                              rot=dict(base=500000.0, dims=ad // 2,
                                                       scaling=dict(factor=8.0, low=1.0, high=4.0, original=8192))))
    mix_d = dict(type="delta", mixer=dict(heads=dh, kv_heads=dk, dim=dd, vdim=dv, conv=4))
    mix_g = dict(type="gla", mixer=dict(heads=gh, dim=gd, vdim=gv, tau=16.0, rank=16))
    dense = dict(kind="dense", ff=size["ff"], limit=7.0)
    moe = dict(kind="moe", expert=dict(ff=eff, limit=7.0), router=dict(experts=ne, top=top))
    layers = [dict(mix_d, mlp=dense), dict(mix_a, mlp=moe), dict(mix_g, mlp=moe), dict(mix_a, mlp=dense)][:LAYERS]
    return dict(architecture="Kalesun", vocab=VOCAB, width=size["width"], postln_alpha=2.0, norm=dict(eps=1e-6),
                layers=layers)

# Tugovik: width -> (attention heads, kv heads, dim, vdim, chunk | state-space heads, vdim, state, groups |
#                    recurrence width, blocks | experts, top, groups, kept, expert ff, shared ff | token-input columns)
TUGOVIK_SIZES = {
    "1k": dict(width=1024, a=(8, 2, 128, 128, 512), m=(32, 64, 128, 4), r=(1024, 4), moe=(8, 2, 4, 2, 512, 1024), side=128),
    "2k": dict(width=2048, a=(16, 4, 128, 128, 1024), m=(64, 64, 128, 8), r=(2048, 8), moe=(16, 4, 4, 2, 1024, 2048), side=256),
    "4k": dict(width=4096, a=(32, 8, 128, 128, 1024), m=(128, 64, 128, 8), r=(4096, 16), moe=(32, 4, 8, 4, 1536, 4096), side=256),
}


def tugovik_config(size: dict) -> dict:
    ah, ag, ad, av, chunk = size["a"]
    mh, mv, mn, mg = size["m"]
    rw, rb = size["r"]
    ne, top, ng, keep, eff, sff = size["moe"]
    mix_a = dict(type="attention", mixer=dict(heads=ah, kv_heads=ag, dim=ad, vdim=av, scale=ad ** -0.5, mask=dict(size=chunk)))
    mix_m = dict(type="mamba2", mixer=dict(heads=mh, vdim=mv, state=mn, groups=mg, conv=4, norm_groups=mg))
    mix_r = dict(type="rglru", mixer=dict(width=rw, blocks=rb, conv=4))
    moe = dict(kind="moe", expert=dict(ff=eff), shared=dict(ff=sff),
               router=dict(experts=ne, top=top, scale=2.5, groups=dict(count=ng, keep=keep)))
    layers = [dict(mix_m, mlp=moe), dict(mix_a, mlp=moe), dict(mix_r, mlp=moe), dict(mix_a, mlp=moe)][:LAYERS]
    return dict(architecture="Tugovik", vocab=VOCAB, width=size["width"], norm=dict(eps=1e-6), layers=layers,
                token_side=dict(dim=size["side"]))

# Vogerax: width -> (pooled attention heads, kv heads, dim, window, pool | sink attention heads, kv heads, dim, vdim |
#                    retention heads, dim, vdim | dense ff | experts, top, expert ff, shared ff | norm groups)
VOGERAX_SIZES = {
    "1k": dict(width=1024, a=(8, 2, 128, 512, 64), l=(8, 2, 128, 128), r=(8, 128, 128), ff=4096, moe=(8, 2, 512, 1024), groups=4),
    "2k": dict(width=2048, a=(16, 4, 128, 1024, 64), l=(16, 4, 128, 128), r=(16, 128, 128), ff=8192, moe=(16, 4, 1024, 2048), groups=4),
    "4k": dict(width=4096, a=(32, 8, 128, 1024, 64), l=(32, 8, 128, 128), r=(32, 128, 128), ff=14336, moe=(32, 4, 1536, 4096), groups=4),
}


def vogerax_config(size: dict) -> dict:
    ah, ag, ad, win, pool = size["a"]
    lh, lg, ld, lv = size["l"]
    rh, rd, rv = size["r"]
    ne, top, eff, sff = size["moe"]
    mix_a = dict(type="attention", mixer=dict(heads=ah, kv_heads=ag, dim=ad, vdim=ad, scale=ad ** -0.5,
                                              mask=dict(size=win, pool=pool),
                                              rot=dict(base=5e5, dims=ad // 2, scaling=dict(factor=4.0))))
    left = dict(heads=lh, kv_heads=lg, dim=ld, vdim=lv, scale=ld ** -0.5,
                rot=dict(base=1e5, dims=ld // 2, scaling=dict(factor=8.0, original=4096, fast=16.0, slow=2.0)))
    right = dict(heads=rh, dim=rd, vdim=rv, rot=dict(base=1e4, dims=rd),
                 decay=[math.exp(-1.0 / (16.0 * 128.0 ** (h / max(1, rh - 1)))) for h in range(rh)])
    mix_p = dict(type="parallel", mixer=dict(left=left, right=right))
    dense = dict(kind="dense", ff=size["ff"])
    moe = dict(kind="moe", expert=dict(ff=eff), shared=dict(ff=sff), router=dict(experts=ne, top=top))
    layers = [dict(mix_a, mlp=dense), dict(mix_p, mlp=moe), dict(mix_a, mlp=moe), dict(mix_p, mlp=dense)][:LAYERS]
    return dict(architecture="Vogerax", vocab=VOCAB, width=size["width"], norm=dict(eps=1e-6, groups=size["groups"]),
                embedding=dict(scale=8.0), layers=layers)


# Lalasun: width -> (attention heads, kv heads, dim, vdim, chunk | latent heads, dim, rot, vdim, rank, window |
#                    gla heads, dim, vdim | dense ff)
LALASUN_SIZES = {
    "1k": dict(width=1024, a=(8, 2, 128, 128, 512), l=(8, 64, 32, 64, 256, 512), g=(4, 128, 256), ff=4096),
    "2k": dict(width=2048, a=(16, 4, 128, 128, 1024), l=(16, 128, 64, 128, 512, 1024), g=(8, 128, 256), ff=8192),
    "4k": dict(width=4096, a=(32, 8, 128, 128, 1024), l=(32, 128, 64, 128, 512, 1024), g=(16, 128, 256), ff=14336),
}


def lalasun_config(size: dict) -> dict:
    ah, ag, ad, av, chunk = size["a"]
    lh, ld, lr, lv, rank, win = size["l"]
    gh, gd, gv = size["g"]
    mix_a = dict(type="attention", mixer=dict(heads=ah, kv_heads=ag, dim=ad, vdim=av, scale=ad ** -0.5, mask=dict(size=chunk),
                                              rot=dict(base=5e5, dims=ad)))
    mix_l = dict(type="latent_attention", mixer=dict(heads=lh, dim=ld, rot_dim=lr, vdim=lv, kv_rank=rank, scale=(ld + lr) ** -0.5,
                                                     mask=dict(size=win), rot=dict(base=1e5, dims=lr)))
    mix_g = dict(type="gla", mixer=dict(heads=gh, dim=gd, vdim=gv, tau=16.0, rank=16))
    mlp = dict(kind="dense", ff=size["ff"])
    layers = [dict(m, mlp=mlp) for m in (mix_g, mix_l, mix_a, mix_l)][:LAYERS]
    return dict(architecture="Lalasun", vocab=VOCAB, width=size["width"], residual_mult=0.4, norm=dict(eps=1e-6), layers=layers)


# Nubodra: width -> (attention heads, kv heads, dim, conv taps | latent heads, dim, rot, vdim, rank, query rank | dense ff)
NUBODRA_SIZES = {
    "1k": dict(width=1024, a=(8, 2, 128, 4), l=(8, 64, 32, 64, 256, 384), ff=2816),
    "2k": dict(width=2048, a=(16, 4, 128, 4), l=(16, 128, 64, 128, 512, 768), ff=5632),
    "4k": dict(width=4096, a=(32, 8, 128, 4), l=(32, 128, 64, 128, 512, 1536), ff=11008),
}


def nubodra_config(size: dict) -> dict:
    ah, ag, ad, taps = size["a"]
    lh, ld, lr, lv, rank, qr = size["l"]
    mix_a = dict(type="attention", mixer=dict(heads=ah, kv_heads=ag, dim=ad, vdim=ad, conv=taps, scale=ad ** -0.5,
                                              q_temp=dict(coef=0.1, every=1024)))
    lat = dict(heads=lh, dim=ld, rot_dim=lr, vdim=lv, kv_rank=rank, q_rank=qr, scale=(ld + lr) ** -0.5,
               rot=dict(base=5e5, dims=lr, scaling=dict(factor=4.0, original=4096, fast=32.0, slow=1.0)))
    mix_l = dict(type="latent_attention", mixer=lat)
    mix_s = dict(type="latent_attention", mixer=dict(lat, kv_from=1))
    mlp = dict(kind="dense", ff=size["ff"])
    layers = [dict(m, mlp=mlp) for m in (mix_a, mix_l, mix_a, mix_s)][:LAYERS]
    return dict(architecture="Nubodra", vocab=VOCAB, width=size["width"], embedding=dict(scale=2.0), norm=dict(eps=1e-6),
                layers=layers)


def _say(msg: str) -> None:
    print(f"[design-compare] {time.strftime('%H:%M:%S')} {msg}", file=sys.stderr, flush=True)


def _time(fn, iters: int = 10, warm: int = 2) -> float:
    for _ in range(warm):
        fn()
    torch.cuda.synchronize()
    a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
    a.record()
    for _ in range(iters):
        fn()
    b.record()
    torch.cuda.synchronize()
    return a.elapsed_time(b) / iters * 1e-3


def _graph(fn):
    fn()
    torch.cuda.synchronize()
    g = torch.cuda.CUDAGraph()
    with torch.cuda.graph(g):
        fn()
    return g.replay


def _model_steps(model, dev, seqs: int, plen: int, rows: int, ctx: int) -> dict:
    """Prefill of ``seqs`` prompts of ``plen`` tokens in one step; then decode steps of ``rows`` rows at context
    ``ctx`` (captured into a graph, as the engine runs them)."""
    from chronos.models.llama import StepBatch

    bs = 16
    need = max(seqs * plen, rows * (ctx + 1))
    nb = need // bs + rows + seqs + 2
    cache = model.make_cache(nb, bs, max(rows, seqs))
    vocab = model.cfg.vocab_size
    g = torch.Generator().manual_seed(0)
    per = (plen + bs - 1) // bs
    chunks = [torch.randint(0, vocab, (plen,), generator=g).tolist() for _ in range(seqs)]
    bts = [list(range(1 + b * per, 1 + (b + 1) * per)) for b in range(seqs)]
    sb = model.prefill_batch(chunks, [0] * seqs, bts, list(range(seqs)), max_blocks=per, nqt=8)
    t_pre = _time(lambda: model.forward(sb, cache), iters=3, warm=1)
    per = (ctx + 1 + bs - 1) // bs
    i32 = dict(dtype=torch.int32, device=dev)
    bt = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    ar = torch.arange(rows + 1, **i32)
    from chronos import ops

    dsb = StepBatch(torch.randint(0, vocab, (rows,), generator=g).to(dev).int(), torch.full((rows,), ctx, **i32),
                    ar[:rows], bt, ar, torch.full((rows,), ctx + 1, **i32), torch.arange(rows, device=dev), None, rows, 1,
                    ops.pick_nsplit(rows * model.hkv, ctx + 1), slots=ar[:rows].clone(), max_q=1)
    t_dec = _time(_graph(lambda: model.forward(dsb, cache)), iters=20)
    return dict(prefill_tokens_s=seqs * plen / t_pre, prefill_ms=t_pre * 1e3, decode_tokens_s=rows / t_dec,
                decode_ms=t_dec * 1e3)


def _kernels(size: dict, dev, T: int, ctx: int, rows: int) -> dict:
    """Each new kernel and its Llama counterpart at this size: seconds, and the fraction of the roofline reached."""
    from chronos import ops
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops

    out = {}
    bf = torch.bfloat16
    d = size["width"]
    g = torch.Generator(device=dev).manual_seed(1)
    rnd = lambda *s, dt=bf, sc=1.0: (torch.randn(*s, device=dev, generator=g) * sc).to(dt)  # noqa: E731
    i32 = dict(dtype=torch.int32, device=dev)

    def rec(name, secs, nbytes=0.0, flops=0.0):
        roof = max(nbytes / HBM_BPS, flops / BF16_FLOPS)
        _say(f"  {name}: {secs * 1e6:.1f} us, roofline {roof * 1e6:.2f} us")
        out[name] = dict(us=round(secs * 1e6, 1), roofline_us=round(roof * 1e6, 2), of_roofline=round(roof / secs, 4))

    # ---- norms on the residual stream
    y, x32, w32 = rnd(T, d), rnd(T, d, dt=torch.float32), rnd(d, dt=torch.float32)
    rec("add_layer_norm", _time(lambda: hops.add_layer_norm(y, x32, w32, 1e-5, bf)), T * d * (2 + 4 + 4 + 2))
    xb, wb = rnd(T, d), rnd(d)
    rec("llama.add_rmsnorm", _time(lambda: ops.add_rmsnorm(y, xb, wb, 1e-5)), T * d * (2 + 2 + 2 + 2))
    # ---- attention: prefill of T tokens (seqs of `ctx`), decode of `rows` rows at context ctx
    H, D, R, Dv, rank = size["a"]
    DK, bs = rank + R, 16
    seqs = max(1, T // ctx)
    per = ctx // bs + 1
    nb = max(seqs, rows) * per + 1
    cache = rnd(nb, bs, DK, sc=0.3)
    qa = rnd(seqs * ctx, H, DK, sc=0.3)
    gate = rnd(seqs * ctx, H, dt=torch.float32)
    bt = torch.arange(1, 1 + seqs * per, **i32).view(seqs, per)
    qs = torch.arange(0, (seqs + 1) * ctx, ctx, **i32)
    pos = torch.arange(ctx, **i32).repeat(seqs)
    pairs = seqs * ctx * (ctx + 1) / 2
    rec("latent_attention.prefill", _time(lambda: hops.latent_attention(qa, cache, bt, qs, pos, gate, 0.1, rank, bf, ctx), iters=3, warm=1),
        flops=2.0 * pairs * H * (DK + rank))
    btd = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    qsd = torch.arange(rows + 1, **i32)
    posd = torch.full((rows,), ctx, **i32)
    qad, gated = rnd(rows, H, DK, sc=0.3), rnd(rows, H, dt=torch.float32)
    rec("latent_attention.decode", _time(lambda: hops.latent_attention(qad, cache, btd, qsd, posd, gated, 0.1, rank, bf, 1)),
        nbytes=rows * (ctx + 1) * DK * 2.0)
    hq = d // 128
    hkv = max(1, hq // 4)
    kc, vc = rnd(nb, hkv, bs, 128, sc=0.3), rnd(nb, hkv, 128, bs, sc=0.3)
    q = rnd(seqs * ctx, hq, 128, sc=0.3)
    ctxl = torch.full((seqs,), ctx, **i32)
    tiles = torch.tensor(ops.attention_tiles([ctx] * seqs, hq, hkv, 8), **i32).view(-1, 2)
    rec("llama.attention.prefill", _time(lambda: ops.paged_attention(q, kc, vc, bt, qs, ctxl, tiles, tiles.shape[0], 8, 1), iters=3, warm=1),
        flops=4.0 * pairs * hq * 128)
    qd = rnd(rows, hq, 128, sc=0.3)
    ctxd = torch.full((rows,), ctx + 1, **i32)
    ns = ops.pick_nsplit(rows * hkv, ctx + 1)
    rec("llama.attention.decode", _time(lambda: ops.paged_attention(qd, kc, vc, btd, qsd, ctxd, None, rows, 1, ns)),
        nbytes=rows * (ctx + 1) * hkv * 128 * 2 * 2.0)
    # ---- the recurrence: prefill (FLOPs of the state update and read-out), decode (state bytes in and out)
    mh, md, mv = size["m"]
    C = 2 * mh * md + 2 * mh * mv
    proj = rnd(seqs * ctx, C, sc=0.5)
    gp = rnd(seqs * ctx, 2 * mh, dt=torch.float32)
    NS = max(seqs, rows) + 1
    S, n, m = (torch.zeros(NS, mh, md, mv, device=dev), torch.zeros(NS, mh, md, device=dev), torch.zeros(NS, mh, device=dev))
    p0 = torch.zeros(seqs, **i32)
    sl = torch.arange(seqs, **i32)
    rec("mlstm_scan.prefill", _time(lambda: hops.mlstm_scan(proj, gp, qs, p0, sl, S, n, m, mh, md, mv, 10.0, ctx), iters=3, warm=1),
        nbytes=seqs * ctx * C * 2.0, flops=seqs * ctx * mh * md * mv * 6.0)
    projd, gpd = rnd(rows, C, sc=0.5), rnd(rows, 2 * mh, dt=torch.float32)
    sld = torch.arange(rows, **i32)
    rec("mlstm_scan.decode", _time(lambda: hops.mlstm_scan(projd, gpd, qsd, posd, sld, S, n, m, mh, md, mv, 10.0, 1)),
        nbytes=rows * mh * md * mv * 4 * 2.0)
    # ---- feed-forwards: the mixture of experts beside a dense SwiGLU of the Llama model at this width
    ne, ni, top, eff = size["moe"]
    wr, corr = rnd(ne + ni, d, sc=0.05), rnd(ne + ni, dt=torch.float32, sc=0.01)
    wu, wd = rnd(ne, eff, d, sc=d ** -0.5), rnd(ne, d, eff, sc=eff ** -0.5)
    for name, tk in (("prefill", T), ("decode", rows)):
        h = rnd(tk, d)
        idx, wt = hops.moe_route(h, wr, corr, top)
        rec(f"moe_route.{name}", _time(lambda: hops.moe_route(h, wr, corr, top)), nbytes=tk * d * 2.0 + (ne + ni) * d * 2.0)
        real = float((idx < ne).sum())
        used = min(ne, real) * 2 * eff * d * 2.0
        rec(f"moe_ffn.{name}", _time(lambda: hops.moe_ffn(h, idx, wt, wu, wd, 1, bf), iters=3, warm=1),
            nbytes=used + tk * d * 4.0, flops=real * 4.0 * eff * d)
        f = int(3.5 * d)
        wgu, wdn = rnd(2 * f, d, sc=d ** -0.5), rnd(d, f, sc=f ** -0.5)
        rec(f"llama.mlp.{name}", _time(lambda: ops.linear(ops.gate_up_silu(h, wgu), wdn), iters=3, warm=1),
            nbytes=3 * f * d * 2.0 + tk * d * 4.0, flops=tk * 6.0 * f * d)
    return out


def _kernels_kalesun(size: dict, zsize: dict, dev, T: int, ctx: int, rows: int) -> dict:
    """Kalesun's kernels and their closest existing kernels at this size: seconds, and the fraction of the roofline
    reached.  ``zsize``: the Zokunex sizes of the same width (for the kernels it stands beside)."""
    from chronos import ops
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops

    out = {}
    bf = torch.bfloat16
    d = size["width"]
    g = torch.Generator(device=dev).manual_seed(1)
    rnd = lambda *s, dt=bf, sc=1.0: (torch.randn(*s, device=dev, generator=g) * sc).to(dt)  # noqa: E731
    i32 = dict(dtype=torch.int32, device=dev)

    def rec(name, secs, nbytes=0.0, flops=0.0):
        roof = max(nbytes / HBM_BPS, flops / BF16_FLOPS)
        _say(f"  {name}: {secs * 1e6:.1f} us, roofline {roof * 1e6:.2f} us")
        out[name] = dict(us=round(secs * 1e6, 1), roofline_us=round(roof * 1e6, 2), of_roofline=round(roof / secs, 4))

    # ---- norms on the residual stream
    y, x32, w32 = rnd(T, d), rnd(T, d, dt=torch.float32), rnd(d, dt=torch.float32)
    rec("scale_add_rms_norm", _time(lambda: hops.scale_add_rms_norm(y, x32, w32, 2.0, 1e-6, bf)), T * d * (2 + 4 + 4 + 2))
    rec("zokunex.add_layer_norm", _time(lambda: hops.add_layer_norm(y, x32, w32, 1e-5, bf)), T * d * (2 + 4 + 4 + 2))
    xb, wb = rnd(T, d), rnd(d)
    rec("llama.add_rmsnorm", _time(lambda: ops.add_rmsnorm(y, xb, wb, 1e-5)), T * d * (2 + 2 + 2 + 2))
    # ---- attention: prefill of T tokens (seqs of `ctx`), decode of `rows` rows at context ctx
    H, G, D, Dv, win, keep = size["a"]
    bs = 16
    seqs = max(1, T // ctx)
    per = ctx // bs + 1
    nb = max(seqs, rows) * per + 1
    kc, vc = rnd(nb, bs, G, D, sc=0.3), rnd(nb, bs, G, Dv, sc=0.3)
    C = (H + G) * D + G * Dv
    qkv = rnd(seqs * ctx, C, sc=0.3)
    gate, sink = rnd(seqs * ctx, H, dt=torch.float32), rnd(H, dt=torch.float32)
    bt = torch.arange(1, 1 + seqs * per, **i32).view(seqs, per)
    qs = torch.arange(0, (seqs + 1) * ctx, ctx, **i32)
    pos = torch.arange(ctx, **i32).repeat(seqs)
    tseq = torch.arange(seqs, **i32).repeat_interleave(ctx)
    vis = sum(min(i + 1, win) + max(0, min(keep, i + 1 - win)) for i in range(ctx))  # visible (query, key) pairs
    pairs = seqs * vis
    rec("window_attention.prefill", _time(lambda: hops.window_attention(qkv, kc, vc, bt, qs, pos, sink, gate, D ** -0.5, win, keep, H, bf, ctx), iters=3, warm=1),
        flops=2.0 * pairs * H * (D + Dv))
    cs = rope_cos_sin(500000.0, D // 2, ctx + 1, dev, (8.0, 1.0, 4.0, 8192.0))
    qn, vf, lam = rnd(D, dt=torch.float32), rnd(seqs * ctx, G * Dv), torch.tensor([0.3], device=dev)
    rec("window_prep.prefill", _time(lambda: hops.window_prep(qkv, H, G, D, Dv, vf, lam, pos, tseq, bt, qn, qn, 1e-6, cs, D // 2, kc, vc, False)),
        nbytes=seqs * ctx * (C * 2 + H * D * 2 + 2 * G * (D + Dv) * 2.0))
    btd = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    qsd = torch.arange(rows + 1, **i32)
    posd = torch.full((rows,), ctx, **i32)
    qkvd, gated = rnd(rows, C, sc=0.3), rnd(rows, H, dt=torch.float32)
    rec("window_attention.decode", _time(lambda: hops.window_attention(qkvd, kc, vc, btd, qsd, posd, sink, gated, D ** -0.5, win, keep, H, bf, 1)),
        nbytes=rows * (min(ctx + 1, win) + keep) * G * (D + Dv) * 2.0)
    # beside: Llama's paged GQA attention (full causal) and Zokunex's latent attention at this width
    hq = d // 128
    hkv = max(1, hq // 4)
    lkc, lvc = rnd(nb, hkv, bs, 128, sc=0.3), rnd(nb, hkv, 128, bs, sc=0.3)
    q = rnd(seqs * ctx, hq, 128, sc=0.3)
    ctxl = torch.full((seqs,), ctx, **i32)
    tiles = torch.tensor(ops.attention_tiles([ctx] * seqs, hq, hkv, 8), **i32).view(-1, 2)
    full_pairs = seqs * ctx * (ctx + 1) / 2
    rec("llama.attention.prefill", _time(lambda: ops.paged_attention(q, lkc, lvc, bt, qs, ctxl, tiles, tiles.shape[0], 8, 1), iters=3, warm=1),
        flops=4.0 * full_pairs * hq * 128)
    qd = rnd(rows, hq, 128, sc=0.3)
    ctxd = torch.full((rows,), ctx + 1, **i32)
    ns = ops.pick_nsplit(rows * hkv, ctx + 1)
    rec("llama.attention.decode", _time(lambda: ops.paged_attention(qd, lkc, lvc, btd, qsd, ctxd, None, rows, 1, ns)),
        nbytes=rows * (ctx + 1) * hkv * 128 * 2 * 2.0)
    zh, zd, zr, zv, rank = zsize["a"]
    DK = rank + zr
    lat = rnd(nb, bs, DK, sc=0.3)
    qa, zg = rnd(seqs * ctx, zh, DK, sc=0.3), rnd(seqs * ctx, zh, dt=torch.float32)
    rec("zokunex.latent_attention.prefill", _time(lambda: hops.latent_attention(qa, lat, bt, qs, pos, zg, 0.1, rank, bf, ctx), iters=3, warm=1),
        flops=2.0 * full_pairs * zh * (DK + rank))
    qad, zgd = rnd(rows, zh, DK, sc=0.3), rnd(rows, zh, dt=torch.float32)
    rec("zokunex.latent_attention.decode", _time(lambda: hops.latent_attention(qad, lat, btd, qsd, posd, zgd, 0.1, rank, bf, 1)),
        nbytes=rows * (ctx + 1) * DK * 2.0)
    # ---- the recurrences: prefill (FLOPs of the state update and read-out), decode (state bytes in and out)
    NS = max(seqs, rows) + 1
    p0, sl, sld = torch.zeros(seqs, **i32), torch.arange(seqs, **i32), torch.arange(rows, **i32)
    for name, (hh, hk, dd, dv), delta in (("delta", size["d"], True), ("gla", (size["g"][0], size["g"][0], *size["g"][1:]), False)):
        Cq = 2 * hk * dd + hh * dv
        S = torch.zeros(NS, hh, dd, dv, device=dev)

        def scan(proj, qs_, p0_, sl_, n):
            if delta:
                qsc, ksc = torch.rand(n, hk, device=dev), torch.rand(n, hk, device=dev)
                dec, beta = torch.rand(n, hh, device=dev), torch.rand(n, hh, device=dev)
                return lambda: hops.linear_scan(proj, 0, hk * dd, 2 * hk * dd, qsc, ksc, 1.0, dec, beta, qs_, p0_, sl_, S, hk, hh, dd, dv)
            dec = torch.rand(n, hh, dd, device=dev)
            return lambda: hops.linear_scan(proj, 0, hk * dd, 2 * hk * dd, None, None, dd ** -0.5, dec, None, qs_, p0_, sl_, S, hk, hh, dd, dv)

        proj = rnd(seqs * ctx, Cq, sc=0.5)
        rec(f"linear_scan.{name}.prefill", _time(scan(proj, qs, p0, sl, seqs * ctx), iters=3, warm=1),
            nbytes=seqs * ctx * Cq * 2.0, flops=seqs * ctx * hh * dd * dv * (6.0 if delta else 4.0))
        projd = rnd(rows, Cq, sc=0.5)
        rec(f"linear_scan.{name}.decode", _time(scan(projd, qsd, posd, sld, rows)), nbytes=rows * hh * dd * dv * 4 * 2.0)
    dh, dk, dd, dv = size["d"]
    Cc = 2 * dk * dd + dh * dv
    xc, taps = rnd(seqs * ctx, Cc + dh * dv), rnd(Cc, 4, dt=torch.float32)
    hist = torch.zeros(NS, 3, Cc, device=dev, dtype=bf)
    rec("short_conv.prefill", _time(lambda: hops.short_conv(xc, taps, tseq, qs, p0, sl, hist, True)), nbytes=seqs * ctx * Cc * 4.0)
    mh, md, mv = zsize["m"]
    Cm = 2 * mh * md + 2 * mh * mv
    mproj, gp = rnd(seqs * ctx, Cm, sc=0.5), rnd(seqs * ctx, 2 * mh, dt=torch.float32)
    mS, mn, mm = (torch.zeros(NS, mh, md, mv, device=dev), torch.zeros(NS, mh, md, device=dev), torch.zeros(NS, mh, device=dev))
    rec("zokunex.mlstm_scan.prefill", _time(lambda: hops.mlstm_scan(mproj, gp, qs, p0, sl, mS, mn, mm, mh, md, mv, 10.0, ctx), iters=3, warm=1),
        nbytes=seqs * ctx * Cm * 2.0, flops=seqs * ctx * mh * md * mv * 6.0)
    mprojd, gpd = rnd(rows, Cm, sc=0.5), rnd(rows, 2 * mh, dt=torch.float32)
    rec("zokunex.mlstm_scan.decode", _time(lambda: hops.mlstm_scan(mprojd, gpd, qsd, posd, sld, mS, mn, mm, mh, md, mv, 10.0, 1)),
        nbytes=rows * mh * md * mv * 4 * 2.0)
    # ---- feed-forwards: gated experts beside Zokunex's experts and Llama's dense SwiGLU; the gated unit's activation
    ne, top, eff = size["moe"]
    wr, br = rnd(ne, d, sc=0.05), rnd(ne, dt=torch.float32, sc=0.01)
    wgu = rnd(ne, 2 * eff, d, sc=d ** -0.5)[:, hops.moe_glu_row_order(eff).to(dev)].contiguous()
    wd = rnd(ne, d, eff, sc=eff ** -0.5)
    ze, zi, ztop, zeff = zsize["moe"]
    zwr, zcorr = rnd(ze + zi, d, sc=0.05), rnd(ze + zi, dt=torch.float32, sc=0.01)
    zwu, zwd = rnd(ze, zeff, d, sc=d ** -0.5), rnd(ze, d, zeff, sc=zeff ** -0.5)
    for name, tk in (("prefill", T), ("decode", rows)):
        h = rnd(tk, d)
        idx, wt = hops.moe_route_topk(h, wr, br, top)
        rec(f"moe_route_topk.{name}", _time(lambda: hops.moe_route_topk(h, wr, br, top)), nbytes=tk * d * 2.0 + ne * d * 2.0)
        used = min(ne, tk * top) * 3 * eff * d * 2.0
        rec(f"moe_glu_ffn.{name}", _time(lambda: hops.moe_glu_ffn(h, idx, wt, wgu, wd, 7.0, 1.702, 1.0, bf, True), iters=3, warm=1),
            nbytes=used + tk * d * 4.0, flops=tk * top * 6.0 * eff * d)
        zidx, zwt = hops.moe_route(h, zwr, zcorr, ztop)
        real = float((zidx < ze).sum())
        rec(f"zokunex.moe_ffn.{name}", _time(lambda: hops.moe_ffn(h, zidx, zwt, zwu, zwd, 1, bf), iters=3, warm=1),
            nbytes=min(ze, real) * 2 * zeff * d * 2.0 + tk * d * 4.0, flops=real * 4.0 * zeff * d)
        f = size["ff"]
        gu = rnd(tk, 2 * f)
        rec(f"glu.{name}", _time(lambda: hops.glu(gu, 7.0, 1.702, 1.0, bf)), nbytes=tk * f * 6.0)
        lf = int(3.5 * d)
        wgl, wdn = rnd(2 * lf, d, sc=d ** -0.5), rnd(d, lf, sc=lf ** -0.5)
        rec(f"llama.mlp.{name}", _time(lambda: ops.linear(ops.gate_up_silu(h, wgl), wdn), iters=3, warm=1),
            nbytes=3 * lf * d * 2.0 + tk * d * 4.0, flops=tk * 6.0 * lf * d)
    return out


def _kernels_tugovik(size: dict, ksize: dict, dev, T: int, ctx: int, rows: int) -> dict:
    """Tugovik's kernels and their closest existing kernels at this size: seconds, and the fraction of the roofline
    reached.  ``ksize``: the Kalesun sizes of the same width (for the kernels it stands beside)."""
    from chronos import ops
    from chronos.ops import hybrid as hops

    out = {}
    bf = torch.bfloat16
    d = size["width"]
    g = torch.Generator(device=dev).manual_seed(1)
    rnd = lambda *s, dt=bf, sc=1.0: (torch.randn(*s, device=dev, generator=g) * sc).to(dt)  # noqa: E731
    i32 = dict(dtype=torch.int32, device=dev)

    def rec(name, secs, nbytes=0.0, flops=0.0):
        roof = max(nbytes / HBM_BPS, flops / BF16_FLOPS)
        _say(f"  {name}: {secs * 1e6:.1f} us, roofline {roof * 1e6:.2f} us")
        out[name] = dict(us=round(secs * 1e6, 1), roofline_us=round(roof * 1e6, 2), of_roofline=round(roof / secs, 4))

    bs = 16
    seqs = max(1, T // ctx)
    per = ctx // bs + 1
    nb = max(seqs, rows) * per + 1
    bt = torch.arange(1, 1 + seqs * per, **i32).view(seqs, per)
    qs = torch.arange(0, (seqs + 1) * ctx, ctx, **i32)
    pos = torch.arange(ctx, **i32).repeat(seqs)
    tseq = torch.arange(seqs, **i32).repeat_interleave(ctx)
    btd = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    qsd = torch.arange(rows + 1, **i32)
    posd = torch.full((rows,), ctx, **i32)
    tseqd = torch.arange(rows, **i32)
    NS = max(seqs, rows) + 1
    p0, sl, sld = torch.zeros(seqs, **i32), torch.arange(seqs, **i32), torch.arange(rows, **i32)
    # ---- the stream's joins
    y, y2, x32, w32 = rnd(T, d), rnd(T, d), rnd(T, d, dt=torch.float32), rnd(d, dt=torch.float32)
    g2 = rnd(T, 1, dt=torch.float32)
    rec("add_rms_norm", _time(lambda: hops.add_rms_norm(y, x32, w32, 1e-6, bf)), T * d * (2 + 4 + 4 + 2))
    rec("add_rms_norm.gated_pair", _time(lambda: hops.add_rms_norm(y, x32, None, 1e-6, bf, y2, g2)), T * d * (2 + 2 + 4 + 4 + 2))
    rec("add_rms_norm.normed_addend", _time(lambda: hops.add_rms_norm(y, x32, w32, 1e-6, bf, w_y=w32)), T * d * (2 + 4 + 4 + 2))
    rec("kalesun.scale_add_rms_norm", _time(lambda: hops.scale_add_rms_norm(y, x32, w32, 1.0, 1e-6, bf)), T * d * (2 + 4 + 4 + 2))
    xb, wb = rnd(T, d), rnd(d)
    rec("llama.add_rmsnorm", _time(lambda: ops.add_rmsnorm(y, xb, wb, 1e-5)), T * d * (2 + 2 + 2 + 2))
    sd = size["side"]
    a_, table, ids = rnd(T, sd), rnd(VOCAB, 4 * sd), torch.randint(0, VOCAB, (T,), device=dev, generator=g).int()
    rec("token_gate", _time(lambda: hops.token_gate(a_, ids, table, sd, bf)), T * sd * 6.0)
    # ---- attention: the chunk mask beside Kalesun's window of the same span (with sink and gate) and Llama's
    H, G, D, Dv, chunk = size["a"]
    kc, vc = rnd(nb, bs, G, D, sc=0.3), rnd(nb, bs, G, Dv, sc=0.3)
    C = (H + G) * D + G * Dv
    qkv = rnd(seqs * ctx, C, sc=0.3)
    vis = sum(i % chunk + 1 for i in range(ctx))
    rec("chunk_attention.prefill", _time(lambda: hops.window_attention(qkv, kc, vc, bt, qs, pos, None, None, D ** -0.5, 0, 0, H, bf, ctx, chunk), iters=3, warm=1),
        flops=2.0 * seqs * vis * H * (D + Dv))
    rec("window_prep.plain.prefill", _time(lambda: hops.window_prep(qkv, H, G, D, Dv, None, None, pos, tseq, bt, None, None, 1e-6, None, 0, kc, vc, False)),
        nbytes=seqs * ctx * 2 * G * (D + Dv) * 2.0)
    qkvd = rnd(rows, C, sc=0.3)
    rec("chunk_attention.decode", _time(lambda: hops.window_attention(qkvd, kc, vc, btd, qsd, posd, None, None, D ** -0.5, 0, 0, H, bf, 1, chunk)),
        nbytes=rows * (ctx % chunk + 1) * G * (D + Dv) * 2.0)
    posm = torch.full((rows,), ctx // chunk * chunk + chunk - 1, **i32)   # the last position of a chunk: every key of it
    btm = torch.arange(1, 1 + rows * (per + chunk // bs), **i32).view(rows, -1) % (nb - 1) + 1
    rec("chunk_attention.decode_full_chunk", _time(lambda: hops.window_attention(qkvd, kc, vc, btm, qsd, posm, None, None, D ** -0.5, 0, 0, H, bf, 1, chunk)),
        nbytes=rows * chunk * G * (D + Dv) * 2.0)
    kH, kG, kD, kDv, win, keep = ksize["a"]
    kkc, kvc = rnd(nb, bs, kG, kD, sc=0.3), rnd(nb, bs, kG, kDv, sc=0.3)
    kqkv = rnd(seqs * ctx, (kH + kG) * kD + kG * kDv, sc=0.3)
    kgate, ksink = rnd(seqs * ctx, kH, dt=torch.float32), rnd(kH, dt=torch.float32)
    kvis = sum(min(i + 1, win) + max(0, min(keep, i + 1 - win)) for i in range(ctx))
    rec("kalesun.window_attention.prefill", _time(lambda: hops.window_attention(kqkv, kkc, kvc, bt, qs, pos, ksink, kgate, kD ** -0.5, win, keep, kH, bf, ctx), iters=3, warm=1),
        flops=2.0 * seqs * kvis * kH * (kD + kDv))
    kqkvd, kgated = rnd(rows, (kH + kG) * kD + kG * kDv, sc=0.3), rnd(rows, kH, dt=torch.float32)
    rec("kalesun.window_attention.decode", _time(lambda: hops.window_attention(kqkvd, kkc, kvc, btd, qsd, posd, ksink, kgated, kD ** -0.5, win, keep, kH, bf, 1)),
        nbytes=rows * (min(ctx + 1, win) + keep) * kG * (kD + kDv) * 2.0)
    hq = d // 128
    hkv = max(1, hq // 4)
    lkc, lvc = rnd(nb, hkv, bs, 128, sc=0.3), rnd(nb, hkv, 128, bs, sc=0.3)
    q = rnd(seqs * ctx, hq, 128, sc=0.3)
    ctxl = torch.full((seqs,), ctx, **i32)
    tiles = torch.tensor(ops.attention_tiles([ctx] * seqs, hq, hkv, 8), **i32).view(-1, 2)
    rec("llama.attention.prefill", _time(lambda: ops.paged_attention(q, lkc, lvc, bt, qs, ctxl, tiles, tiles.shape[0], 8, 1), iters=3, warm=1),
        flops=4.0 * seqs * ctx * (ctx + 1) / 2 * hq * 128)
    qd = rnd(rows, hq, 128, sc=0.3)
    ctxd = torch.full((rows,), ctx + 1, **i32)
    ns = ops.pick_nsplit(rows * hkv, ctx + 1)
    rec("llama.attention.decode", _time(lambda: ops.paged_attention(qd, lkc, lvc, btd, qsd, ctxd, None, rows, 1, ns)),
        nbytes=rows * (ctx + 1) * hkv * 128 * 2 * 2.0)
    # ---- the state-space layer: convolution, per-token scalars, scan, gated group norm
    mh, mv, mn, mg = size["m"]
    inner, Cc = mh * mv, mh * mv + 2 * mg * mn
    proj, taps, cb = rnd(seqs * ctx, inner + Cc, sc=0.5), rnd(Cc, 4, dt=torch.float32), rnd(Cc, dt=torch.float32)
    hist = torch.zeros(NS, 3, Cc, device=dev, dtype=bf)
    rec("short_conv.bias.prefill", _time(lambda: hops.short_conv(proj, taps, tseq, qs, p0, sl, hist, True, cb, inner)),
        nbytes=seqs * ctx * Cc * 4.0)
    xbc = hops.short_conv(proj, taps, tseq, qs, p0, sl, hist, True, cb, inner)
    dtp, alog = rnd(seqs * ctx, mh, dt=torch.float32), rnd(mh, dt=torch.float32, sc=0.3)
    rec("ssm_prep.prefill", _time(lambda: hops.ssm_prep(dtp, alog)), nbytes=seqs * ctx * mh * 12.0)
    decay, dts = hops.ssm_prep(dtp, alog)
    S = torch.zeros(NS, mh, mn, mv, device=dev)
    rec("linear_scan.ssm.prefill", _time(lambda: hops.linear_scan(xbc, inner + mg * mn, inner, 0, None, None, 1.0, decay, None, qs, p0, sl, S, mg, mh, mn, mv, dts), iters=3, warm=1),
        nbytes=seqs * ctx * Cc * 2.0, flops=seqs * ctx * mh * mn * mv * 4.0)
    xbcd = rnd(rows, Cc, sc=0.5)
    decd, dtd = torch.rand(rows, mh, device=dev), torch.rand(rows, mh, device=dev)
    rec("linear_scan.ssm.decode", _time(lambda: hops.linear_scan(xbcd, inner + mg * mn, inner, 0, None, None, 1.0, decd, None, qsd, posd, sld, S, mg, mh, mn, mv, dtd)),
        nbytes=rows * mh * mn * mv * 4 * 2.0)
    o = torch.randn(seqs * ctx, mh, mv, device=dev)
    skip, nw = rnd(mh, dt=torch.float32), rnd(inner, dt=torch.float32)
    rec("gated_group_norm.prefill", _time(lambda: hops.gated_group_norm(o, xbc, 0, skip, proj, 0, nw, mg, 1e-6, bf)),
        nbytes=seqs * ctx * inner * (4 + 2 + 2 + 2.0))
    rec("kalesun.head_norm_gate.prefill", _time(lambda: hops.head_norm_gate(o, proj, 0, nw, 1e-6, True, bf)),
        nbytes=seqs * ctx * inner * (4 + 2 + 2.0))
    for name, (hh, hk, dd, dv), delta in (("delta", ksize["d"], True), ("gla", (ksize["g"][0], ksize["g"][0], *ksize["g"][1:]), False)):
        Cq = 2 * hk * dd + hh * dv
        kS = torch.zeros(NS, hh, dd, dv, device=dev)

        def scan(pr, qs_, p0_, sl_, n):
            if delta:
                qsc, ksc = torch.rand(n, hk, device=dev), torch.rand(n, hk, device=dev)
                dec, beta = torch.rand(n, hh, device=dev), torch.rand(n, hh, device=dev)
                return lambda: hops.linear_scan(pr, 0, hk * dd, 2 * hk * dd, qsc, ksc, 1.0, dec, beta, qs_, p0_, sl_, kS, hk, hh, dd, dv)
            dec = torch.rand(n, hh, dd, device=dev)
            return lambda: hops.linear_scan(pr, 0, hk * dd, 2 * hk * dd, None, None, dd ** -0.5, dec, None, qs_, p0_, sl_, kS, hk, hh, dd, dv)

        kp = rnd(seqs * ctx, Cq, sc=0.5)
        rec(f"kalesun.linear_scan.{name}.prefill", _time(scan(kp, qs, p0, sl, seqs * ctx), iters=3, warm=1),
            nbytes=seqs * ctx * Cq * 2.0, flops=seqs * ctx * hh * dd * dv * (6.0 if delta else 4.0))
        kpd = rnd(rows, Cq, sc=0.5)
        rec(f"kalesun.linear_scan.{name}.decode", _time(scan(kpd, qsd, posd, sld, rows)), nbytes=rows * hh * dd * dv * 4 * 2.0)
    # ---- the gated linear recurrence: block-diagonal gate projections (float32 library product) and the scan
    rw, rb = size["r"]
    bw = rw // rb
    yx = rnd(seqs * ctx, 2 * rw, sc=0.5)
    u = rnd(seqs * ctx, rw, sc=0.5)
    wg, bg = rnd(rb, bw, 2 * bw, sc=bw ** -0.5), rnd(rb, 1, 2 * bw, dt=torch.float32)   # bfloat16 weights, float32 out
    rec("block_gates.prefill", _time(lambda: hops.block_gates(u, wg, bg), iters=3, warm=1),
        nbytes=seqs * ctx * rw * (2 + 8.0), flops=seqs * ctx * rw * bw * 4.0)
    gates = hops.block_gates(u, wg, bg)
    sp = torch.rand(rw, device=dev)
    Sr = torch.zeros(NS, rw, device=dev)
    rec("rglru_scan.prefill", _time(lambda: hops.rglru_scan(u, gates, sp, 8.0, yx, 0, qs, p0, sl, Sr, bf, ctx), iters=3, warm=1),
        nbytes=seqs * ctx * rw * (8 + 2 + 2 + 2.0))
    ud, yxd = rnd(rows, rw, sc=0.5), rnd(rows, 2 * rw, sc=0.5)
    rec("block_gates.decode", _time(lambda: hops.block_gates(ud, wg, bg)), nbytes=rb * bw * 2 * bw * 4.0)
    gd = hops.block_gates(ud, wg, bg)
    rec("rglru_scan.decode", _time(lambda: hops.rglru_scan(ud, gd, sp, 8.0, yxd, 0, qsd, posd, sld, Sr, bf, 1)),
        nbytes=rows * rw * (8 + 2 + 2 + 2 + 8.0))
    # ---- feed-forwards: the grouped sigmoid router beside the top-k softmax router; the experts are Kalesun's kernel
    ne, top, ng, keep, eff, sff = size["moe"]
    wr, br = rnd(ne, d, sc=0.05), rnd(ne, dt=torch.float32, sc=0.01)
    wgu = rnd(ne, 2 * eff, d, sc=d ** -0.5)[:, hops.moe_glu_row_order(eff).to(dev)].contiguous()
    wd = rnd(ne, d, eff, sc=eff ** -0.5)
    inf = float("inf")
    for name, tk in (("prefill", T), ("decode", rows)):
        h = rnd(tk, d)
        rec(f"moe_route_group.{name}", _time(lambda: hops.moe_route_group(h, wr, top, ng, keep, 2.5)), nbytes=tk * d * 2.0 + ne * d * 2.0)
        rec(f"kalesun.moe_route_topk.{name}", _time(lambda: hops.moe_route_topk(h, wr, br, top)), nbytes=tk * d * 2.0 + ne * d * 2.0)
        idx, wt = hops.moe_route_group(h, wr, top, ng, keep, 2.5)
        used = min(ne, tk * top) * 3 * eff * d * 2.0
        rec(f"moe_glu_ffn.silu.{name}", _time(lambda: hops.moe_glu_ffn(h, idx, wt, wgu, wd, inf, 1.0, 0.0, bf, True), iters=3, warm=1),
            nbytes=used + tk * d * 4.0, flops=tk * top * 6.0 * eff * d)
        rec(f"kalesun.moe_glu_ffn.{name}", _time(lambda: hops.moe_glu_ffn(h, idx, wt, wgu, wd, 7.0, 1.702, 1.0, bf, True), iters=3, warm=1),
            nbytes=used + tk * d * 4.0, flops=tk * top * 6.0 * eff * d)
        lf = int(3.5 * d)
        wgl, wdn = rnd(2 * lf, d, sc=d ** -0.5), rnd(d, lf, sc=lf ** -0.5)
        rec(f"llama.mlp.{name}", _time(lambda: ops.linear(ops.gate_up_silu(h, wgl), wdn), iters=3, warm=1),
            nbytes=3 * lf * d * 2.0 + tk * d * 4.0, flops=tk * 6.0 * lf * d)
    return out


def run_tugovik(sizes: list, seqs: int = 4, plen: int = 2048, rows: int = 64, ctx: int = 2048, device: str = "cuda") -> dict:
    from chronos import ops
    from chronos.models import kalesun, llama, tugovik
    from chronos.models.hybrid import HybridDecoder

    dev = torch.device(device if ":" in device else device + ":0")
    torch.cuda.set_device(dev)
    ops.load()
    ops.device_init()
    res = {}
    P = ctx + plen + 16
    for name in sizes:
        size, ksize = TUGOVIK_SIZES[name], KALESUN_SIZES[name]
        t0 = time.time()
        cfg = tugovik.config_from_dict(tugovik_config(size), name=f"tugovik-{name}", max_position=P)
        tm = HybridDecoder(cfg, tugovik.pack_weights(cfg, tugovik.random_tensors(cfg, 0), dev, torch.bfloat16), dev, P,
                           torch.bfloat16)
        entry = dict(tugovik=dict(params=cfg.param_count(), **_model_steps(tm, dev, seqs, plen, rows, ctx)))
        _say(f"size {name}: tugovik {entry['tugovik']}")
        del tm
        kcfg = kalesun.config_from_dict(kalesun_config(ksize), name=f"kalesun-{name}", max_position=P)
        km = HybridDecoder(kcfg, kalesun.pack_weights(kcfg, kalesun.random_tensors(kcfg, 0), dev, torch.bfloat16), dev, P,
                           torch.bfloat16)
        entry["kalesun"] = dict(params=kcfg.param_count(), **_model_steps(km, dev, seqs, plen, rows, ctx))
        _say(f"  kalesun {entry['kalesun']}")
        del km
        d = size["width"]
        lc = llama.LlamaConfig(name=f"llama-{name}", vocab_size=VOCAB, hidden_size=d, intermediate_size=int(3.5 * d),
                               num_layers=LAYERS, num_heads=d // 128, num_kv_heads=max(1, d // 512), max_position=P)
        lm = llama.LlamaModel(lc, llama.random_weights(lc, None, dev, 0), None, dev, P)
        entry["llama"] = dict(params=lc.param_count(), **_model_steps(lm, dev, seqs, plen, rows, ctx))
        _say(f"  llama {entry['llama']}")
        del lm
        torch.cuda.empty_cache()
        entry["kernels"] = _kernels_tugovik(size, ksize, dev, seqs * plen, ctx, rows)
        entry["seconds"] = round(time.time() - t0, 1)
        res[name] = entry
        torch.cuda.empty_cache()
    return dict(metric="design_compare", design="tugovik", beside="kalesun and llama (equal width and depth)",
                layers=LAYERS, workload=dict(prefill=f"{seqs} x {plen} tokens in one step",
                                             decode=f"{rows} rows at context {ctx}"),
                dtype="bf16", data="synthetic", sizes=res)


def _kernels_vogerax(size: dict, ksize: dict, dev, T: int, ctx: int, rows: int) -> dict:
    """Vogerax's kernels and their closest existing kernels at this size: seconds, and the fraction of the roofline
    reached.  ``ksize``: the Kalesun sizes of the same width (for the kernels it stands beside)."""
    from chronos import ops
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops

    out = {}
    bf = torch.bfloat16
    d, ng = size["width"], size["groups"]
    g = torch.Generator(device=dev).manual_seed(1)
    rnd = lambda *s, dt=bf, sc=1.0: (torch.randn(*s, device=dev, generator=g) * sc).to(dt)  # noqa: E731
    i32 = dict(dtype=torch.int32, device=dev)

    def rec(name, secs, nbytes=0.0, flops=0.0):
        roof = max(nbytes / HBM_BPS, flops / BF16_FLOPS)
        _say(f"  {name}: {secs * 1e6:.1f} us, roofline {roof * 1e6:.2f} us")
        out[name] = dict(us=round(secs * 1e6, 1), roofline_us=round(roof * 1e6, 2), of_roofline=round(roof / secs, 4))

    bs = 16
    seqs = max(1, T // ctx)
    per = ctx // bs + 1
    nb = max(seqs, rows) * per + 1
    bt = torch.arange(1, 1 + seqs * per, **i32).view(seqs, per)
    qs = torch.arange(0, (seqs + 1) * ctx, ctx, **i32)
    pos = torch.arange(ctx, **i32).repeat(seqs)
    tseq = torch.arange(seqs, **i32).repeat_interleave(ctx)
    btd = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    qsd = torch.arange(rows + 1, **i32)
    posd = torch.full((rows,), ctx, **i32)
    NS = max(seqs, rows) + 1
    p0, sl, sld = torch.zeros(seqs, **i32), torch.arange(seqs, **i32), torch.arange(rows, **i32)
    # ---- the stream's joins: norm of the addend, add, norm for the next sublayer, in one kernel
    y, y2, x32 = rnd(T, d), rnd(T, d), rnd(T, d, dt=torch.float32)
    w1, w2, w3, w4 = (rnd(d, dt=torch.float32) for _ in range(4))
    rec("sandwich_join", _time(lambda: hops.sandwich_join(y, x32, w1, w2, ng, 1e-5, bf)), T * d * (2 + 4 + 4 + 2))
    rec("sandwich_join.two_addends", _time(lambda: hops.sandwich_join(y, x32, w1, w2, ng, 1e-5, bf, y2)), T * d * (2 + 2 + 4 + 4 + 2))
    rec("sandwich_join.pair", _time(lambda: hops.sandwich_join(y, x32, w1, w2, ng, 1e-5, bf, y2, (w3, w4))), T * d * (2 + 2 + 4 + 4 + 2))
    yd, y2d, xd = rnd(rows, d), rnd(rows, d), rnd(rows, d, dt=torch.float32)
    rec("sandwich_join.pair.decode", _time(lambda: hops.sandwich_join(yd, xd, w1, w2, ng, 1e-5, bf, y2d, (w3, w4))), rows * d * 14.0)
    rec("kalesun.scale_add_rms_norm", _time(lambda: hops.scale_add_rms_norm(y, x32, w1, 1.0, 1e-6, bf)), T * d * (2 + 4 + 4 + 2))
    rec("tugovik.add_rms_norm.normed_addend", _time(lambda: hops.add_rms_norm(y, x32, w1, 1e-6, bf, w_y=w2)), T * d * (2 + 4 + 4 + 2))
    xb, wb = rnd(T, d), rnd(d)
    rec("llama.add_rmsnorm", _time(lambda: ops.add_rmsnorm(y, xb, wb, 1e-5)), T * d * (2 + 2 + 2 + 2))
    # ---- pooled-window attention beside Kalesun's window of the same span (with sink and gate) and Llama's
    H, G, D, win, pool = size["a"]
    ep = (bs + pool - 1) // pool
    kc, vc = rnd(nb, bs, G, D, sc=0.3), rnd(nb, bs, G, D, sc=0.3)
    kp, vp = rnd(nb, ep, G, D, sc=0.3), rnd(nb, ep, G, D, sc=0.3)
    C = (H + G) * D
    qk = rnd(seqs * ctx, C, sc=0.3)
    tab = rope_cos_sin(5e5, D // 2, ctx + 2, dev, ("linear", 4.0))
    vis = sum(min(i + 1, win) + max(0, i - win + 1) // pool for i in range(ctx))
    rec("pooled_attention.prefill", _time(lambda: hops.window_attention(qk, kc, vc, bt, qs, pos, None, None, D ** -0.5, win, 0, H, bf, ctx, 0, pool, kp, vp), iters=3, warm=1),
        flops=4.0 * seqs * vis * H * D)
    rec("window_prep.values_are_keys.prefill", _time(lambda: hops.window_prep(qk, H, G, D, D, None, None, pos, tseq, bt, None, None, 1e-5, tab, D // 2, kc, vc, False, H * D)),
        nbytes=seqs * ctx * (2 * (H + G) * D + 2 * G * D) * 2.0)
    rec("pool_blocks.prefill", _time(lambda: hops.pool_blocks(kc, vc, kp, vp, bt, qs, p0, pool, ctx)),
        nbytes=seqs * ctx * 2 * G * D * 2.0 * (1 + 1.0 / pool))
    qkd = rnd(rows, C, sc=0.3)
    rec("pooled_attention.decode", _time(lambda: hops.window_attention(qkd, kc, vc, btd, qsd, posd, None, None, D ** -0.5, win, 0, H, bf, 1, 0, pool, kp, vp)),
        nbytes=rows * (min(ctx + 1, win) + max(0, ctx - win + 1) // pool) * G * 2 * D * 2.0)
    rec("pool_blocks.decode", _time(lambda: hops.pool_blocks(kc, vc, kp, vp, btd, qsd, posd, pool, 1)), nbytes=1.0)
    kH, kG, kD, kDv, kwin, keep = ksize["a"]
    kkc, kvc = rnd(nb, bs, kG, kD, sc=0.3), rnd(nb, bs, kG, kDv, sc=0.3)
    kqkv = rnd(seqs * ctx, (kH + kG) * kD + kG * kDv, sc=0.3)
    kgate, ksink = rnd(seqs * ctx, kH, dt=torch.float32), rnd(kH, dt=torch.float32)
    kvis = sum(min(i + 1, kwin) + max(0, min(keep, i + 1 - kwin)) for i in range(ctx))
    rec("kalesun.window_attention.prefill", _time(lambda: hops.window_attention(kqkv, kkc, kvc, bt, qs, pos, ksink, kgate, kD ** -0.5, kwin, keep, kH, bf, ctx), iters=3, warm=1),
        flops=2.0 * seqs * kvis * kH * (kD + kDv))
    kqkvd, kgated = rnd(rows, (kH + kG) * kD + kG * kDv, sc=0.3), rnd(rows, kH, dt=torch.float32)
    rec("kalesun.window_attention.decode", _time(lambda: hops.window_attention(kqkvd, kkc, kvc, btd, qsd, posd, ksink, kgated, kD ** -0.5, kwin, keep, kH, bf, 1)),
        nbytes=rows * (min(ctx + 1, kwin) + keep) * kG * (kD + kDv) * 2.0)
    # ---- causal sink attention with rotated values and a gate per column, beside Llama's causal attention
    lH, lG, lD, lDv = size["l"]
    lkc, lvc = rnd(nb, bs, lG, lD, sc=0.3), rnd(nb, bs, lG, lDv, sc=0.3)
    Cl = (lH + lG) * lD + lG * lDv + lH * lDv
    lq = rnd(seqs * ctx, Cl, sc=0.3)
    lsink = rnd(lH, dt=torch.float32)
    vtab = rope_cos_sin(1e5, lDv, ctx + 2, dev)
    ltab = rope_cos_sin(1e5, lD // 2, ctx + 2, dev, ("ramp", 8.0, 4096.0, 16.0, 2.0))
    qn, kn = rnd(lD, dt=torch.float32), rnd(lD, dt=torch.float32)
    full_pairs = seqs * ctx * (ctx + 1) / 2
    lg_off = (lH + lG) * lD + lG * lDv   # outputs turned back and gated per column in the attention's epilogue
    rec("sink_attention.prefill", _time(lambda: hops.window_attention(lq, lkc, lvc, bt, qs, pos, lsink, None, lD ** -0.5, 0, 0, lH, bf, ctx, 0, 0, None, None, vtab, lg_off), iters=3, warm=1),
        flops=2.0 * full_pairs * lH * (lD + lDv))
    rec("window_prep.rotated_values.prefill", _time(lambda: hops.window_prep(lq, lH, lG, lD, lDv, None, None, pos, tseq, bt, qn, kn, 1e-5, ltab, lD // 2, lkc, lvc, False, -1, vtab)),
        nbytes=seqs * ctx * (2 * (lH + lG) * lD + 2 * lG * lDv) * 2.0)
    lo = rnd(seqs * ctx, lH * lDv)
    rec("unrotate_gate.prefill", _time(lambda: hops.unrotate_gate(lo, pos, vtab, lq, (lH + lG) * lD + lG * lDv, lH, lDv, bf)),
        nbytes=seqs * ctx * lH * lDv * 6.0)
    lqd = rnd(rows, Cl, sc=0.3)
    rec("sink_attention.decode", _time(lambda: hops.window_attention(lqd, lkc, lvc, btd, qsd, posd, lsink, None, lD ** -0.5, 0, 0, lH, bf, 1, 0, 0, None, None, vtab, lg_off)),
        nbytes=rows * (ctx + 1) * lG * (lD + lDv) * 2.0)
    hq = d // 128
    hkv = max(1, hq // 4)
    akc, avc = rnd(nb, hkv, bs, 128, sc=0.3), rnd(nb, hkv, 128, bs, sc=0.3)
    q = rnd(seqs * ctx, hq, 128, sc=0.3)
    ctxl = torch.full((seqs,), ctx, **i32)
    tiles = torch.tensor(ops.attention_tiles([ctx] * seqs, hq, hkv, 8), **i32).view(-1, 2)
    rec("llama.attention.prefill", _time(lambda: ops.paged_attention(q, akc, avc, bt, qs, ctxl, tiles, tiles.shape[0], 8, 1), iters=3, warm=1),
        flops=4.0 * full_pairs * hq * 128)
    qd = rnd(rows, hq, 128, sc=0.3)
    ctxd = torch.full((rows,), ctx + 1, **i32)
    ns = ops.pick_nsplit(rows * hkv, ctx + 1)
    rec("llama.attention.decode", _time(lambda: ops.paged_attention(qd, akc, avc, btd, qsd, ctxd, None, rows, 1, ns)),
        nbytes=rows * (ctx + 1) * hkv * 128 * 2 * 2.0)
    # ---- retention: the linear-state scan with fixed decays beside Kalesun's gated linear attention on the same kernel
    rh, rd, rv = size["r"]
    Cr = 2 * rh * rd + 2 * rh * rv
    S = torch.zeros(NS, rh, rd, rv, device=dev)
    dec = torch.tensor([math.exp(-1.0 / (16.0 * 128.0 ** (h / max(1, rh - 1)))) for h in range(rh)], device=dev)
    rtab = rope_cos_sin(1e4, rd, ctx + 2, dev)
    ones = torch.ones(rh * rv, device=dev)
    proj, projd = rnd(seqs * ctx, Cr, sc=0.5), rnd(rows, Cr, sc=0.5)
    rec("rotate_qk.prefill", _time(lambda: hops.rotate_qk(proj, 0, rh * rd, rh, rh, rd, rd, rtab, pos, 1.0, 1.0)), nbytes=seqs * ctx * 2 * rh * rd * 4.0)
    rec("retention_scan.prefill", _time(lambda: hops.linear_scan(proj, 0, rh * rd, 2 * rh * rd, None, None, 1.0, dec, None, qs, p0, sl, S, rh, rh, rd, rv), iters=3, warm=1),
        nbytes=seqs * ctx * Cr * 2.0, flops=seqs * ctx * rh * rd * rv * 4.0)
    rec("retention_scan.decode", _time(lambda: hops.linear_scan(projd, 0, rh * rd, 2 * rh * rd, None, None, 1.0, dec, None, qsd, posd, sld, S, rh, rh, rd, rv)),
        nbytes=rows * rh * rd * rv * 4 * 2.0)
    o32 = rnd(seqs * ctx, rh, rv, dt=torch.float32)
    rec("head_norm_gate.prefill", _time(lambda: hops.head_norm_gate(o32, proj, 2 * rh * rd + rh * rv, ones, 1e-5, True, bf)), nbytes=seqs * ctx * rh * rv * 8.0)
    gh, gd, gv = ksize["g"]
    gS = torch.zeros(NS, gh, gd, gv, device=dev)
    gproj, gprojd = rnd(seqs * ctx, 2 * gh * gd + gh * gv, sc=0.5), rnd(rows, 2 * gh * gd + gh * gv, sc=0.5)
    gdec, gdecd = torch.rand(seqs * ctx, gh, gd, device=dev), torch.rand(rows, gh, gd, device=dev)
    rec("kalesun.linear_scan.gla.prefill", _time(lambda: hops.linear_scan(gproj, 0, gh * gd, 2 * gh * gd, None, None, gd ** -0.5, gdec, None, qs, p0, sl, gS, gh, gh, gd, gv), iters=3, warm=1),
        nbytes=seqs * ctx * (2 * gh * gd + gh * gv) * 2.0, flops=seqs * ctx * gh * gd * gv * 4.0)
    rec("kalesun.linear_scan.gla.decode", _time(lambda: hops.linear_scan(gprojd, 0, gh * gd, 2 * gh * gd, None, None, gd ** -0.5, gdecd, None, qsd, posd, sld, gS, gh, gh, gd, gv)),
        nbytes=rows * gh * gd * gv * 4 * 2.0)
    # ---- feed-forwards: squared-ReLU experts behind a softmax router beside Kalesun's gated experts and Llama's MLP
    ne, top, eff, sff = size["moe"]
    wr, corr = rnd(ne, d, sc=0.05), torch.zeros(ne, device=dev)
    wu, wd = rnd(ne, eff, d, sc=d ** -0.5), rnd(ne, d, eff, sc=eff ** -0.5)
    kne, ktop, keff = ksize["moe"]
    kwr, kbr = rnd(kne, d, sc=0.05), rnd(kne, dt=torch.float32, sc=0.01)
    kwgu = rnd(kne, 2 * keff, d, sc=d ** -0.5)[:, hops.moe_glu_row_order(keff).to(dev)].contiguous()
    kwd = rnd(kne, d, keff, sc=keff ** -0.5)
    for name, tk in (("prefill", T), ("decode", rows)):
        h = rnd(tk, d)
        idx, wt = hops.moe_route(h, wr, corr, top)
        rec(f"moe_route.{name}", _time(lambda: hops.moe_route(h, wr, corr, top)), nbytes=tk * d * 2.0 + ne * d * 2.0)
        rec(f"moe_ffn.relu2.{name}", _time(lambda: hops.moe_ffn(h, idx, wt, wu, wd, hops.ACT_RELU2, bf), iters=3, warm=1),
            nbytes=min(ne, tk * top) * 2 * eff * d * 2.0 + tk * d * 4.0, flops=tk * top * 4.0 * eff * d)
        kidx, kwt = hops.moe_route_topk(h, kwr, kbr, ktop)
        rec(f"kalesun.moe_route_topk.{name}", _time(lambda: hops.moe_route_topk(h, kwr, kbr, ktop)), nbytes=tk * d * 2.0 + kne * d * 2.0)
        rec(f"kalesun.moe_glu_ffn.{name}", _time(lambda: hops.moe_glu_ffn(h, kidx, kwt, kwgu, kwd, 7.0, 1.702, 1.0, bf, True), iters=3, warm=1),
            nbytes=min(kne, tk * ktop) * 3 * keff * d * 2.0 + tk * d * 4.0, flops=tk * ktop * 6.0 * keff * d)
        lf = int(3.5 * d)
        wgl, wdn = rnd(2 * lf, d, sc=d ** -0.5), rnd(d, lf, sc=lf ** -0.5)
        rec(f"llama.mlp.{name}", _time(lambda: ops.linear(ops.gate_up_silu(h, wgl), wdn), iters=3, warm=1),
            nbytes=3 * lf * d * 2.0 + tk * d * 4.0, flops=tk * 6.0 * lf * d)
    return out


def run_vogerax(sizes: list, seqs: int = 4, plen: int = 2048, rows: int = 64, ctx: int = 2048, device: str = "cuda") -> dict:
    from chronos import ops
    from chronos.models import kalesun, llama, vogerax
    from chronos.models.hybrid import HybridDecoder

    dev = torch.device(device if ":" in device else device + ":0")
    torch.cuda.set_device(dev)
    ops.load()
    ops.device_init()
    res = {}
    P = ctx + plen + 16
    for name in sizes:
        size, ksize = VOGERAX_SIZES[name], KALESUN_SIZES[name]
        t0 = time.time()
        cfg = vogerax.config_from_dict(vogerax_config(size), name=f"vogerax-{name}", max_position=P)
        vm = HybridDecoder(cfg, vogerax.pack_weights(cfg, vogerax.random_tensors(cfg, 0), dev, torch.bfloat16), dev, P,
                           torch.bfloat16)
        entry = dict(vogerax=dict(params=cfg.param_count(), **_model_steps(vm, dev, seqs, plen, rows, ctx)))
        _say(f"size {name}: vogerax {entry['vogerax']}")
        del vm
        kcfg = kalesun.config_from_dict(kalesun_config(ksize), name=f"kalesun-{name}", max_position=P)
        km = HybridDecoder(kcfg, kalesun.pack_weights(kcfg, kalesun.random_tensors(kcfg, 0), dev, torch.bfloat16), dev, P,
                           torch.bfloat16)
        entry["kalesun"] = dict(params=kcfg.param_count(), **_model_steps(km, dev, seqs, plen, rows, ctx))
        _say(f"  kalesun {entry['kalesun']}")
        del km
        d = size["width"]
        lc = llama.LlamaConfig(name=f"llama-{name}", vocab_size=VOCAB, hidden_size=d, intermediate_size=int(3.5 * d),
                               num_layers=LAYERS, num_heads=d // 128, num_kv_heads=max(1, d // 512), max_position=P)
        lm = llama.LlamaModel(lc, llama.random_weights(lc, None, dev, 0), None, dev, P)
        entry["llama"] = dict(params=lc.param_count(), **_model_steps(lm, dev, seqs, plen, rows, ctx))
        _say(f"  llama {entry['llama']}")
        del lm
        torch.cuda.empty_cache()
        entry["kernels"] = _kernels_vogerax(size, ksize, dev, seqs * plen, ctx, rows)
        entry["seconds"] = round(time.time() - t0, 1)
        res[name] = entry
        torch.cuda.empty_cache()
    return dict(metric="design_compare", design="vogerax", beside="kalesun and llama (equal width and depth)",
                layers=LAYERS, workload=dict(prefill=f"{seqs} x {plen} tokens in one step",
                                             decode=f"{rows} rows at context {ctx}"),
                dtype="bf16", data="synthetic", sizes=res)


def _kernels_lalasun(size: dict, ksize: dict, zsize: dict, dev, T: int, ctx: int, rows: int) -> dict:
    """Lalasun's kernels and their closest existing kernels at this size: seconds, and the fraction of the roofline
    reached.  ``ksize``, ``zsize``: the Kalesun and Zokunex sizes of the same width (for the kernels it stands beside)."""
    from chronos import ops
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops

    out = {}
    bf = torch.bfloat16
    d = size["width"]
    g = torch.Generator(device=dev).manual_seed(1)
    rnd = lambda *s, dt=bf, sc=1.0: (torch.randn(*s, device=dev, generator=g) * sc).to(dt)  # noqa: E731
    f32 = lambda *s, sc=1.0: rnd(*s, dt=torch.float32, sc=sc)  # noqa: E731
    i32 = dict(dtype=torch.int32, device=dev)

    def rec(name, secs, nbytes=0.0, flops=0.0):
        roof = max(nbytes / HBM_BPS, flops / BF16_FLOPS)
        _say(f"  {name}: {secs * 1e6:.1f} us, roofline {roof * 1e6:.2f} us")
        out[name] = dict(us=round(secs * 1e6, 1), roofline_us=round(roof * 1e6, 2), of_roofline=round(roof / secs, 4))

    bs = 16
    seqs = max(1, T // ctx)
    n = seqs * ctx
    per = ctx // bs + 1
    nb = max(seqs, rows) * per + 1
    bt = torch.arange(1, 1 + seqs * per, **i32).view(seqs, per)
    qs = torch.arange(0, (seqs + 1) * ctx, ctx, **i32)
    pos = torch.arange(ctx, **i32).repeat(seqs)
    tseq = torch.arange(seqs, **i32).repeat_interleave(ctx)
    btd = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    qsd = torch.arange(rows + 1, **i32)
    posd = torch.full((rows,), ctx, **i32)
    NS = max(seqs, rows) + 1
    p0, sl, sld = torch.zeros(seqs, **i32), torch.arange(seqs, **i32), torch.arange(rows, **i32)
    full_pairs = n * (ctx + 1) / 2
    # ---- the stream's joins (gate, multiply, add, next norm; at a layer's end also the depth average)
    y, x32, w1 = rnd(T, d), f32(T, d), f32(d)
    wba, gb = torch.cat([w1, f32(d, sc=0.1), torch.tensor([0.7], device=dev)]), f32(d, sc=0.1)
    F = size["ff"]
    src = rnd(T, F + d)   # the gate's columns lie behind the feed-forward's up-projection
    for run in (0, 2):
        hist, dwa = f32(LAYERS, T, d), f32(run + 2, sc=0.3)
        rec(f"gated_join.depth_average_{run + 2}", _time(lambda: hops.gated_join(y, x32, src, F, gb, 0.4, wba, bf, hist, run, dwa)),
            T * d * (2 + 2 + 4 + 4 + 2 + 4 * (run + 1) + 4))
    del hist
    rec("gated_join", _time(lambda: hops.gated_join(y, x32, src, F, gb, 0.4, wba, bf)), T * d * (2 + 2 + 4 + 4 + 2))
    yd, xd, srcd = rnd(rows, d), f32(rows, d), rnd(rows, F + d)
    rec("gated_join.decode", _time(lambda: hops.gated_join(yd, xd, srcd, F, gb, 0.4, wba, bf)), rows * d * 14.0)
    rec("kalesun.scale_add_rms_norm.decode", _time(lambda: hops.scale_add_rms_norm(yd, xd, w1, 1.0, 1e-6, bf)), rows * d * 12.0)
    rec("dyn_tanh", _time(lambda: hops.dyn_tanh(x32, wba, bf)), T * d * (4 + 2))
    rec("rms_norm", _time(lambda: hops.rms_norm(x32, w1, 1e-6, bf)), T * d * (4 + 2))
    rec("kalesun.scale_add_rms_norm", _time(lambda: hops.scale_add_rms_norm(y, x32, w1, 1.0, 1e-6, bf)), T * d * (2 + 4 + 4 + 2))
    rec("zokunex.add_layer_norm", _time(lambda: hops.add_layer_norm(y, x32, w1, 1e-6, bf)), T * d * (2 + 4 + 4 + 2))
    xb, wb = rnd(T, d), rnd(d)
    rec("llama.add_rmsnorm", _time(lambda: ops.add_rmsnorm(y, xb, wb, 1e-5)), T * d * (2 + 2 + 2 + 2))
    # ---- chunked attention with one added to the denominator beside Kalesun's window of the same span and Llama's
    H, G, D, Dv, chunk = size["a"]
    kc, vc = rnd(nb, bs, G, D, sc=0.3), rnd(nb, bs, G, Dv, sc=0.3)
    C = (H + G) * D + G * Dv + d    # (the residual gate's rows ride along)
    qkv, qkvd = rnd(n, C, sc=0.3), rnd(rows, C, sc=0.3)
    tab = rope_cos_sin(5e5, D, ctx + 2, dev)
    zero = torch.zeros(H, device=dev)
    vis = sum(i % chunk + 1 for i in range(ctx))
    rec("chunk_attention.prefill", _time(lambda: hops.window_attention(qkv, kc, vc, bt, qs, pos, zero, None, D ** -0.5, 0, 0, H, bf, ctx, chunk), iters=3, warm=1),
        flops=2.0 * seqs * vis * H * (D + Dv))
    posc = torch.full((rows,), (ctx // chunk) * chunk - 1, **i32)   # the last position of a chunk: all of it is visible
    rec("chunk_attention.decode", _time(lambda: hops.window_attention(qkvd, kc, vc, btd, qsd, posc, zero, None, D ** -0.5, 0, 0, H, bf, 1, chunk)),
        nbytes=rows * chunk * G * (D + Dv) * 2.0)
    rec("window_prep.rotated.prefill", _time(lambda: hops.window_prep(qkv, H, G, D, Dv, None, None, pos, tseq, bt, None, None, 1e-5, tab, D, kc, vc, False)),
        nbytes=n * (2 * (H + G) * D + 2 * G * Dv) * 2.0)
    kH, kG, kD, kDv, kwin, keep = ksize["a"]
    kkc, kvc = rnd(nb, bs, kG, kD, sc=0.3), rnd(nb, bs, kG, kDv, sc=0.3)
    kqkv, kqkvd = rnd(n, (kH + kG) * kD + kG * kDv, sc=0.3), rnd(rows, (kH + kG) * kD + kG * kDv, sc=0.3)
    kgate, kgated, ksink = f32(n, kH), f32(rows, kH), f32(kH)
    qn, kn, ktab = f32(kD), f32(kD), rope_cos_sin(5e5, kD // 2, ctx + 2, dev)
    kvis = sum(min(i + 1, kwin) + max(0, min(keep, i + 1 - kwin)) for i in range(ctx))
    rec("kalesun.window_attention.prefill", _time(lambda: hops.window_attention(kqkv, kkc, kvc, bt, qs, pos, ksink, kgate, kD ** -0.5, kwin, keep, kH, bf, ctx), iters=3, warm=1),
        flops=2.0 * seqs * kvis * kH * (kD + kDv))
    rec("kalesun.window_attention.decode", _time(lambda: hops.window_attention(kqkvd, kkc, kvc, btd, qsd, posd, ksink, kgated, kD ** -0.5, kwin, keep, kH, bf, 1)),
        nbytes=rows * (min(ctx + 1, kwin) + keep) * kG * (kD + kDv) * 2.0)
    rec("kalesun.window_prep.prefill", _time(lambda: hops.window_prep(kqkv, kH, kG, kD, kDv, None, None, pos, tseq, bt, qn, kn, 1e-5, ktab, kD // 2, kkc, kvc, False)),
        nbytes=n * (2 * (kH + kG) * kD + 2 * kG * kDv) * 2.0)
    hq = d // 128
    hkv = max(1, hq // 4)
    akc, avc = rnd(nb, hkv, bs, 128, sc=0.3), rnd(nb, hkv, 128, bs, sc=0.3)
    q, qd = rnd(n, hq, 128, sc=0.3), rnd(rows, hq, 128, sc=0.3)
    ctxl, ctxd = torch.full((seqs,), ctx, **i32), torch.full((rows,), ctx + 1, **i32)
    tiles = torch.tensor(ops.attention_tiles([ctx] * seqs, hq, hkv, 8), **i32).view(-1, 2)
    rec("llama.attention.prefill", _time(lambda: ops.paged_attention(q, akc, avc, bt, qs, ctxl, tiles, tiles.shape[0], 8, 1), iters=3, warm=1),
        flops=4.0 * full_pairs * hq * 128)
    ns = ops.pick_nsplit(rows * hkv, ctx + 1)
    rec("llama.attention.decode", _time(lambda: ops.paged_attention(qd, akc, avc, btd, qsd, ctxd, None, rows, 1, ns)),
        nbytes=rows * (ctx + 1) * hkv * 128 * 2 * 2.0)
    del kc, vc, kkc, kvc, akc, avc, qkv, kqkv, q
    # ---- latent attention through a window (two-term weights) beside Zokunex's causal latent attention
    H, D, R, Dv, rank, win = size["l"]
    DK, nq = rank + R, H * (D + R)
    lat = rnd(nb, bs, DK, sc=0.3)
    Cl = nq + DK + H * Dv + d
    proj, projd = rnd(n, Cl, sc=0.3), rnd(rows, Cl, sc=0.3)
    qa, qad = rnd(n, H, DK, sc=0.3), rnd(rows, H, DK, sc=0.3)
    ltab, wn = rope_cos_sin(1e5, R, ctx + 2, dev), f32(rank)
    wvis = sum(min(i + 1, win) for i in range(ctx))
    rec("latent_window.prefill", _time(lambda: hops.latent_attention(qa, lat, bt, qs, pos, None, 0.1, rank, bf, ctx, win, True), iters=3, warm=1),
        flops=2.0 * seqs * wvis * H * (DK + rank))
    rec("latent_window.prefill.one_term", _time(lambda: hops.latent_attention(qa, lat, bt, qs, pos, None, 0.1, rank, bf, ctx, win, False), iters=3, warm=1),
        flops=2.0 * seqs * wvis * H * (DK + rank))
    rec("latent_window.decode", _time(lambda: hops.latent_attention(qad, lat, btd, qsd, posd, None, 0.1, rank, bf, 1, win, True)),
        nbytes=rows * min(ctx + 1, win) * DK * 2.0)
    rec("latent_prep.prefill", _time(lambda: hops.latent_prep(proj[:, :nq].view(n, H, D + R), proj[:, nq:nq + DK], pos, tseq, bt, wn, 1e-5, ltab, R, rank, lat, qa, True)),
        nbytes=n * (2 * DK + 2 * H * R) * 2.0)
    zH, zD, zR, zDv, zrank = zsize["a"]
    zlat = rnd(nb, bs, zrank + zR, sc=0.3)
    zqa, zqad = rnd(n, zH, zrank + zR, sc=0.3), rnd(rows, zH, zrank + zR, sc=0.3)
    zg, zgd = f32(n, zH), f32(rows, zH)
    rec("zokunex.latent_attention.prefill", _time(lambda: hops.latent_attention(zqa, zlat, bt, qs, pos, zg, 0.1, zrank, bf, ctx), iters=3, warm=1),
        flops=2.0 * full_pairs * zH * (2 * zrank + zR))
    rec("zokunex.latent_attention.decode", _time(lambda: hops.latent_attention(zqad, zlat, btd, qsd, posd, zgd, 0.1, zrank, bf, 1)),
        nbytes=rows * (ctx + 1) * (zrank + zR) * 2.0)
    # per-head products beside the library's batched product (which leaves the result in another layout)
    wuk, wuv = rnd(H, rank, D, sc=D ** -0.5), rnd(H, Dv, rank, sc=rank ** -0.5)
    ukt, uvt = wuk.transpose(1, 2).contiguous(), wuv.transpose(1, 2).contiguous()
    for name, m, pr, qx in (("prefill", n, proj, qa), ("decode", rows, projd, qad)):
        qv = pr[:, :nq].view(m, H, D + R)[:, :, :D]
        oa = rnd(m, H, rank)
        nb1, fl = (m * H * (D + rank) + H * D * rank) * 2.0, 2.0 * m * H * D * rank
        rec(f"head_matmul.to_latent.{name}", _time(lambda: hops.head_matmul(qv, wuk, qx[:, :, :rank])), nbytes=nb1, flops=fl)
        rec(f"library.bmm.to_latent.{name}", _time(lambda: torch.bmm(qv.transpose(0, 1), ukt)), nbytes=nb1, flops=fl)
        nb2 = (m * H * (2 * Dv + rank) + H * Dv * rank) * 2.0
        rec(f"head_matmul.from_latent_gated.{name}", _time(lambda: hops.head_matmul(oa, wuv, None, pr, nq + DK)), nbytes=nb2, flops=2.0 * m * H * Dv * rank)
        rec(f"library.bmm.from_latent.{name}", _time(lambda: torch.bmm(oa.transpose(0, 1), uvt)), nbytes=nb2 - m * H * Dv * 2.0, flops=2.0 * m * H * Dv * rank)
    del lat, zlat, proj, qa, zqa, oa
    # ---- gated linear attention: Kalesun's kernels
    gh, gd, gv = size["g"]
    S = torch.zeros(NS, gh, gd, gv, device=dev)
    gproj, gprojd = rnd(n, 2 * gh * gd + 2 * gh * gv + d, sc=0.5), rnd(rows, 2 * gh * gd + 2 * gh * gv + d, sc=0.5)
    gdec, gdecd = torch.rand(n, gh, gd, device=dev), torch.rand(rows, gh, gd, device=dev)
    rec("linear_scan.gla.prefill", _time(lambda: hops.linear_scan(gproj, 0, gh * gd, 2 * gh * gd, None, None, gd ** -0.5, gdec, None, qs, p0, sl, S, gh, gh, gd, gv), iters=3, warm=1),
        nbytes=n * (2 * gh * gd + gh * gv) * 2.0, flops=n * gh * gd * gv * 4.0)
    rec("linear_scan.gla.decode", _time(lambda: hops.linear_scan(gprojd, 0, gh * gd, 2 * gh * gd, None, None, gd ** -0.5, gdecd, None, qsd, posd, sld, S, gh, gh, gd, gv)),
        nbytes=rows * gh * gd * gv * 4 * 2.0)
    kgh, kgd, kgv = ksize["g"]
    kS = torch.zeros(NS, kgh, kgd, kgv, device=dev)
    kproj = rnd(n, 2 * kgh * kgd + 2 * kgh * kgv, sc=0.5)
    kdec = torch.rand(n, kgh, kgd, device=dev)
    rec("kalesun.linear_scan.gla.prefill", _time(lambda: hops.linear_scan(kproj, 0, kgh * kgd, 2 * kgh * kgd, None, None, kgd ** -0.5, kdec, None, qs, p0, sl, kS, kgh, kgh, kgd, kgv), iters=3, warm=1),
        nbytes=n * (2 * kgh * kgd + kgh * kgv) * 2.0, flops=n * kgh * kgd * kgv * 4.0)
    # ---- feed-forwards: PolyNorm beside Zokunex's activation in place and Kalesun's gated unit, then whole units
    abce = torch.tensor([0.6, -0.3, 0.2, 0.1], device=dev)
    kff, zff, lf = ksize["ff"], zsize["ff"], int(3.5 * d)
    wup, wdn = rnd(F + d, d, sc=d ** -0.5), rnd(d, F, sc=F ** -0.5)
    kgu, kdn = rnd(2 * kff, d, sc=d ** -0.5), rnd(d, kff, sc=kff ** -0.5)
    zup, zdn = rnd(zff, d, sc=d ** -0.5), rnd(d, zff, sc=zff ** -0.5)
    lgu, ldn = rnd(2 * lf, d, sc=d ** -0.5), rnd(d, lf, sc=lf ** -0.5)
    for name, tk in (("prefill", T), ("decode", rows)):
        h, z, kz = rnd(tk, d), rnd(tk, F + d), rnd(tk, 2 * kff)
        zz = rnd(tk, zff)
        rec(f"poly_norm.{name}", _time(lambda: hops.poly_norm(z, F, abce, 1e-6, bf)), nbytes=tk * F * 4.0)
        rec(f"zokunex.act.{name}", _time(lambda: hops.act_inplace(zz, hops.ACT_RELU2)), nbytes=tk * zff * 4.0)
        rec(f"kalesun.glu.{name}", _time(lambda: hops.glu(kz, 7.0, 1.702, 1.0, bf)), nbytes=tk * kff * 6.0)
        rec(f"poly_ff.{name}", _time(lambda: hops.matmul(hops.poly_norm(hops.matmul(h, wup), F, abce, 1e-6, bf), wdn), iters=3, warm=1),
            nbytes=(2 * F + d) * d * 2.0 + tk * d * 4.0, flops=tk * 2.0 * (2 * F + d) * d)
        rec(f"zokunex.dense_ff.{name}", _time(lambda: hops.matmul(hops.act_inplace(hops.matmul(h, zup), hops.ACT_RELU2), zdn), iters=3, warm=1),
            nbytes=2 * zff * d * 2.0 + tk * d * 4.0, flops=tk * 4.0 * zff * d)
        rec(f"kalesun.glu_ff.{name}", _time(lambda: hops.matmul(hops.glu(hops.matmul(h, kgu), 7.0, 1.702, 1.0, bf), kdn), iters=3, warm=1),
            nbytes=3 * kff * d * 2.0 + tk * d * 4.0, flops=tk * 6.0 * kff * d)
        rec(f"llama.mlp.{name}", _time(lambda: ops.linear(ops.gate_up_silu(h, lgu), ldn), iters=3, warm=1),
            nbytes=3 * lf * d * 2.0 + tk * d * 4.0, flops=tk * 6.0 * lf * d)
    return out


def run_lalasun(sizes: list, seqs: int = 4, plen: int = 2048, rows: int = 64, ctx: int = 2048, device: str = "cuda") -> dict:
    from chronos import ops
    from chronos.models import kalesun, lalasun, llama, zokunex
    from chronos.models.hybrid import HybridDecoder

    dev = torch.device(device if ":" in device else device + ":0")
    torch.cuda.set_device(dev)
    ops.load()
    ops.device_init()
    res = {}
    P = ctx + plen + 16
    for name in sizes:
        size, ksize, zsize = LALASUN_SIZES[name], KALESUN_SIZES[name], SIZES[name]
        t0 = time.time()
        entry = {}
        for mod, key, conf in ((lalasun, "lalasun", lalasun_config(size)), (kalesun, "kalesun", kalesun_config(ksize)),
                               (zokunex, "zokunex", zokunex_config(zsize))):
            cfg = mod.config_from_dict(conf, name=f"{key}-{name}", max_position=P)
            m = HybridDecoder(cfg, mod.pack_weights(cfg, mod.random_tensors(cfg, 0), dev, torch.bfloat16), dev, P, torch.bfloat16)
            entry[key] = dict(params=cfg.param_count(), **_model_steps(m, dev, seqs, plen, rows, ctx))
            _say(f"size {name}: {key} {entry[key]}")
            del m
        d = size["width"]
        lc = llama.LlamaConfig(name=f"llama-{name}", vocab_size=VOCAB, hidden_size=d, intermediate_size=int(3.5 * d),
                               num_layers=LAYERS, num_heads=d // 128, num_kv_heads=max(1, d // 512), max_position=P)
        lm = llama.LlamaModel(lc, llama.random_weights(lc, None, dev, 0), None, dev, P)
        entry["llama"] = dict(params=lc.param_count(), **_model_steps(lm, dev, seqs, plen, rows, ctx))
        _say(f"  llama {entry['llama']}")
        del lm
        torch.cuda.empty_cache()
        entry["kernels"] = _kernels_lalasun(size, ksize, zsize, dev, seqs * plen, ctx, rows)
        entry["seconds"] = round(time.time() - t0, 1)
        res[name] = entry
        torch.cuda.empty_cache()
    return dict(metric="design_compare", design="lalasun", beside="kalesun, zokunex and llama (equal width and depth)",
                layers=LAYERS, workload=dict(prefill=f"{seqs} x {plen} tokens in one step",
                                             decode=f"{rows} rows at context {ctx}"),
                dtype="bf16", data="synthetic", sizes=res)


def _kernels_nubodra(size: dict, ksize: dict, zsize: dict, dev, T: int, ctx: int, rows: int) -> dict:
    """Nubodra's kernels and their closest existing kernels at this size: seconds, and the fraction of the roofline
    reached.  ``ksize``, ``zsize``: the Kalesun and Zokunex sizes of the same width (for the kernels it stands beside)."""
    from chronos import ops
    from chronos.models.hybrid import query_temperature, rope_cos_sin
    from chronos.ops import hybrid as hops

    out = {}
    bf = torch.bfloat16
    d = size["width"]
    g = torch.Generator(device=dev).manual_seed(1)
    rnd = lambda *s, dt=bf, sc=1.0: (torch.randn(*s, device=dev, generator=g) * sc).to(dt)  # noqa: E731
    f32 = lambda *s, sc=1.0: rnd(*s, dt=torch.float32, sc=sc)  # noqa: E731
    i32 = dict(dtype=torch.int32, device=dev)

    def rec(name, secs, nbytes=0.0, flops=0.0):
        roof = max(nbytes / HBM_BPS, flops / BF16_FLOPS)
        _say(f"  {name}: {secs * 1e6:.1f} us, roofline {roof * 1e6:.2f} us")
        out[name] = dict(us=round(secs * 1e6, 1), roofline_us=round(roof * 1e6, 2), of_roofline=round(roof / secs, 4))

    bs = 16
    seqs = max(1, T // ctx)
    n = seqs * ctx
    per = ctx // bs + 1
    nb = max(seqs, rows) * per + 1
    bt = torch.arange(1, 1 + seqs * per, **i32).view(seqs, per)
    qs = torch.arange(0, (seqs + 1) * ctx, ctx, **i32)
    pos = torch.arange(ctx, **i32).repeat(seqs)
    tseq = torch.arange(seqs, **i32).repeat_interleave(ctx)
    btd = torch.arange(1, 1 + rows * per, **i32).view(rows, per)
    qsd = torch.arange(rows + 1, **i32)
    tseqd = torch.arange(rows, **i32)
    posd = torch.full((rows,), ctx, **i32)
    NS = max(seqs, rows) + 1
    p0, sl, sld = torch.zeros(seqs, **i32), torch.arange(seqs, **i32), torch.arange(rows, **i32)
    full_pairs = n * (ctx + 1) / 2
    # ---- the stream's joins
    for name, m in (("", T), (".decode", rows)):
        y, y2, x32, w1 = rnd(m, d), rnd(m, d), f32(m, d), f32(d)
        wb = torch.cat([w1, f32(d, sc=0.1)])
        rec("layer_norm_join" + name, _time(lambda: hops.layer_norm_join(y, x32, wb, 1e-6, bf)), m * d * (2 + 4 + 4 + 2))
        rec("layer_norm_join.two" + name, _time(lambda: hops.layer_norm_join(y, x32, wb, 1e-6, bf, y2)), m * d * (2 + 2 + 4 + 4 + 2))
        rec("kalesun.scale_add_rms_norm" + name, _time(lambda: hops.scale_add_rms_norm(y, x32, w1, 1.0, 1e-6, bf)), m * d * (2 + 4 + 4 + 2))
        rec("zokunex.add_layer_norm" + name, _time(lambda: hops.add_layer_norm(y, x32, w1, 1e-6, bf)), m * d * (2 + 4 + 4 + 2))
        xb, wbf = rnd(m, d), rnd(d)
        rec("llama.add_rmsnorm" + name, _time(lambda: ops.add_rmsnorm(y, xb, wbf, 1e-5)), m * d * (2 + 2 + 2 + 2))
    # ---- attention on unit keys beside the same attention over stored keys, Kalesun's window and Llama's
    H, G, D, K = size["a"]
    F = size["ff"]
    C = (H + G) * D
    width = (C + 2 * F + H + 15) // 16 * 16
    vc, ks = rnd(nb, bs, G, D, sc=0.3), torch.rand(nb, bs, G, device=dev) + 0.5
    proj, projd = rnd(n, width, sc=0.3), rnd(rows, width, sc=0.3)
    taps, temp = f32(C, K, sc=0.5), query_temperature(0.1, 1024, ctx + 2, dev)
    hist = rnd(NS, K - 1, C)
    q, gate = hops.conv_prep(proj, taps, tseq, qs, p0, sl, hist, pos, bt, H, G, D, 1e-6, temp, ks, vc, C + 2 * F, ctx)
    qd, gated = hops.conv_prep(projd, taps, tseqd, qsd, posd, sld, hist, posd, btd, H, G, D, 1e-6, temp, ks, vc, C + 2 * F, 1)
    kc = rnd(nb, bs, G, D, sc=0.3)
    wide, wided = rnd(n, H * D + F), rnd(rows, H * D + F)
    at, atd = (bt, qs, pos), (btd, qsd, posd)
    fl = 4.0 * full_pairs * H * D
    rec("unit_attention.prefill", _time(lambda: hops.window_attention(q, None, vc, *at, None, gate, D ** -0.5, 0, 0, H, bf, ctx, ks=ks, out=wide[:, :H * D]), iters=3, warm=1), flops=fl)
    rec("stored_keys.attention.prefill", _time(lambda: hops.window_attention(q, kc, vc, *at, None, gate, D ** -0.5, 0, 0, H, bf, ctx), iters=3, warm=1), flops=fl)
    rec("unit_attention.decode", _time(lambda: hops.window_attention(qd, None, vc, *atd, None, gated, D ** -0.5, 0, 0, H, bf, 1, ks=ks, out=wided[:, :H * D])),
        nbytes=rows * (ctx + 1) * G * (D * 2.0 + 4.0))
    rec("stored_keys.attention.decode", _time(lambda: hops.window_attention(qd, kc, vc, *atd, None, gated, D ** -0.5, 0, 0, H, bf, 1)),
        nbytes=rows * (ctx + 1) * G * D * 4.0)
    rec("conv_prep.prefill", _time(lambda: hops.conv_prep(proj, taps, tseq, qs, p0, sl, hist, pos, bt, H, G, D, 1e-6, temp, ks, vc, C + 2 * F, ctx)),
        nbytes=n * (C * 4.0 + G * 4.0 + H * 6.0))
    rec("conv_prep.decode", _time(lambda: hops.conv_prep(projd, taps, tseqd, qsd, posd, sld, hist, posd, btd, H, G, D, 1e-6, temp, ks, vc, C + 2 * F, 1)),
        nbytes=rows * (C * 4.0 + 2 * (K - 1) * C * 2.0 + G * 4.0 + H * 6.0))
    kH, kG, kD, kDv, kwin, keep = ksize["a"]
    kkc, kvc = rnd(nb, bs, kG, kD, sc=0.3), rnd(nb, bs, kG, kDv, sc=0.3)
    kqkv, kqkvd = rnd(n, (kH + kG) * kD + kG * kDv, sc=0.3), rnd(rows, (kH + kG) * kD + kG * kDv, sc=0.3)
    kgate, kgated, ksink = f32(n, kH), f32(rows, kH), f32(kH)
    qn, ktab = f32(kD), rope_cos_sin(5e5, kD // 2, ctx + 2, dev)
    kvis = sum(min(i + 1, kwin) + max(0, min(keep, i + 1 - kwin)) for i in range(ctx))
    rec("kalesun.window_attention.prefill", _time(lambda: hops.window_attention(kqkv, kkc, kvc, *at, ksink, kgate, kD ** -0.5, kwin, keep, kH, bf, ctx), iters=3, warm=1),
        flops=2.0 * seqs * kvis * kH * (kD + kDv))
    rec("kalesun.window_attention.decode", _time(lambda: hops.window_attention(kqkvd, kkc, kvc, *atd, ksink, kgated, kD ** -0.5, kwin, keep, kH, bf, 1)),
        nbytes=rows * (min(ctx + 1, kwin) + keep) * kG * (kD + kDv) * 2.0)
    for name, m, x, ps, ts, b_ in (("prefill", n, kqkv, pos, tseq, bt), ("decode", rows, kqkvd, posd, tseqd, btd)):
        rec(f"kalesun.window_prep.{name}", _time(lambda: hops.window_prep(x, kH, kG, kD, kDv, None, None, ps, ts, b_, qn, qn, 1e-5, ktab, kD // 2, kkc, kvc, False)),
            nbytes=m * (2 * (kH + kG) * kD + 2 * kG * kDv) * 2.0)
    dh, dk, dd, dv = ksize["d"]
    Cc = 2 * dk * dd + dh * dv
    xc, xcd, ktaps = rnd(n, Cc + dh * dv), rnd(rows, Cc + dh * dv), f32(Cc, 4)
    khist = torch.zeros(NS, 3, Cc, device=dev, dtype=bf)
    rec("kalesun.short_conv.prefill", _time(lambda: hops.short_conv(xc, ktaps, tseq, qs, p0, sl, khist, True)), nbytes=n * Cc * 4.0)
    rec("kalesun.short_conv.decode", _time(lambda: hops.short_conv(xcd, ktaps, tseqd, qsd, posd, sld, khist, True)), nbytes=rows * Cc * 16.0)
    hq = d // 128
    hkv = max(1, hq // 4)
    akc, avc = rnd(nb, hkv, bs, 128, sc=0.3), rnd(nb, hkv, 128, bs, sc=0.3)
    lq, lqd = rnd(n, hq, 128, sc=0.3), rnd(rows, hq, 128, sc=0.3)
    ctxl, ctxd = torch.full((seqs,), ctx, **i32), torch.full((rows,), ctx + 1, **i32)
    tiles = torch.tensor(ops.attention_tiles([ctx] * seqs, hq, hkv, 8), **i32).view(-1, 2)
    rec("llama.attention.prefill", _time(lambda: ops.paged_attention(lq, akc, avc, bt, qs, ctxl, tiles, tiles.shape[0], 8, 1), iters=3, warm=1),
        flops=4.0 * full_pairs * hq * 128)
    nsp = ops.pick_nsplit(rows * hkv, ctx + 1)
    rec("llama.attention.decode", _time(lambda: ops.paged_attention(lqd, akc, avc, btd, qsd, ctxd, None, rows, 1, nsp)),
        nbytes=rows * (ctx + 1) * hkv * 128 * 2 * 2.0)
    del kc, vc, kkc, kvc, akc, avc, kqkv, lq, xc
    # ---- latent attention with sinks beside Zokunex's
    lH, lD, R, Dv, rank, qr = size["l"]
    DK, nq = rank + R, lH * (lD + R)
    lat = rnd(nb, bs, DK, sc=0.3)
    qa, qad, sink = rnd(n, lH, DK, sc=0.3), rnd(rows, lH, DK, sc=0.3), f32(lH)
    rec("latent_sink.prefill", _time(lambda: hops.latent_attention(qa, lat, *at, None, 0.1, rank, bf, ctx, 0, True, sink), iters=3, warm=1),
        flops=2.0 * full_pairs * lH * (DK + rank))
    rec("latent_sink.decode", _time(lambda: hops.latent_attention(qad, lat, *atd, None, 0.1, rank, bf, 1, 0, True, sink)),
        nbytes=rows * (ctx + 1) * DK * 2.0)
    zH, zD, zR, zDv, zrank = zsize["a"]
    zlat = rnd(nb, bs, zrank + zR, sc=0.3)
    zqa, zqad = rnd(n, zH, zrank + zR, sc=0.3), rnd(rows, zH, zrank + zR, sc=0.3)
    zg, zgd = f32(n, zH), f32(rows, zH)
    rec("zokunex.latent_attention.prefill", _time(lambda: hops.latent_attention(zqa, zlat, *at, zg, 0.1, zrank, bf, ctx), iters=3, warm=1),
        flops=2.0 * full_pairs * zH * (2 * zrank + zR))
    rec("zokunex.latent_attention.decode", _time(lambda: hops.latent_attention(zqad, zlat, *atd, zgd, 0.1, zrank, bf, 1)),
        nbytes=rows * (ctx + 1) * (zrank + zR) * 2.0)
    ltab, wn, wq = rope_cos_sin(5e5, R, ctx + 2, dev, ("ramp", 4.0, 4096.0, 32.0, 1.0)), f32(rank), f32(qr)
    wuk, wuv = rnd(lH, rank, lD, sc=lD ** -0.5), rnd(lH, Dv, rank, sc=rank ** -0.5)
    for name, m, qx, ps, ts, b_ in (("prefill", n, qa, pos, tseq, bt), ("decode", rows, qad, posd, tseqd, btd)):
        lw = (qr + DK + 7) // 8 * 8 + 2 * F
        lproj, lqq, w_out = rnd(m, lw, sc=0.3), rnd(m, lH, lD + R, sc=0.3), rnd(m, lH * Dv + F)
        xf = f32(m, qr)
        rec(f"norm_cols.{name}", _time(lambda: hops.norm_cols(lproj, 0, qr, wq, 1e-6)), nbytes=m * qr * 4.0)
        rec(f"rms_norm.{name}", _time(lambda: hops.rms_norm(xf, wq, 1e-6, bf)), nbytes=m * qr * 6.0)
        rec(f"latent_prep.{name}", _time(lambda: hops.latent_prep(lqq, lproj[:, qr:qr + DK], ps, ts, b_, wn, 1e-6, ltab, R, rank, lat, qx, True)),
            nbytes=m * (2 * DK + 2 * lH * R) * 2.0)
        rec(f"latent_prep.shared.{name}", _time(lambda: hops.latent_prep(lqq, None, ps, ts, b_, None, 1e-6, ltab, R, rank, lat, qx, True)),
            nbytes=m * 2 * lH * R * 2.0)
        oa = rnd(m, lH, rank)
        rec(f"head_matmul.to_latent.{name}", _time(lambda: hops.head_matmul(lqq[:, :, :lD], wuk, qx[:, :, :rank])),
            nbytes=(m * lH * (lD + rank) + lH * lD * rank) * 2.0, flops=2.0 * m * lH * lD * rank)
        rec(f"head_matmul.from_latent.{name}", _time(lambda: hops.head_matmul(oa, wuv, w_out[:, :lH * Dv].view(m, lH, Dv))),
            nbytes=(m * lH * (Dv + rank) + lH * Dv * rank) * 2.0, flops=2.0 * m * lH * Dv * rank)
        # ---- the gated unit on columns, and a layer's products: shared with the mixer's, or each its own
        kz = rnd(m, 2 * ksize["ff"])
        rec(f"glu_cols.{name}", _time(lambda: hops.glu_cols(lproj, lw - 2 * F, F, float("inf"), 1.0, 0.0, w_out[:, lH * Dv:])), nbytes=m * F * 6.0)
        rec(f"kalesun.glu.{name}", _time(lambda: hops.glu(kz, 7.0, 1.702, 1.0, bf)), nbytes=m * ksize["ff"] * 6.0)
    del lat, zlat, qa, zqa, oa, lproj, lqq
    w_in, w_o = rnd(width, d, sc=d ** -0.5), rnd(d, H * D + F, sc=d ** -0.5)
    wq_, wg_, wo_, wd_ = w_in[:C].contiguous(), w_in[C:C + 2 * F].contiguous(), w_o[:, :H * D].contiguous(), w_o[:, H * D:].contiguous()
    wgate = w_in[C + 2 * F:C + 2 * F + H].contiguous()
    lf = int(3.5 * d)
    lgu, ldn = rnd(2 * lf, d, sc=d ** -0.5), rnd(d, lf, sc=lf ** -0.5)
    for name, m in (("prefill", T), ("decode", rows)):
        h, o = rnd(m, d), rnd(m, H * D)
        w_out = rnd(m, H * D + F)

        def fused():
            p = hops.matmul(h, w_in)
            hops.glu_cols(p, C, F, float("inf"), 1.0, 0.0, w_out[:, H * D:])
            return hops.matmul(w_out, w_o)

        def apart():
            hops.matmul(h, wq_)
            hops.rowdot(h, wgate)
            return hops.matmul(o, wo_), hops.matmul(hops.glu(hops.matmul(h, wg_), float("inf"), 1.0, 0.0, bf), wd_)

        fl = 2.0 * m * d * (C + 3 * F + H * D)
        nby = (d * (C + 3 * F + H * D) + m * d * 2) * 2.0
        rec(f"layer_products.shared.{name}", _time(fused, iters=3, warm=1), nbytes=nby, flops=fl)
        rec(f"layer_products.apart.{name}", _time(apart, iters=3, warm=1), nbytes=nby, flops=fl)
        rec(f"llama.mlp.{name}", _time(lambda: ops.linear(ops.gate_up_silu(h, lgu), ldn), iters=3, warm=1),
            nbytes=3 * lf * d * 2.0 + m * d * 4.0, flops=m * 6.0 * lf * d)
    return out


def run_nubodra(sizes: list, seqs: int = 4, plen: int = 2048, rows: int = 64, ctx: int = 2048, device: str = "cuda") -> dict:
    from chronos import ops
    from chronos.models import kalesun, llama, nubodra, zokunex
    from chronos.models.hybrid import HybridDecoder

    dev = torch.device(device if ":" in device else device + ":0")
    torch.cuda.set_device(dev)
    ops.load()
    ops.device_init()
    res = {}
    P = ctx + plen + 16
    for name in sizes:
        size, ksize, zsize = NUBODRA_SIZES[name], KALESUN_SIZES[name], SIZES[name]
        t0 = time.time()
        entry = {}
        for mod, key, conf in ((nubodra, "nubodra", nubodra_config(size)), (kalesun, "kalesun", kalesun_config(ksize)),
                               (zokunex, "zokunex", zokunex_config(zsize))):
            cfg = mod.config_from_dict(conf, name=f"{key}-{name}", max_position=P)
            m = HybridDecoder(cfg, mod.pack_weights(cfg, mod.random_tensors(cfg, 0), dev, torch.bfloat16), dev, P, torch.bfloat16)
            entry[key] = dict(params=cfg.param_count(), **_model_steps(m, dev, seqs, plen, rows, ctx))
            _say(f"size {name}: {key} {entry[key]}")
            del m
        d = size["width"]
        lc = llama.LlamaConfig(name=f"llama-{name}", vocab_size=VOCAB, hidden_size=d, intermediate_size=int(3.5 * d),
                               num_layers=LAYERS, num_heads=d // 128, num_kv_heads=max(1, d // 512), max_position=P)
        lm = llama.LlamaModel(lc, llama.random_weights(lc, None, dev, 0), None, dev, P)
        entry["llama"] = dict(params=lc.param_count(), **_model_steps(lm, dev, seqs, plen, rows, ctx))
        _say(f"  llama {entry['llama']}")
        del lm
        torch.cuda.empty_cache()
        entry["kernels"] = _kernels_nubodra(size, ksize, zsize, dev, seqs * plen, ctx, rows)
        entry["seconds"] = round(time.time() - t0, 1)
        res[name] = entry
        torch.cuda.empty_cache()
    return dict(metric="design_compare", design="nubodra", beside="kalesun, zokunex and llama (equal width and depth)",
                layers=LAYERS, workload=dict(prefill=f"{seqs} x {plen} tokens in one step",
                                             decode=f"{rows} rows at context {ctx}"),
                dtype="bf16", data="synthetic", sizes=res)


def run_kalesun(sizes: list, seqs: int = 4, plen: int = 2048, rows: int = 64, ctx: int = 2048, device: str = "cuda") -> dict:
    from chronos import ops
    from chronos.models import kalesun, llama, zokunex
    from chronos.models.hybrid import HybridDecoder

    dev = torch.device(device if ":" in device else device + ":0")
    torch.cuda.set_device(dev)
    ops.load()
    ops.device_init()
    res = {}
    P = ctx + plen + 16
    for name in sizes:
        size, zsize = KALESUN_SIZES[name], SIZES[name]
        t0 = time.time()
        cfg = kalesun.config_from_dict(kalesun_config(size), name=f"kalesun-{name}", max_position=P)
        km = HybridDecoder(cfg, kalesun.pack_weights(cfg, kalesun.random_tensors(cfg, 0), dev, torch.bfloat16), dev, P,
                           torch.bfloat16)
        entry = dict(kalesun=dict(params=cfg.param_count(), **_model_steps(km, dev, seqs, plen, rows, ctx)))
        _say(f"size {name}: kalesun {entry['kalesun']}")
        del km
        zcfg = zokunex.config_from_dict(zokunex_config(zsize), name=f"zokunex-{name}", max_position=P)
        zk = HybridDecoder(zcfg, zokunex.pack_weights(zcfg, zokunex.random_tensors(zcfg, 0), dev, torch.bfloat16), dev, P,
                           torch.bfloat16)
        entry["zokunex"] = dict(params=zcfg.param_count(), **_model_steps(zk, dev, seqs, plen, rows, ctx))
        _say(f"  zokunex {entry['zokunex']}")
        del zk
        d = size["width"]
        lc = llama.LlamaConfig(name=f"llama-{name}", vocab_size=VOCAB, hidden_size=d, intermediate_size=int(3.5 * d),
                               num_layers=LAYERS, num_heads=d // 128, num_kv_heads=max(1, d // 512), max_position=P)
        lm = llama.LlamaModel(lc, llama.random_weights(lc, None, dev, 0), None, dev, P)
        entry["llama"] = dict(params=lc.param_count(), **_model_steps(lm, dev, seqs, plen, rows, ctx))
        _say(f"  llama {entry['llama']}")
        del lm
        torch.cuda.empty_cache()
        entry["kernels"] = _kernels_kalesun(size, zsize, dev, seqs * plen, ctx, rows)
        entry["seconds"] = round(time.time() - t0, 1)
        res[name] = entry
        torch.cuda.empty_cache()
    return dict(metric="design_compare", design="kalesun", beside="zokunex and llama (equal width and depth)",
                layers=LAYERS, workload=dict(prefill=f"{seqs} x {plen} tokens in one step",
                                             decode=f"{rows} rows at context {ctx}"),
                dtype="bf16", data="synthetic", sizes=res)


def run(sizes: list, seqs: int = 4, plen: int = 2048, rows: int = 64, ctx: int = 2048, device: str = "cuda") -> dict:
    from chronos import ops
    from chronos.models import llama, zokunex
    from chronos.models.hybrid import HybridDecoder

    dev = torch.device(device if ":" in device else device + ":0")
    torch.cuda.set_device(dev)
    ops.load()
    ops.device_init()
    res = {}
    for name in sizes:
        size = SIZES[name]
        t0 = time.time()
        cfg = zokunex.config_from_dict(zokunex_config(size), name=f"zokunex-{name}", max_position=ctx + plen + 16)
        zk = HybridDecoder(cfg, zokunex.pack_weights(cfg, zokunex.random_tensors(cfg, 0), dev, torch.bfloat16), dev,
                           ctx + plen + 16, torch.bfloat16)
        d = size["width"]
        lc = llama.LlamaConfig(name=f"llama-{name}", vocab_size=VOCAB, hidden_size=d, intermediate_size=int(3.5 * d),
                               num_layers=LAYERS, num_heads=d // 128, num_kv_heads=max(1, d // 512),
                               max_position=ctx + plen + 16)
        lm = llama.LlamaModel(lc, llama.random_weights(lc, None, dev, 0), None, dev, ctx + plen + 16)
        _say(f"size {name}: models built")
        entry = dict(zokunex=dict(params=cfg.param_count(), **_model_steps(zk, dev, seqs, plen, rows, ctx)))
        _say(f"  zokunex {entry['zokunex']}")
        entry["llama"] = dict(params=lc.param_count(), **_model_steps(lm, dev, seqs, plen, rows, ctx))
        _say(f"  llama {entry['llama']}")
        entry["kernels"] = _kernels(size, dev, seqs * plen, ctx, rows)
        entry["seconds"] = round(time.time() - t0, 1)
        res[name] = entry
        del zk, lm
        torch.cuda.empty_cache()
    return dict(metric="design_compare", design="zokunex", beside="llama (equal width and depth)", layers=LAYERS,
                workload=dict(prefill=f"{seqs} x {plen} tokens in one step", decode=f"{rows} rows at context {ctx}"),
                dtype="bf16", data="synthetic", sizes=res)


def main(a) -> int:
    sizes = [s for s in a.design_sizes.split(",") if s]
    fn = {"kalesun": run_kalesun, "tugovik": run_tugovik, "vogerax": run_vogerax,
          "lalasun": run_lalasun, "nubodra": run_nubodra}.get(getattr(a, "design", "zokunex"), run)
    out = fn(sizes, device=a.device)
    print(json.dumps(out), flush=True)
    return 0
