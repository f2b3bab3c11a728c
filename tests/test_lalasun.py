"""Lalasun through the framework (registry -> engine -> block manager / state slots -> step batches -> ops) against the
plain token-by-token oracle of tests/oracles/lalasun_plain.py.

CPU runs take the ops' PyTorch path, the ``cuda`` parametrisations (marked gpu) the HIP kernels; both go through the
same engine code.  Sizes are deliberately unlike each other: head groups of 1, 2 and 3, chunks and windows shorter than
a page and longer than two, of one position and none at all, partial and full rotations, latents narrower and wider than
the heads, decay ranks other than the default, layers without a feed-forward, residual multipliers of one and others.
"""
import copy
import json

import pytest
import torch

from tests.oracles import lalasun_plain as plain

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
TOL = {"fp32": 2e-4, "bf16": 0.1}


def _attn(heads=4, kv_heads=2, dim=12, vdim=20, scale=0.4, size=21, rot=8, base=1000.0):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if size:
        mx["mask"] = dict(size=size)
    if rot:
        mx["rot"] = dict(base=base, dims=rot)
    return dict(type="attention", mixer=mx)


def _lat(heads=3, dim=10, rot_dim=6, vdim=14, kv_rank=24, scale=0.3, size=19, base=500.0):
    mx = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, scale=scale,
              rot=dict(base=base, dims=rot_dim))
    if size:
        mx["mask"] = dict(size=size)
    return dict(type="latent_attention", mixer=mx)


def _gla(heads=3, dim=10, vdim=12, tau=8.0, rank=5):
    return dict(type="gla", mixer=dict(heads=heads, dim=dim, vdim=vdim, tau=tau, rank=rank))


def _config(layers, width=64, vocab=97, eps=1e-5, mult=0.45):
    """layers: (mixer, ff size or None)."""
    return dict(architecture="Lalasun", vocab=vocab, width=width, norm=dict(eps=eps), residual_mult=mult,
                layers=[dict(m, mlp=dict(kind="dense", ff=ff) if ff else None) for m, ff in layers])


MIXED = _config([(_gla(), 40), (_attn(), 52), (_lat(), None),
                 (_attn(heads=3, kv_heads=3, dim=16, vdim=8, size=40, scale=0.2, rot=16), 24),
                 (_lat(heads=2, dim=20, rot_dim=8, vdim=6, kv_rank=12, size=33), 36),
                 (_gla(heads=1, dim=24, vdim=40, tau=16.0, rank=16), None)])


def _model(cfg_dict, device, dtype="fp32", seed=0, tensors=None):
    from chronos.models import lalasun
    from chronos.models.hybrid import HybridDecoder

    cfg = lalasun.config_from_dict(cfg_dict, max_position=1024)
    if tensors is None:
        tensors = lalasun.random_tensors(cfg, seed)
    at = torch.float32 if dtype == "fp32" else torch.bfloat16
    return HybridDecoder(cfg, lalasun.pack_weights(cfg, tensors, device, at), device, 1024, at), tensors


def _engine(cfg_dict, device, dtype="fp32", slots=4, max_len=512, blocks=0, seed=0, tensors=None, **kw):
    from chronos.brain.engine.engine import Engine, EngineConfig

    model, tensors = _model(cfg_dict, device, dtype, seed, tensors)
    bs = kw.pop("block_size", 16)
    ec = EngineConfig(model="lalasun-test", device=device, dtype=dtype, max_slots=slots, block_size=bs,
                      max_model_len=max_len, kv_blocks=blocks or slots * (max_len // bs) + 1, warm_formats=(), **kw)
    return Engine(ec, model=model), tensors


def _errs(got, want):
    """Per position: the spread of the difference over the vocabulary relative to the spread of the logits."""
    d = got.double() - want.double()
    d = d - d.mean(-1, keepdim=True)
    w = want.double() - want.double().mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-9)


def _err(got, want):
    return float(_errs(got, want).max())


def _tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def _replay(eng, schedule, reqs):
    """schedule: list of steps, each [(request name, count)].  Returns {name: logits of every token}."""
    from chronos.brain.engine.replay import TraceSession

    ses = TraceSession(eng)
    at = {k: 0 for k in reqs}
    out = {k: [] for k in reqs}
    for step in schedule:
        entries, end = [], []
        for name, count in step:
            lo = at[name]
            entries.append(dict(id=name, tokens=reqs[name][lo:lo + count], want=list(range(count))))
            at[name] = lo + count
            if at[name] == len(reqs[name]):
                end.append(name)
        logits = ses.step(entries, end)
        k = 0
        for name, count in step:
            out[name].append(logits[k:k + count])
            k += count
    assert not ses.live
    return {k: torch.cat(v) for k, v in out.items()}


def _want(cfg, tensors, toks):
    return plain.run(cfg, tensors, toks)[0]


_memo = {}


def _mixed_want(dtype_free_seed, toks):
    """The oracle's answer for MIXED under random weights of that seed (several tests ask for the same)."""
    from chronos.models import lalasun

    key = (dtype_free_seed, tuple(toks))
    if key not in _memo:
        _memo[key] = _want(MIXED, lalasun.random_tensors(lalasun.config_from_dict(MIXED), dtype_free_seed), toks)
    return _memo[key]


# ---- each mechanism alone, layer by layer -------------------------------------------------------------------------
SINGLE = [(_attn(), None), (_attn(heads=3, kv_heads=3, dim=6, vdim=4, size=0, rot=0), None),
          (_attn(heads=6, kv_heads=1, dim=10, vdim=70, size=5, rot=10), 33),
          (_attn(heads=2, kv_heads=2, dim=4, vdim=2, size=1, scale=2.0, rot=2), None),
          (_lat(), None), (_lat(heads=1, dim=3, rot_dim=2, vdim=70, kv_rank=7, size=0), 20),
          (_lat(heads=6, dim=16, rot_dim=16, vdim=16, kv_rank=80, size=5), 64), (_lat(size=1), None),
          (_gla(), None), (_gla(heads=1, dim=5, vdim=3, tau=1.0, rank=1), 40), (_gla(heads=6, dim=20, vdim=40, tau=32.0, rank=9), None)]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("mult", [0.3, 1.0])
@pytest.mark.parametrize("layer", SINGLE)
def test_single_layer_and_residual_stream(device, layer, mult):
    cfg = _config([layer, layer], mult=mult)
    model, tensors = _model(cfg, device)
    toks = _tokens(37, cfg["vocab"], 3)
    taps = []
    model.layer_tap = lambda li, x: taps.append(x.detach().clone().cpu())
    cache = model.make_cache(8, 16, 2)
    sb = model.prefill_batch([toks], [0], [[1, 2, 3]], [1], want=list(range(len(toks))))
    got = model.forward(sb, cache).cpu()
    want, per_layer = plain.run(cfg, tensors, toks)
    assert len(taps) == len(per_layer) == 2
    for li, x in enumerate(taps):
        assert float((x.double() - per_layer[li]).abs().max()) < 2e-4 * float(per_layer[li].abs().max()), f"layer {li}"
    assert _err(got, want) < TOL["fp32"]


def test_the_oracle_feels_every_part():
    """Leaving a part out (by its weights or constants) moves the oracle's logits: what the tests above compare is
    sensitive to every mechanism."""
    from chronos.models import lalasun

    t = lalasun.random_tensors(lalasun.config_from_dict(MIXED), 1)
    toks = _tokens(60, 97, 1)
    want = _want(MIXED, t, toks)
    for name, change in (("l1.rg1.b", lambda x: x + 1), ("l1.rg2", lambda x: x * 0), ("l0.norm1.alpha", lambda x: x * 1.2),
                         ("l1.norm2.b", lambda x: x * 0), ("l3.dwa", lambda x: torch.cat([x[:1] * 0, x[1:]])),
                         ("l4.mlp.act", lambda x: x * torch.tensor([1, 0, 1, 1])), ("l4.mlp.act", lambda x: x * torch.tensor([1, 1, 0, 1])),
                         ("l1.mlp.act", lambda x: x * torch.tensor([1, 1, 1, 0])), ("l2.mix.g", lambda x: x * 0),
                         ("l2.mix.dkv.norm", lambda x: x * 1.5), ("l3.mix.o.b", lambda x: x * 0), ("l3.mix.v.b", lambda x: x * 0),
                         ("l3.mix.q.b", lambda x: x * 0), ("l0.mix.a2.b", lambda x: x - 4), ("final.norm.b", lambda x: x * 0)):
        other = dict(t)
        other[name] = change(t[name].float())
        assert _err(_want(MIXED, other, toks), want) > 2e-3, name
    for path, value in ((("layers", 1, "mixer", "mask", "size"), 22), (("layers", 2, "mixer", "mask", "size"), 20),
                        (("layers", 0, "mixer", "tau"), 9.0), (("residual_mult",), 0.5), (("layers", 2, "mixer", "rot", "base"), 50.0),
                        (("layers", 1, "mixer", "rot", "base"), 100.0), (("layers", 1, "mixer", "scale"), 0.5)):
        c = copy.deepcopy(MIXED)
        at = c
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        assert _err(_want(c, t, toks), want) > 1e-3, path


# ---- visible sets ---------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_sharp_softmax_around_the_edges(device, decode, kind):
    """A large score scale lets single keys carry the answer: a key one position outside the window or chunk, or the
    first one inside dropped, moves the logits.  One edge shorter than a page, the other longer than two; the sequence
    runs through many of both, in portions cut inside them and token by token."""
    one = (lambda size, scale: _attn(heads=2, kv_heads=1, dim=8, vdim=8, scale=scale, size=size)) if kind == "attention" else \
        (lambda size, scale: _lat(heads=2, dim=6, rot_dim=4, vdim=8, kv_rank=12, scale=scale, size=size))
    cfg = _config([(one(11, 5.0), None), (one(37, 3.0), 24)], width=32)
    eng, tensors = _engine(cfg, device, max_len=256)
    toks = _tokens(150, cfg["vocab"], 2)
    sched = [[("r0", 8)]] + [[("r0", 1)] for _ in range(142)] if decode else [[("r0", 33)], [("r0", 2)], [("r0", 115)]]
    want = _want(cfg, tensors, toks)
    assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]
    for size in (10, 12):   # the test must feel an edge that is one position off
        other = copy.deepcopy(cfg)
        other["layers"][0]["mixer"]["mask"]["size"] = size
        assert _err(_want(other, tensors, toks[:40]), want[:40]) > 1e-2


@pytest.mark.parametrize("device,dt", [("cpu", torch.float32), pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
                                       pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)])
@pytest.mark.parametrize("size", [1, 9, 16, 64, 70, 0])
def test_visible_sets_key_by_key(device, dt, size):
    """Zero queries weigh every visible key the same and one-hot values make a query's output its visibility pattern:
    the latent attention's window and the chunked attention (there the added one takes a share of the softmax: every
    visible key weighs 1 / (1 + visible))."""
    from chronos.ops import hybrid as hops

    ctx, bs, H, D = 160, 16, 2, 32
    nb = ctx // bs + 2
    pages = list(range(nb - 1, 0, -1))
    lat = torch.zeros(nb, bs, ctx + D, dtype=dt)
    vc = torch.zeros(nb, bs, 1, ctx, dtype=dt)
    kc = torch.randn(nb, bs, 1, D).to(dt)
    for j in range(ctx):
        lat[pages[j // bs], j % bs, j] = 1.0
        vc[pages[j // bs], j % bs, 0, j] = 1.0
    tol = 1e-6 if dt == torch.float32 else 4e-3
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=device)  # noqa: E731
    bt = torch.zeros(2, nb, dtype=torch.int32)
    bt[1, :len(pages)] = torch.tensor(pages, dtype=torch.int32)
    lat, vc, kc, bt = (t.to(device) for t in (lat, vc, kc, bt))
    for lo, hi in [(0, 160), (0, 1), (63, 65), (64, 130), (159, 160), (5, 6), (69, 71), (8, 10)]:
        n = hi - lo
        qs, pos = i32([0, 0, n]), i32(list(range(lo, hi)))
        a = hops.latent_attention(torch.zeros(n, H, ctx + D, dtype=dt, device=device), lat, bt, qs, pos, None, 1.0, ctx, dt, n,
                                  size, True).float().cpu()
        b = hops.window_attention(torch.zeros(n, (H + 1) * D + ctx, dtype=dt, device=device), kc, vc, bt, qs, pos,
                                  torch.zeros(H, device=device), None, 1.0, 0, 0, H, dt, n, size).view(n, H, ctx).float().cpu()
        for r, i in enumerate(range(lo, hi)):
            for o, sees, extra in ((a, plain.window_visible, 0), (b, plain.chunk_visible, 1)):
                vis = torch.tensor([1.0 if sees(i, j, size) else 0.0 for j in range(ctx)])
                want = vis / (vis.sum() + extra)
                for h in range(H):
                    assert torch.equal(o[r, h] != 0, vis != 0), (lo, hi, i, h)
                    assert float((o[r, h] - want).abs().max()) <= tol * float(want.max()) + 1e-7, (lo, hi, i, h)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_a_far_key(device, kind):
    """One key hundreds of positions back, its score lifted above the others' by scaled query and key weights: the
    answer rests on that key's value alone, across many pages, in a prompt and in decoding."""
    from chronos.models import lalasun

    one = _attn(heads=2, kv_heads=1, dim=8, vdim=8, scale=1.0, size=300) if kind == "attention" else \
        _lat(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=16, scale=1.0, size=290)
    cfg = _config([(one, None)], width=32)
    t = lalasun.random_tensors(lalasun.config_from_dict(cfg), 7)
    for n in ("l0.mix.q", "l0.mix.k", "l0.mix.uk"):
        if n in t:
            t[n] = t[n] * 5
    eng, tensors = _engine(cfg, device, tensors=t, max_len=512)
    toks = _tokens(300, cfg["vocab"], 12)
    want = _want(cfg, tensors, toks)
    sched = [[("r0", 200)], [("r0", 70)]] + [[("r0", 1)] for _ in range(30)]
    assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


@pytest.mark.parametrize("device", DEVICES)
def test_the_added_one_in_the_denominator(device):
    """Scores far below zero: the added one takes nearly the whole softmax; far above: it vanishes."""
    from chronos.models import lalasun

    cfg = _config([(_attn(heads=2, kv_heads=2, dim=8, vdim=8, scale=2.0, size=30), None)], width=32)
    t = lalasun.random_tensors(lalasun.config_from_dict(cfg), 3)
    t["l0.mix.q.b"] = torch.full((16,), 2.0)
    t["l0.mix.k.b"] = torch.cat([torch.full((8,), -1.0), torch.full((8,), 1.0)])
    cfg["layers"][0]["mixer"].pop("rot")
    eng, tensors = _engine(cfg, device, tensors=t)
    toks = _tokens(45, cfg["vocab"], 5)
    want = _want(cfg, tensors, toks)
    assert _err(_replay(eng, [[("r0", 20)]] + [[("r0", 1)] for _ in range(25)], {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


# ---- schedules: whole prompts, decoding, portions, mixed batches ---------------------------------------------------
def _requests(cfg, lens, seed=0):
    return {f"r{i}": _tokens(n, cfg["vocab"], seed + i) for i, n in enumerate(lens)}


def _check(eng, tensors, cfg, schedule, reqs, dtype):
    got = _replay(eng, schedule, reqs)
    for name, toks in reqs.items():
        want = _mixed_want(0, toks) if cfg is MIXED else _want(cfg, tensors, toks)
        assert _err(got[name].cpu(), want) < TOL[dtype], (name, _errs(got[name].cpu(), want))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_prefill_equals_token_by_token(device, dtype):
    eng, tensors = _engine(MIXED, device, dtype)
    reqs = _requests(MIXED, [75, 1, 18])
    sched = [[("r0", 75)], [("r1", 1)]] + [[("r2", 1)] for _ in range(18)]
    _check(eng, tensors, MIXED, sched, reqs, dtype)
    # the same prompt once more, a little of it at once and the rest decoded: the slot and pages are reused, and the
    # decoded tokens pass every window and chunk edge
    sched = [[("r0", 13)]] + [[("r0", 1)] for _ in range(62)]
    _check(eng, tensors, MIXED, sched, {"r0": reqs["r0"]}, dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_portions_of_every_size(device):
    eng, tensors = _engine(MIXED, device)
    reqs = _requests(MIXED, [100], seed=5)
    cuts = [3, 2, 16, 2, 15, 17, 2, 31, 1, 1, 2, 7, 1]
    assert sum(cuts) == 100
    _check(eng, tensors, MIXED, [[("r0", c)] for c in cuts], reqs, "fp32")
    _check(eng, tensors, MIXED, [[("r0", 2)] for _ in range(50)], reqs, "fp32")


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("dtype", ["fp32", "bf16"])
def test_mixed_batches_with_reused_pages_and_slots(device, dtype):
    """Four slots and a pool of 14 pages (block 0 is scratch) for six requests of 212 tokens in all: requests end,
    their pages and slots go to new ones (whose state must start from zero); portions run beside single decoded
    tokens."""
    eng, tensors = _engine(MIXED, device, dtype, slots=4, max_len=128, blocks=15)
    reqs = _requests(MIXED, [70, 9, 33, 1, 40, 59], seed=11)
    sched = [[("r0", 3), ("r1", 1)],
             [("r0", 30), ("r1", 1), ("r2", 2)],
             [("r0", 1), ("r1", 2), ("r2", 29), ("r3", 1)],
             [("r0", 1), ("r1", 1), ("r2", 1), ("r4", 17)],
             [("r0", 16), ("r1", 4), ("r2", 1), ("r4", 1)],      # r1, r2 end
             [("r0", 1), ("r4", 1), ("r5", 2)],
             [("r0", 18), ("r4", 21), ("r5", 31)],               # r0, r4 end
             [("r5", 1)]] + [[("r5", 1)] for _ in range(25)]
    _check(eng, tensors, MIXED, sched, reqs, dtype)
    assert eng.blocks.free == 14 and len(eng.free_slots) == 4


@pytest.mark.parametrize("device", DEVICES)
def test_batch_members_do_not_see_each_other(device):
    eng, tensors = _engine(MIXED, device)
    reqs = _requests(MIXED, [21, 64, 5], seed=21)
    alone = {k: _replay(eng, [[(k, len(v))]], {k: v})[k] for k, v in reqs.items()}
    together = _replay(eng, [[("r0", 21), ("r1", 64), ("r2", 5)]], reqs)
    for k in reqs:
        assert _err(together[k], alone[k]) < 1e-5


@pytest.mark.parametrize("device", DEVICES)
def test_a_request_may_sit_out_steps(device):
    eng, tensors = _engine(MIXED, device)
    reqs = _requests(MIXED, [30, 26], seed=31)
    sched = [[("r0", 7)], [("r1", 5)], [("r1", 1)], [("r0", 2), ("r1", 1)], [("r1", 19)], [("r0", 21)]]
    _check(eng, tensors, MIXED, sched, reqs, "fp32")


@pytest.mark.parametrize("device", DEVICES)
def test_page_borders_and_first_tokens(device):
    """Every position from just before a page border to just after it, decoded and in portions that start and end at
    the border; the first tokens of a sequence one by one (zero state, a lone key)."""
    cfg = _config([(_attn(scale=3.0, size=18), 24), (_lat(scale=2.0, size=17), None), (_gla(), 16)], width=48)
    eng, tensors = _engine(cfg, device, block_size=16)
    toks = _tokens(52, cfg["vocab"], 8)
    want = _want(cfg, tensors, toks)
    for sched in ([[("r0", 1)] for _ in range(52)],
                  [[("r0", 16)], [("r0", 16)], [("r0", 15)], [("r0", 2)], [("r0", 3)]],
                  [[("r0", 15)], [("r0", 2)], [("r0", 30)], [("r0", 5)]]):
        assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding_carries_the_state(device):
    """Decays near one in some channels and near zero in others: 160 decoded tokens after three portions."""
    from chronos.models import lalasun

    cfg = _config([(_gla(heads=2, dim=8, vdim=8, tau=16.0, rank=4), None), (_gla(heads=1, dim=8, vdim=12, tau=2.0, rank=4), 16)],
                  width=32)
    t = lalasun.random_tensors(lalasun.config_from_dict(cfg), 4)
    t["l0.mix.a2.b"] = torch.cat([torch.full((8,), 6.0), torch.full((8,), -30.0)])
    t["l1.mix.a2.b"] = torch.cat([torch.full((4,), 5.0), torch.full((4,), -40.0)])
    eng, tensors = _engine(cfg, device, tensors=t)
    toks = _tokens(210, cfg["vocab"], 6)
    want = _want(cfg, tensors, toks)
    sched = [[("r0", 7)], [("r0", 2)], [("r0", 41)]] + [[("r0", 1)] for _ in range(160)]
    assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]
    assert _err(_want(cfg, dict(t, **{"l0.mix.a2.b": torch.zeros(16)}), toks[:60]), want[:60]) > 1e-2, "must feel the decays"


# ---- designs drawn at random: sizes, order of layers, windows, constants --------------------------------------------
def _random_design(seed, tile_sizes=False):
    """A configuration drawn at random.  ``tile_sizes``: head sizes on the grids of the matrix-core kernels, so that
    bfloat16 runs take them."""
    import random

    r = random.Random(seed)
    pick = r.choice
    layers = []
    for _ in range(r.randint(2, 5)):
        kind = pick("alg")
        size = pick([0, 1, 5, 16, 33, 64, 100])
        if kind == "a":
            kv = pick([1, 2, 3])
            dim = pick([32, 64, 96]) if tile_sizes else pick([6, 10, 24])
            mixer = _attn(heads=kv * pick([1, 2, 4]), kv_heads=kv, dim=dim, vdim=pick([16, 48, 80]) if tile_sizes else pick([6, 20, 34]),
                          scale=pick([0.1, 0.5, 1.5]), size=size, rot=pick([0, 4, dim]), base=pick([100.0, 1e4, 1e6]))
        elif kind == "l":
            mixer = _lat(heads=pick([1, 2, 5]), dim=pick([16, 32, 72]) if tile_sizes else pick([4, 9, 18]),
                         rot_dim=pick([8, 16, 32]) if tile_sizes else pick([2, 6, 10]), vdim=pick([16, 40]) if tile_sizes else pick([5, 12]),
                         kv_rank=pick([32, 64, 144]) if tile_sizes else pick([7, 20, 70]), scale=pick([0.1, 0.4, 1.2]), size=size,
                         base=pick([100.0, 1e4, 1e6]))
            if not tile_sizes and (mixer["mixer"]["kv_rank"] + mixer["mixer"]["rot_dim"]) % 2:
                mixer["mixer"]["kv_rank"] += 1
        else:
            mixer = _gla(heads=pick([1, 2, 4]), dim=pick([4, 16, 36]), vdim=pick([8, 24, 72]), tau=pick([1.0, 4.0, 16.0]), rank=pick([2, 16, 20]))
        layers.append((mixer, pick([None, 24, 50, 64])))
    return _config(layers, width=128 if tile_sizes else pick([24, 40, 70]), vocab=pick([50, 131, 300]),
                   eps=pick([1e-6, 1e-5]), mult=pick([0.2, 1.0, 0.7]))


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("seed", range(8))
def test_designs_drawn_at_random(device, seed):
    cfg = _random_design(seed)
    eng, tensors = _engine(cfg, device, slots=3, max_len=160, blocks=14)
    reqs = _requests(cfg, [90, 37, 2, 61], seed=seed)
    sched = [[("r0", 40), ("r1", 2)], [("r0", 1), ("r1", 33), ("r2", 2)], [("r0", 2), ("r1", 1)], [("r0", 30), ("r1", 1), ("r3", 17)],
             [("r0", 1), ("r3", 3)]] + [[("r0", 1), ("r3", 1)] for _ in range(16)] + [[("r3", 25)]]
    _check(eng, tensors, cfg, sched, reqs, "fp32")


@pytest.mark.gpu
@pytest.mark.parametrize("seed", [11, 12, 13, 14, 15, 16])
def test_designs_drawn_at_random_on_the_matrix_cores(seed):
    """bfloat16 at sizes the matrix-core attention kernels serve, against the oracle; and the same requests cut
    differently."""
    cfg = _random_design(seed, tile_sizes=True)
    eng, tensors = _engine(cfg, "cuda", "bf16", slots=3, max_len=160, blocks=14)
    reqs = _requests(cfg, [90, 61], seed=seed)
    _check(eng, tensors, cfg, [[("r0", 90)], [("r1", 61)]], reqs, "bf16")
    _check(eng, tensors, cfg, [[("r0", 40), ("r1", 2)], [("r0", 1), ("r1", 33)], [("r0", 30), ("r1", 25)], [("r0", 19), ("r1", 1)]],
           reqs, "bf16")


# ---- generation through the engine's own entry point and scheduler ------------------------------------------------
def _greedy(cfg, tensors, prompt, n):
    m = plain.PlainLalasun(cfg, tensors)
    logits = None
    for t in prompt:
        logits = m.step(int(t))[0]
    out = []
    for _ in range(n):
        out.append(int(logits.argmax()))
        logits = m.step(out[-1])[0]
    return out


GEN = _config([(_gla(heads=2, dim=8, vdim=8), 24), (_attn(heads=2, kv_heads=1, dim=8, vdim=8, size=12), None),
               (_lat(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12, size=9), 16),
               (_attn(heads=2, kv_heads=1, dim=8, vdim=8, size=20), None)], width=32, vocab=61)


def _gen_tensors(cfg, seed):
    from chronos.models import lalasun

    t = lalasun.random_tensors(lalasun.config_from_dict(cfg), seed)
    t["head"] = t["head"] * 3   # logits far enough apart for a stable argmax
    t["head"][59:] = 0          # the byte tokenizer's specials score 0 and are never the largest
    return t


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("graphs", [False, True])
def test_greedy_generation_through_the_scheduler(device, graphs):
    """submit() -> admission -> prefill / mixed steps -> decode bursts -> harvest, five requests over two slots and a
    small page pool (slots and pages are reused, arrivals join running decodes), greedy tokens equal to the oracle's."""
    if graphs and device == "cpu":
        pytest.skip("graphs are a GPU feature")
    eng, tensors = _engine(GEN, device, slots=2, max_len=96, blocks=9, tensors=_gen_tensors(GEN, 3), use_graphs=graphs,
                           decode_burst=4, max_prefill_tokens=24, mixed_prefill_tokens=8, prefill_ramp=0)
    prompts = [_tokens(n, 59, 30 + n) for n in (5, 31, 12, 2, 40)]   # (ids 59 and 60 are the byte tokenizer's specials)
    reqs = [eng.submit(p, num_predict=9) for p in prompts[:3]]
    eng.step()
    eng.step()
    reqs += [eng.submit(p, num_predict=9) for p in prompts[3:]]
    eng.run_until_idle(max_steps=2000)
    for r, p in zip(reqs, prompts):
        assert r.done_reason in ("length", "stop"), (r.done_reason, r.error)
        want = _greedy(GEN, tensors, p, 9)
        n = len(r.out_ids)
        # (the engine's free-text automaton spends the last token of the budget on the end-of-text token)
        assert n >= 8 and r.out_ids == want[:n], (r.out_ids, want)
    assert eng.blocks.free == 8 and len(eng.free_slots) == 2


@pytest.mark.parametrize("device", DEVICES)
def test_slot_compaction_and_preemption_carry_the_state(device):
    """Requests that finish at different times leave holes in the low slots, so running sequences are moved down
    (recurrent state moves with them); a page pool too small for all of them forces recompute preemption.  Greedy
    tokens must equal the oracle's throughout."""
    prompts = [_tokens(n, 59, 50 + n) for n in (4, 6, 9, 30)]
    budgets = [3, 5, 24, 26]
    eng, tensors = _engine(GEN, device, slots=4, max_len=96, tensors=_gen_tensors(GEN, 5), use_graphs=False, decode_burst=2,
                           prefill_ramp=0)
    wants = [_greedy(GEN, tensors, p, n) for p, n in zip(prompts, budgets)]
    reqs = [eng.submit(p, num_predict=n) for p, n in zip(prompts, budgets)]
    eng.run_until_idle(max_steps=2000)
    assert eng.stats["compactions"] >= 1
    for r, want in zip(reqs, wants):
        assert len(r.out_ids) >= len(want) - 1 and r.out_ids == want[:len(r.out_ids)], (r.out_ids, want)
    eng, _ = _engine(GEN, device, slots=4, max_len=96, blocks=6, tensors=tensors, use_graphs=False, decode_burst=2,
                     prefill_ramp=0, kv_alloc="lazy", kv_lookahead=2, kv_watermark=0.0)
    reqs = [eng.submit(p, num_predict=n) for p, n in zip(prompts, budgets)]
    eng.run_until_idle(max_steps=4000)
    assert eng.stats["preemptions"] >= 1
    for r, want in zip(reqs, wants):
        assert r.done_reason in ("length", "stop"), (r.done_reason, r.error)
        assert len(r.out_ids) >= len(want) - 1 and r.out_ids == want[:len(r.out_ids)], (r.out_ids, want)


@pytest.mark.parametrize("device", DEVICES)
def test_shared_prefixes_without_recurrent_layers(device):
    """A design without recurrent layers keeps everything in pages: sequences may share a common prefix's pages, and
    greedy tokens stay the oracle's."""
    cfg = _config([(_attn(heads=2, kv_heads=1, dim=8, vdim=8, size=40), 16),
                   (_lat(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12, size=25), None)], width=32, vocab=61)
    eng, tensors = _engine(cfg, device, slots=2, max_len=128, tensors=_gen_tensors(cfg, 2), use_graphs=False, decode_burst=2,
                           prefill_ramp=0, prefix_cache=True)
    assert not eng.model.recurrent
    head = _tokens(50, 59, 1)
    for tail in (_tokens(5, 59, 2), _tokens(9, 59, 3), _tokens(5, 59, 2)):
        r = eng.submit(head + tail, num_predict=8)
        eng.run_until_idle(max_steps=500)
        want = _greedy(cfg, tensors, head + tail, 8)
        assert len(r.out_ids) >= 7 and r.out_ids == want[:len(r.out_ids)]


def test_registry_reads_the_checkpoint_layout(tmp_path):
    from chronos.models import lalasun, registry

    cfg = lalasun.config_from_dict(MIXED)
    tensors = lalasun.random_tensors(cfg, 1)
    assert cfg.param_count() == sum(t.numel() for t in tensors.values())
    lalasun.save(cfg, tensors, str(tmp_path))
    c = json.load(open(tmp_path / "config.json"))
    for l in c["layers"]:
        l["mixer"].pop("rank", None)     # the decay projection's rank is then the stored matrix's
    json.dump(c, open(tmp_path / "config.json", "w"))
    assert registry.family_of(str(tmp_path)).name == "lalasun"
    model = registry.build_model(str(tmp_path), "cpu", dtype="fp32", max_position=64)
    assert model.recurrent and model.cfg.residual_mult == 0.45 and model.cfg.layers[0].mixer.rank == 5
    toks = _tokens(9, cfg.vocab_size, 0)
    sb = model.prefill_batch([toks], [0], [[1]], [0], want=list(range(9)))
    assert _err(model.forward(sb, model.make_cache(2, 16, 1)), _mixed_want(1, toks)) < TOL["fp32"]
    # keys a configuration may leave out take their neutral values
    lean = copy.deepcopy(c)
    lean.pop("residual_mult")
    for l in lean["layers"]:
        for k in ("mask", "rot", "kv_heads"):
            l["mixer"].pop(k, None)
    c2 = lalasun.config_from_dict(lean)
    a, b = c2.layers[1].mixer, c2.layers[2].mixer
    assert (a.chunk, a.rope_dims, a.kv_heads, b.window, b.rope_dims, c2.residual_mult) == (0, 0, 4, 0, 0, 1.0)
    for change in (lambda q: q["layers"][0].update(type="conv"), lambda q: q["layers"][1]["mixer"].update(kv_heads=3),
                   lambda q: q["layers"][1]["mixer"]["rot"].update(dims=14), lambda q: q["layers"][2]["mixer"]["rot"].update(dims=5),
                   lambda q: q["layers"][0]["mlp"].update(kind="moe")):
        bad = copy.deepcopy(MIXED)
        change(bad)
        with pytest.raises(ValueError):
            lalasun.config_from_dict(bad)
    assert "lalasun-tiny" in registry.family_of("lalasun-tiny").presets()
    wrong = dict(tensors)
    wrong["l1.dwa"] = wrong["l1.dwa"][:2]
    with pytest.raises(ValueError):
        lalasun.pack_weights(cfg, wrong, "cpu", torch.float32)


def test_gated_stream_options_on_their_own():
    """The stream's options are independent: RMS norms with gates from a projection of their own, no depth average; and
    combinations that make no sense are refused."""
    import dataclasses

    from chronos.models import lalasun
    from chronos.models.hybrid import HybridDecoder

    d = dict(_config([(_attn(), 20), (_gla(), None)], width=24, mult=0.6))
    cfg = lalasun.config_from_dict(d)
    t = lalasun.random_tensors(cfg, 2)
    w = lalasun.pack_weights(cfg, t, "cpu", torch.float32)
    for i, lw in enumerate(w.layers):     # the gate's rows leave the sublayers' projections
        for mix, key, gate, name in ((lw.mix, "w_qkv" if i == 0 else "w_proj", lw.gate1, f"l{i}.rg1"), (lw.ff, "w_up", lw.gate2, f"l{i}.rg2")):
            if mix:
                off = mix.pop("rg_off")
                mix[key] = mix[key][:off].contiguous()
                if "b_qkv" in mix:
                    mix["b_qkv"] = mix["b_qkv"][:off].contiguous()
                gate["w"] = t[name].float()
    toks = _tokens(20, d["vocab"], 4)

    def logits(c, ww):
        m = HybridDecoder(c, ww, "cpu", 64, torch.float32)
        return m.forward(m.prefill_batch([toks], [0], [[1, 2]], [0], want=list(range(20))), m.make_cache(3, 16, 1))

    assert _err(logits(cfg, w), _want(d, t, toks)) < TOL["fp32"]
    rms = dataclasses.replace(cfg, norm="rms", depth_average=False)
    for lw in w.layers:
        lw.dwa = None
        lw.norm1 = torch.ones(24)
        lw.norm2 = torch.ones(24) if lw.norm2 is not None else None
    w.final_norm = torch.ones(24)
    assert torch.isfinite(logits(rms, w)).all()
    for bad in (dict(residual="sandwich"), dict(norm="batch"), dict(loop=(0, 1, 2)), dict(token_side=4)):
        with pytest.raises(ValueError):
            HybridDecoder(dataclasses.replace(cfg, **bad), w, "cpu", 64, torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("width", [512, 1024])
def test_wide_model_on_the_routed_projections(width):
    """Widths at which single decode rows take the framework's GEMV and the projections its tiled GEMMs: bfloat16
    prefill against token-by-token decoding against the oracle."""
    cfg = _config([(_gla(heads=4, dim=64, vdim=128, tau=16.0, rank=16), 1024),
                   (_attn(heads=8, kv_heads=2, dim=64, vdim=64, scale=0.125, size=24, rot=64), 640),
                   (_lat(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=256, scale=0.1, size=21), None)], width=width, vocab=320)
    eng, tensors = _engine(cfg, "cuda", "bf16", max_len=128)
    toks = _tokens(40, 320, 3)
    want = _want(cfg, tensors, toks)
    for sched in ([[("r0", 40)]], [[("r0", 9)]] + [[("r0", 1)] for _ in range(31)]):
        assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["bf16"]
