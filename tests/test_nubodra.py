"""Nubodra through the framework (registry -> engine -> block manager / state slots -> step batches -> ops) against the
plain token-by-token oracle of tests/oracles/nubodra_plain.py.

CPU runs take the ops' PyTorch path, the ``cuda`` parametrisations (marked gpu) the HIP kernels; both go through the
same engine code.  Sizes are deliberately unlike each other: head groups of 1, 2 and 3, value heads wider and narrower
than query heads, latents narrower and wider than the heads, 1 to 6 convolution taps, layers without a feed-forward,
feed-forwards on and off the grid on which they share the mixer's products, embedding scales of one and others.
"""
import copy
import json

import pytest
import torch

from tests.oracles import nubodra_plain as plain

DEVICES = ["cpu", pytest.param("cuda", marks=pytest.mark.gpu)]
TOL = {"fp32": 2e-4, "bf16": 0.1}


def _attn(heads=4, kv_heads=2, dim=12, scale=0.4, conv=3, coef=0.7, every=5):
    mx = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=dim, conv=conv, scale=scale)
    if every:
        mx["q_temp"] = dict(coef=coef, every=every)
    return dict(type="attention", mixer=mx)


RAMP = dict(factor=4.0, original=100, fast=6.0, slow=1.0)


def _lat(heads=3, dim=10, rot_dim=12, vdim=14, kv_rank=24, q_rank=20, scale=0.3, base=50.0, scaling=RAMP, kv_from=None):
    mx = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, kv_rank=kv_rank, q_rank=q_rank, scale=scale,
              rot=dict(base=base, dims=rot_dim))
    if scaling:
        mx["rot"]["scaling"] = dict(scaling)
    if kv_from is not None:
        mx["kv_from"] = kv_from
    return dict(type="latent_attention", mixer=mx)


def _config(layers, width=64, vocab=97, eps=1e-5, embed=1.7):
    """layers: (mixer, ff size or None)."""
    return dict(architecture="Nubodra", vocab=vocab, width=width, norm=dict(eps=eps), embedding=dict(scale=embed),
                layers=[dict(m, mlp=dict(kind="dense", ff=ff) if ff else None) for m, ff in layers])


MIXED = _config([(_lat(), 40), (_attn(), 52), (_lat(kv_from=0, heads=2, dim=6, vdim=8, q_rank=9, scale=0.5), None),
                 (_attn(heads=3, kv_heads=3, dim=16, conv=4, scale=0.2, coef=-0.3, every=9), 24),
                 (_lat(heads=2, dim=20, rot_dim=8, vdim=6, kv_rank=12, q_rank=33, scaling=None), 36),
                 (_lat(heads=4, dim=8, rot_dim=8, vdim=8, kv_rank=12, q_rank=16, scaling=None, kv_from=4), 48),
                 (_attn(heads=1, kv_heads=1, dim=24, conv=1, every=0), None)])


def _model(cfg_dict, device, dtype="fp32", seed=0, tensors=None):
    from chronos.models import nubodra
    from chronos.models.hybrid import HybridDecoder

    cfg = nubodra.config_from_dict(cfg_dict, max_position=1024)
    if tensors is None:
        tensors = nubodra.random_tensors(cfg, seed)
    at = torch.float32 if dtype == "fp32" else torch.bfloat16
    return HybridDecoder(cfg, nubodra.pack_weights(cfg, tensors, device, at), device, 1024, at), tensors


def _engine(cfg_dict, device, dtype="fp32", slots=4, max_len=512, blocks=0, seed=0, tensors=None, **kw):
    from chronos.brain.engine.engine import Engine, EngineConfig

    model, tensors = _model(cfg_dict, device, dtype, seed, tensors)
    bs = kw.pop("block_size", 16)
    ec = EngineConfig(model="nubodra-test", device=device, dtype=dtype, max_slots=slots, block_size=bs,
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


def _mixed_want(seed, toks):
    """The oracle's answer for MIXED under random weights of that seed (several tests ask for the same)."""
    from chronos.models import nubodra

    key = (seed, tuple(toks))
    if key not in _memo:
        _memo[key] = _want(MIXED, nubodra.random_tensors(nubodra.config_from_dict(MIXED), seed), toks)
    return _memo[key]


# ---- each mechanism alone, layer by layer -------------------------------------------------------------------------
SINGLE = [[(_attn(), None)] * 2, [(_attn(heads=3, kv_heads=3, dim=6, conv=1, every=0), 17)] * 2,
          [(_attn(heads=6, kv_heads=1, dim=70, conv=6, scale=0.1, coef=2.0, every=1), 33)] * 2,
          [(_attn(heads=2, kv_heads=2, dim=32, conv=2, every=7.5), 48)] * 2, [(_lat(), None)] * 2,
          [(_lat(heads=1, dim=3, rot_dim=2, vdim=70, kv_rank=8, q_rank=1, scaling=None), 20)] * 2,
          [(_lat(heads=6, dim=16, rot_dim=16, vdim=16, kv_rank=80, q_rank=40), 64), (_lat(heads=5, dim=4, rot_dim=16, vdim=8, kv_rank=80, q_rank=7, kv_from=0), 24)],
          [(_lat(heads=2, vdim=12, q_rank=70, scaling=dict(factor=16.0, original=8, fast=32.0, slow=0.5)), 40)] * 2]


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("layers", SINGLE)
def test_single_layers_and_residual_stream(device, layers):
    cfg = _config(layers, embed=1.0 if len(layers[0][0]["mixer"]) % 2 else 2.5)
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
    from chronos.models import nubodra

    t = nubodra.random_tensors(nubodra.config_from_dict(MIXED), 1)
    toks = _tokens(40, 97, 1)
    want = _want(MIXED, t, toks)
    for name, change in (("l0.norm1.b", lambda x: x * 0), ("l1.norm1", lambda x: x * 0 + 1), ("final.norm.b", lambda x: x * 0),
                         ("l0.mix.dq.norm", lambda x: x * 0 + 1), ("l0.mix.dkv.norm", lambda x: x * 0 + 1), ("l0.mix.sink", lambda x: x - 30),
                         ("l2.mix.sink", lambda x: x + 2), ("l1.mix.g", lambda x: x * 0), ("l1.mix.q.conv", lambda x: x * torch.tensor([0, 1, 1])),
                         ("l1.mix.k.conv", lambda x: x * torch.tensor([1, 0, 1])), ("l3.mix.q.conv", lambda x: x.flip(1)),
                         ("l6.mix.k.conv", lambda x: x * 0 + 1), ("l1.mlp.gate", lambda x: x * 0), ("l4.mlp.up", lambda x: x * 1.2),
                         ("l5.mix.uk", lambda x: x * 0)):
        other = dict(t)
        other[name] = change(t[name].float())
        assert _err(_want(MIXED, other, toks), want) > 2e-3, name
    mixer = lambda i, *k: ("layers", i, "mixer", *k)  # noqa: E731
    for path, value in ((("embedding", "scale"), 1.0), (mixer(0, "scale"), 0.4), (mixer(0, "rot", "base"), 500.0),
                        (mixer(0, "rot", "scaling", "factor"), 2.0), (mixer(0, "rot", "scaling", "original"), 1000),
                        (mixer(0, "rot", "scaling", "fast"), 1.2), (mixer(0, "rot", "scaling", "slow"), 0.2), (mixer(1, "scale"), 0.5),
                        (mixer(1, "q_temp", "coef"), 0.0), (mixer(1, "q_temp", "every"), 4), (mixer(4, "rot", "base"), 500.0),
                        (("norm", "eps"), 1e-2)):
        c = copy.deepcopy(MIXED)
        at = c
        for k in path[:-1]:
            at = at[k]
        at[path[-1]] = value
        assert _err(_want(c, t, toks), want) > 1e-3, path
    c = copy.deepcopy(MIXED)      # a layer on another layer's latents: of the layer it names and no other
    c["layers"][5]["mixer"]["kv_from"] = None
    other = dict(t, **{"l5.mix.dkv": t["l4.mix.dkv"].flip(0), "l5.mix.dkv.norm": t["l4.mix.dkv.norm"]})
    assert _err(_want(c, other, toks), want) > 1e-2


# ---- single keys ----------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_sharp_softmax(device, decode, kind):
    """A large score scale lets single keys carry the answer: one key missing, twice there or under a wrong page moves
    the logits.  Pages of 8 positions, a sequence that runs through 19 of them, in portions cut inside pages and token by
    token; the query's temperature passes many of its steps."""
    one = (lambda s: _attn(heads=2, kv_heads=1, dim=8, scale=s, conv=3, coef=0.4, every=3)) if kind == "attention" else \
        (lambda s: _lat(heads=2, dim=6, rot_dim=4, vdim=8, kv_rank=12, q_rank=10, scale=s))
    cfg = _config([(one(5.0), None), (one(3.0), 24)], width=32)
    eng, tensors = _engine(cfg, device, max_len=256, block_size=8)
    toks = _tokens(150, cfg["vocab"], 2)
    sched = [[("r0", 8)]] + [[("r0", 1)] for _ in range(142)] if decode else [[("r0", 33)], [("r0", 2)], [("r0", 115)]]
    want = _want(cfg, tensors, toks)
    assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


@pytest.mark.parametrize("device,dt", [("cpu", torch.float32), pytest.param("cuda", torch.float32, marks=pytest.mark.gpu),
                                       pytest.param("cuda", torch.bfloat16, marks=pytest.mark.gpu)])
def test_visible_sets_key_by_key(device, dt):
    """Zero queries weigh every visible key the same and one-hot values make a query's output its visibility pattern, in
    both attentions; the latent one with a sink of score 0 (every visible key weighs 1 / (1 + visible)) and with one
    far below."""
    from chronos.ops import hybrid as hops

    ctx, bs, H, D = 160, 16, 2, 32
    nb = ctx // bs + 2
    pages = list(range(nb - 1, 0, -1))
    lat = torch.zeros(nb, bs, ctx + D, dtype=dt)
    vc = torch.zeros(nb, bs, 1, ctx, dtype=dt)
    for j in range(ctx):
        lat[pages[j // bs], j % bs, j] = 1.0
        vc[pages[j // bs], j % bs, 0, j] = 1.0
    ks = torch.rand(nb, bs, 1) + 0.5
    tol = 1e-6 if dt == torch.float32 else 4e-3
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=device)  # noqa: E731
    bt = torch.zeros(2, nb, dtype=torch.int32)
    bt[1, :len(pages)] = torch.tensor(pages, dtype=torch.int32)
    lat, vc, ks, bt = (t.to(device) for t in (lat, vc, ks, bt))
    sink = torch.tensor([0.0, -80.0], device=device)
    for lo, hi in [(0, 160), (0, 1), (63, 65), (64, 130), (159, 160), (5, 6), (69, 71), (8, 10)]:
        n = hi - lo
        qs, pos = i32([0, 0, n]), i32(list(range(lo, hi)))
        a = hops.latent_attention(torch.zeros(n, H, ctx + D, dtype=dt, device=device), lat, bt, qs, pos, None, 1.0, ctx, dt, n,
                                  0, True, sink).float().cpu()
        b = hops.window_attention(torch.zeros(n, H * ctx, dtype=dt, device=device), None, vc, bt, qs, pos, None, None, 1.0, 0, 0,
                                  H, dt, n, ks=ks).view(n, H, ctx).float().cpu()
        for r, i in enumerate(range(lo, hi)):
            vis = (torch.arange(ctx) <= i).float()
            for o, extra in ((a[r, 0], 1), (a[r, 1], 0), (b[r, 0], 0), (b[r, 1], 0)):
                want = vis / (vis.sum() + extra)
                assert torch.equal(o != 0, vis != 0), (lo, hi, i)
                assert float((o - want).abs().max()) <= tol * float(want.max()) + 1e-7, (lo, hi, i)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_a_far_key(device, kind):
    """One key hundreds of positions back whose score stands out: the answer rests on that key's value alone, across
    many pages, in a prompt and in decoding.  (Unit keys: the score stands out by the temperature; latents: by scaled
    query and key weights.)"""
    from chronos.models import nubodra

    one = _attn(heads=2, kv_heads=1, dim=8, scale=1.0, coef=3.0, every=20) if kind == "attention" else \
        _lat(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=16, q_rank=12, scale=1.0)
    cfg = _config([(one, None)], width=32)
    t = nubodra.random_tensors(nubodra.config_from_dict(cfg), 7)
    for n in ("l0.mix.uq", "l0.mix.uk"):
        if n in t:
            t[n] = t[n] * 5
    eng, tensors = _engine(cfg, device, tensors=t, max_len=512)
    toks = _tokens(300, cfg["vocab"], 12)
    want = _want(cfg, tensors, toks)
    sched = [[("r0", 200)], [("r0", 70)]] + [[("r0", 1)] for _ in range(30)]
    assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


@pytest.mark.parametrize("device", DEVICES)
def test_sinks_below_among_and_above_the_scores(device):
    from chronos.models import nubodra

    cfg = _config([(_lat(heads=4), None), (_lat(heads=4, kv_from=0, q_rank=8), 16)], width=32)
    t = nubodra.random_tensors(nubodra.config_from_dict(cfg), 3)
    t["l0.mix.sink"] = torch.tensor([-40.0, 0.5, 6.0, 30.0])
    t["l1.mix.sink"] = torch.tensor([9.0, -1.0, -90.0, 3.0])
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
    # the same prompt once more, a little of it at once and the rest decoded: the slot and pages are reused
    sched = [[("r0", 13)]] + [[("r0", 1)] for _ in range(62)]
    _check(eng, tensors, MIXED, sched, {"r0": reqs["r0"]}, dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_portions_of_every_size(device):
    """Also portions shorter than the convolution's history (of one and two tokens, four taps)."""
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
    their pages and slots go to new ones (whose convolutions must start from zeros); portions run beside single decoded
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
    the border; the first tokens of a sequence one by one (an empty convolution history, a lone key beside the sink)."""
    cfg = _config([(_attn(scale=3.0), 24), (_lat(scale=2.0), None), (_lat(scale=1.0, kv_from=1), 16)], width=48)
    eng, tensors = _engine(cfg, device, block_size=16)
    toks = _tokens(52, cfg["vocab"], 8)
    want = _want(cfg, tensors, toks)
    for sched in ([[("r0", 1)] for _ in range(52)],
                  [[("r0", 16)], [("r0", 16)], [("r0", 15)], [("r0", 2)], [("r0", 3)]],
                  [[("r0", 15)], [("r0", 2)], [("r0", 30)], [("r0", 5)]]):
        assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


@pytest.mark.parametrize("device", DEVICES)
def test_long_decoding(device):
    """220 decoded tokens after three portions, with a convolution whose weight lies on the OLDEST of five taps."""
    from chronos.models import nubodra

    cfg = _config([(_attn(heads=2, kv_heads=1, dim=8, conv=5, scale=1.0, coef=0.5, every=16), None),
                   (_lat(heads=2, dim=8, rot_dim=8, vdim=8, kv_rank=12, q_rank=8, scale=0.7), 16)], width=32)
    t = nubodra.random_tensors(nubodra.config_from_dict(cfg), 4)
    for n in ("l0.mix.q.conv", "l0.mix.k.conv"):
        t[n] = t[n].flip(1).contiguous()
    eng, tensors = _engine(cfg, device, tensors=t)
    toks = _tokens(270, cfg["vocab"], 6)
    want = _want(cfg, tensors, toks)
    sched = [[("r0", 7)], [("r0", 2)], [("r0", 41)]] + [[("r0", 1)] for _ in range(220)]
    assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["fp32"]


# ---- designs drawn at random: sizes, order of layers, constants -----------------------------------------------------
def _random_design(seed, tile_sizes=False):
    """A configuration drawn at random.  ``tile_sizes``: head sizes on the grids of the matrix-core kernels, so that
    bfloat16 runs take them."""
    import random

    r = random.Random(seed)
    pick = r.choice
    layers, own = [], []
    for i in range(r.randint(2, 6)):
        kind = pick("al" if not own else "alss")
        if kind == "a":
            kv = pick([1, 2, 3])
            m = _attn(heads=kv * pick([1, 2, 4]), kv_heads=kv, dim=pick([32, 64, 96, 128]) if tile_sizes else pick([6, 10, 24, 32]),
                      scale=pick([0.1, 0.5, 1.5]), conv=pick([1, 2, 3, 4, 5]), coef=pick([0.1, 1.0]), every=pick([0, 1, 7, 64]))
        else:
            kw = dict(heads=pick([1, 2, 5]), dim=pick([16, 32, 72]) if tile_sizes else pick([4, 9, 18]), scale=pick([0.1, 0.4, 1.2]),
                      vdim=pick([16, 40]) if tile_sizes else pick([5, 12]), q_rank=pick([16, 48, 120]) if tile_sizes else pick([3, 12, 33]))
            if kind == "l":
                own.append(i)
                own_kw = dict(rot_dim=pick([8, 16, 32]) if tile_sizes else pick([2, 6, 10]), base=pick([100.0, 1e4, 1e6]),
                              kv_rank=pick([32, 64, 144]) if tile_sizes else pick([8, 20, 70]),
                              scaling=pick([None, dict(factor=8.0, original=64, fast=32.0, slow=1.0), dict(factor=2.5, original=30, fast=3.0, slow=0.7)]))
                own[-1] = (i, own_kw)
                m = _lat(**kw, **own_kw)
            else:
                src, own_kw = pick(own)
                m = _lat(**kw, **own_kw, kv_from=src)
        layers.append((m, pick([None, 24, 50, 64])))
    return _config(layers, width=128 if tile_sizes else pick([24, 40, 70]), vocab=pick([50, 131, 300]),
                   eps=pick([1e-6, 1e-5]), embed=pick([1.0, 0.4, 3.0]))


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
    m = plain.PlainNubodra(cfg, tensors)
    logits = None
    for t in prompt:
        logits = m.step(int(t))[0]
    out = []
    for _ in range(n):
        out.append(int(logits.argmax()))
        logits = m.step(out[-1])[0]
    return out


GEN = _config([(_attn(heads=2, kv_heads=1, dim=8, conv=4), 24), (_lat(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12, q_rank=10), None),
               (_attn(heads=2, kv_heads=2, dim=16, conv=2), 16), (_lat(heads=2, dim=4, rot_dim=4, vdim=12, kv_rank=12, q_rank=7, kv_from=1), 32)],
              width=32, vocab=61)


def _gen_tensors(cfg, seed):
    from chronos.models import nubodra

    t = nubodra.random_tensors(nubodra.config_from_dict(cfg), seed)
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
def test_slot_compaction_and_preemption_carry_the_history(device):
    """Requests that finish at different times leave holes in the low slots, so running sequences are moved down (the
    convolutions' histories move with them); a page pool too small for all of them forces recompute preemption.  Greedy
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
def test_shared_prefixes_without_convolutions(device):
    """A design of latent layers (or of one-tap convolutions) keeps everything in pages: sequences may share a common
    prefix's pages, and greedy tokens stay the oracle's."""
    cfg = _config([(_attn(heads=2, kv_heads=1, dim=8, conv=1), 16), (_lat(heads=2, dim=8, rot_dim=4, vdim=8, kv_rank=12, q_rank=9), None),
                   (_lat(heads=1, dim=8, rot_dim=4, vdim=8, kv_rank=12, q_rank=9, kv_from=1), 16)], width=32, vocab=61)
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
    from chronos.models import nubodra, registry

    cfg = nubodra.config_from_dict(MIXED)
    tensors = nubodra.random_tensors(cfg, 1)
    assert cfg.param_count() == sum(t.numel() for t in tensors.values())
    assert nubodra.config_from_dict(nubodra.config_to_dict(cfg)) == cfg
    nubodra.save(cfg, tensors, str(tmp_path))
    c = json.load(open(tmp_path / "config.json"))
    for l in c["layers"]:     # sizes that the stored tensors have too
        l["mixer"].pop("conv", None)
        l["mixer"].pop("q_rank", None)
    json.dump(c, open(tmp_path / "config.json", "w"))
    assert registry.family_of(str(tmp_path)).name == "nubodra"
    model = registry.build_model(str(tmp_path), "cpu", dtype="fp32", max_position=64)
    assert model.recurrent and model.cfg.embed_scale == 1.7 and [getattr(l.mixer, "conv", 0) for l in model.cfg.layers] == [0, 3, 0, 4, 0, 0, 1]
    toks = _tokens(9, cfg.vocab_size, 0)
    sb = model.prefill_batch([toks], [0], [[1]], [0], want=list(range(9)))
    assert _err(model.forward(sb, model.make_cache(2, 16, 1)), _mixed_want(1, toks)) < TOL["fp32"]
    # keys a configuration may leave out take their neutral values
    lean = copy.deepcopy(MIXED)
    lean.pop("embedding")
    for l in lean["layers"]:
        for k in ("q_temp", "kv_heads", "rot", "kv_from"):
            l["mixer"].pop(k, None)
    c2 = nubodra.config_from_dict(lean)
    a, b = c2.layers[1].mixer, c2.layers[2].mixer
    assert (a.q_temp, a.kv_heads, b.rope_dims, b.kv_from, c2.embed_scale) == (None, 4, 0, None, 1.0)
    mixer = lambda q, i: q["layers"][i]["mixer"]  # noqa: E731
    for change in (lambda q: q["layers"][0].update(type="conv"), lambda q: mixer(q, 1).update(kv_heads=3), lambda q: mixer(q, 1).update(vdim=20),
                   lambda q: mixer(q, 1).pop("conv"), lambda q: mixer(q, 0).pop("q_rank"), lambda q: mixer(q, 0)["rot"].update(dims=14),
                   lambda q: mixer(q, 0)["rot"].update(dims=5), lambda q: q["layers"][0]["mlp"].update(kind="moe")):
        bad = copy.deepcopy(MIXED)
        change(bad)
        with pytest.raises(ValueError):
            nubodra.config_from_dict(bad)
    for change in (lambda q: mixer(q, 2).update(kv_from=4), lambda q: mixer(q, 2).update(kv_from=1), lambda q: mixer(q, 5).update(kv_from=2),
                   lambda q: mixer(q, 2).update(kv_rank=20), lambda q: mixer(q, 2)["rot"].update(base=400.0), lambda q: mixer(q, 2).update(kv_from=-1)):
        bad = copy.deepcopy(MIXED)
        change(bad)
        with pytest.raises(ValueError):
            _model(bad, "cpu")
    assert "nubodra-tiny" in registry.family_of("nubodra-tiny").presets()
    wrong = dict(tensors)
    wrong["l1.mix.q.conv"] = wrong["l1.mix.q.conv"][:, :2]
    with pytest.raises(ValueError):
        nubodra.pack_weights(cfg, wrong, "cpu", torch.float32)


def test_shared_latents_take_no_pages_of_their_own():
    from chronos.models import nubodra
    from chronos.models.hybrid import HybridCache

    cfg = nubodra.config_from_dict(MIXED)
    cache = HybridCache(cfg, 3, 16, "cpu", torch.bfloat16, 2)
    assert cache.lat[2] is cache.lat[0] and cache.lat[5] is cache.lat[4] and not cache.kc and set(cache.ks) == {1, 3, 6}
    held = {id(t): t for d in (cache.lat, cache.vc, cache.ks) for t in d.values()}
    per_page = sum(t[0].numel() * t.element_size() for t in held.values())
    assert HybridCache.bytes_per_block(cfg, 16, torch.bfloat16) == per_page


def test_mechanisms_in_other_combinations():
    """The pieces are options of their own: a convolution before weighted norms, rotation and separately cached keys and
    values; a feed-forward with products of its own; unit keys without a convolution.  And combinations that make no
    sense are refused."""
    import dataclasses

    from chronos.models import nubodra
    from chronos.models.hybrid import FEED_FORWARDS, MIXERS, HybridDecoder, LayerSpec, WindowAttentionSpec

    d = _config([(_attn(heads=4, kv_heads=2, dim=16), 24), (_lat(), 40)], width=24)
    cfg = nubodra.config_from_dict(d)
    t = nubodra.random_tensors(cfg, 2)
    w = nubodra.pack_weights(cfg, t, "cpu", torch.float32)
    assert "ff" in w.layers[0].mix and not w.layers[0].ff
    toks = _tokens(20, d["vocab"], 4)

    def logits(c, ww, cuts=(20,)):
        m = HybridDecoder(c, ww, "cpu", 64, torch.float32)
        cache, out, at = m.make_cache(3, 16, 1), [], 0
        for n in cuts:
            out.append(m.forward(m.prefill_batch([toks[at:at + n]], [at], [[1, 2]], [0], want=list(range(n))), cache))
            at += n
        return torch.cat(out)

    want = _want(d, t, toks)
    assert _err(logits(cfg, w), want) < TOL["fp32"]
    # the feed-forward's products leave the mixer's
    sub = lambda p: {n[len(p):]: x for n, x in t.items() if n.startswith(p)}  # noqa: E731
    for i, l in enumerate(cfg.layers):
        w.layers[i].mix = MIXERS[l.mixer.kind][1](l.mixer, sub(f"l{i}.mix."), "cpu", torch.float32)
        w.layers[i].ff = FEED_FORWARDS["glu"][1](l.ff, sub(f"l{i}.mlp."), "cpu", torch.float32)
        assert "ff" not in w.layers[i].mix
    assert _err(logits(cfg, w), want) < TOL["fp32"]
    # the same attention with stored keys and norms whose weights are one: another cache, the same numbers
    spec = dataclasses.replace(cfg.layers[0].mixer, qk_norm_weight=True)
    assert cfg.layers[0].mixer.unit_keys and not spec.unit_keys
    stored = dataclasses.replace(cfg, layers=[LayerSpec(spec, cfg.layers[0].ff), cfg.layers[1]])
    w.layers[0].mix = MIXERS[spec.kind][1](spec, {**sub("l0.mix."), "q.norm": torch.ones(16), "k.norm": torch.ones(16)}, "cpu", torch.float32)
    assert _err(logits(stored, w, (7, 1, 12)), want) < TOL["fp32"]
    # convolved values of their own, rotation, partly rotated heads: cut anywhere, the same
    full = WindowAttentionSpec(4, 2, 16, 8, 0.3, rope_dims=8, conv=3, sink=False, q_temp=(0.5, 3.0))
    g = torch.Generator().manual_seed(1)
    rn = lambda *s: torch.randn(*s, generator=g) * 0.3  # noqa: E731
    w.layers[0].mix = MIXERS[full.kind][1](full, {"q": rn(64, 24), "k": rn(32, 24), "v": rn(16, 24), "q.norm": rn(16) + 1, "k.norm": rn(16) + 1,
                                                  "q.conv": rn(64, 3), "k.conv": rn(32, 3), "v.conv": rn(16, 3), "g": rn(4, 24), "o": rn(24, 32)},
                                           "cpu", torch.float32)
    c3 = dataclasses.replace(cfg, layers=[LayerSpec(full, cfg.layers[0].ff), cfg.layers[1]])
    assert _err(logits(c3, w, (1, 2, 9, 1, 7)), logits(c3, w)) < 1e-5
    # unit keys without a convolution
    plain_keys = dataclasses.replace(cfg.layers[0].mixer, conv=0)
    c4 = dataclasses.replace(cfg, layers=[LayerSpec(plain_keys, cfg.layers[0].ff), cfg.layers[1]])
    w.layers[0].mix = MIXERS[plain_keys.kind][1](plain_keys, sub("l0.mix."), "cpu", torch.float32)
    one_tap = {n: (torch.ones_like(x[:, :1]) if n.startswith("l0") and n.endswith(".conv") else x) for n, x in t.items()}
    assert _err(logits(c4, w, (5, 15)), _want(d, one_tap, toks)) < TOL["fp32"]
    for bad in (dict(norm="rms"), dict(residual="pre_norm"), dict(norm="batch"), dict(residual="both")):
        with pytest.raises(ValueError):
            HybridDecoder(dataclasses.replace(cfg, **bad), w, "cpu", 64, torch.float32)


@pytest.mark.gpu
@pytest.mark.parametrize("width", [512, 1024])
def test_wide_model_on_the_routed_projections(width):
    """Widths at which single decode rows take the framework's GEMV and the projections its tiled GEMMs: bfloat16
    prefill against token-by-token decoding against the oracle."""
    cfg = _config([(_attn(heads=8, kv_heads=2, dim=64, scale=0.125, conv=4, coef=0.2, every=16), 512),
                   (_lat(heads=8, dim=64, rot_dim=32, vdim=64, kv_rank=256, q_rank=512, scale=0.1), 1024),
                   (_lat(heads=8, dim=64, rot_dim=32, vdim=128, kv_rank=256, q_rank=128, scale=0.1, kv_from=1), None)], width=width, vocab=320)
    eng, tensors = _engine(cfg, "cuda", "bf16", max_len=128)
    toks = _tokens(40, 320, 3)
    want = _want(cfg, tensors, toks)
    for sched in ([[("r0", 40)]], [[("r0", 9)]] + [[("r0", 1)] for _ in range(31)]):
        assert _err(_replay(eng, sched, {"r0": toks})["r0"].cpu(), want) < TOL["bf16"]
