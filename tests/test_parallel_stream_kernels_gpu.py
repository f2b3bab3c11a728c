"""The kernels of the parallel stream (layer norm with the join, gated unit and RMS norm on columns of wider rows), of the
convolved attention with unit keys and of the latent attention with sinks and shared latents, against their PyTorch
references (chronos.ops.hybrid_ref), in both activation dtypes, at sizes on and off the kernels' tiles."""
import pytest
import torch

pytestmark = pytest.mark.gpu

DEV = "cuda"
DTYPES = [torch.bfloat16, torch.float32]


@pytest.fixture(scope="module", autouse=True)
def _lib():
    from chronos.ops import hybrid as hops

    hops.load()
    import chronos.native as n

    assert "_H" in n._loaded, "the hybrid HIP library must be the one running"


def _gen(seed):
    return torch.Generator(device=DEV).manual_seed(seed)


def _rand(g, *shape, dtype=torch.float32, scale=1.0):
    return (torch.randn(*shape, device=DEV, generator=g) * scale).to(dtype)


def _i32(x):
    return torch.tensor(x, dtype=torch.int32, device=DEV)


def _close(a, b, tol):
    a, b = a.float(), b.float()
    err = float((a - b).abs().max()) if a.numel() else 0.0
    ref = float(b.abs().max()) + 1e-6 if b.numel() else 1.0
    assert err <= tol * ref, f"max err {err:.4g} vs magnitude {ref:.4g}"


def _tol(dt, f32=2e-5, bf16=1.5e-2):
    return f32 if dt == torch.float32 else bf16


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,d", [(1, 96), (7, 257), (65, 1000), (6, 1024), (3, 4096), (2, 5000), (2, 8196), (1, 20000), (1, 6001)])
def test_layer_norm_join(dt, T, d):
    """Plain norm, one summand, two summands, nothing emitted; rows with a large mean, where a one-pass variance would
    cancel."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(T * d)
    wb = torch.cat([_rand(g, d) + 1, _rand(g, d)])
    for mean in (0.0, 50.0):
        x0 = _rand(g, T, d, scale=1.5) + mean
        y, y2 = _rand(g, T, d, dtype=dt), _rand(g, T, d, dtype=dt)
        for a, b, emit in ((None, None, True), (y, None, True), (y, y2, True), (y, y2, False)):
            xa, xb = x0.clone(), x0.clone()
            ha = hops.layer_norm_join(a, xa, wb, 1e-5, dt, b, emit)
            hb = ref.layer_norm_join(a, xb, wb, 1e-5, dt, b, emit)
            _close(xa, xb, 1e-6)
            if emit:
                assert ha.dtype == dt
                _close(ha, hb, _tol(dt, 3e-5, 8e-3))
            else:
                assert ha is None


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,F,off,pad,left", [(1, 40, 0, 0, 0), (9, 333, 3, 5, 7), (65, 256, 64, 16, 512), (3, 1404, 8, 4, 20), (70, 64, 16, 0, 8)])
def test_glu_and_norm_on_columns(dt, T, F, off, pad, left):
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(F + off)
    src = _rand(g, T, off + 2 * F + pad, dtype=dt, scale=3.0)
    for limit, slope, shift in ((float("inf"), 1.0, 0.0), (2.0, 1.702, 1.0)):
        a, b = (torch.full((T, left + F + pad), 7.0, device=DEV, dtype=dt) for _ in range(2))
        hops.glu_cols(src, off, F, limit, slope, shift, a[:, left:left + F])
        ref.glu_cols(src, off, F, limit, slope, shift, b[:, left:left + F])
        _close(a, b, _tol(dt, 3e-6, 8e-3))
        assert bool((a[:, :left] == 7).all()) and bool((a[:, left + F:] == 7).all())
    for n in (1, F, min(2 * F, 2100)):
        w = _rand(g, n) + 1
        _close(hops.norm_cols(src, off, n, w, 1e-5), ref.norm_cols(src, off, n, w, 1e-5), _tol(dt, 3e-6, 8e-3))


def _stream(lens, starts, bs):
    """Flattened step: metadata tensors and page tables (pages in falling order; block 0 is scratch)."""
    B = len(lens)
    per = max((s + n + bs - 1) // bs for s, n in zip(starts, lens))
    ids = list(range(B * per, 0, -1))
    bt = _i32([ids[b * per:(b + 1) * per] for b in range(B)])
    pos = [s + i for s, n in zip(starts, lens) for i in range(n)]
    seq = [b for b, n in enumerate(lens) for _ in range(n)]
    qs = [0]
    for n in lens:
        qs.append(qs[-1] + n)
    return dict(bt=bt, pos=_i32(pos), seq=_i32(seq), qs=_i32(qs), pos0=_i32(starts), T=qs[-1], NB=B * per + 1, slots=_i32(list(range(B, 0, -1))))


CONV = [(4, 2, 32, 3), (3, 3, 64, 4), (8, 1, 128, 2), (2, 1, 256, 1), (6, 2, 24, 3), (5, 1, 64, 6), (4, 4, 80, 2), (40, 8, 128, 4),
        (1, 1, 7, 3)]


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D,K", CONV)
@pytest.mark.parametrize("lens,starts", [([37], [0]), ([1, 1, 1], [0, 9, 40]), ([5, 1, 70, 2], [0, 33, 7, 1]), ([1], [1]), ([2100], [3])])
def test_conv_prep(dt, H, G, D, K, lens, starts):
    """Convolution, norms, temperature, cache write and the gates' copy against the separate references, and the history
    a later step starts from; sequences that start, go on, and bring fewer tokens than the history holds."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    m = _stream(lens, starts, 16)
    g = _gen(H * D + K + m["T"])
    C, off = (H + G) * D, (H + G) * D + 8 * (D % 8 == 0)
    proj = _rand(g, m["T"], (off + H + 15) // 16 * 16, dtype=dt)
    taps, temp = _rand(g, C, K, scale=0.6), torch.rand(m["T"] + 64, device=DEV, generator=g) + 0.5
    hist0 = _rand(g, len(lens) + 2, K - 1, C, dtype=dt)
    for tm, go in ((temp, off), (None, -1)):
        out = []
        for f in (lambda h, ks, vc: hops.conv_prep(proj, taps, m["seq"], m["qs"], m["pos0"], m["slots"], h, m["pos"], m["bt"], H, G, D,
                                                   1e-6, tm, ks, vc, go, max(lens)),
                  lambda h, ks, vc: ref.conv_prep(proj, taps, m["qs"], m["pos0"], m["slots"], h, m["pos"], m["seq"], m["bt"], H, G, D,
                                                  1e-6, tm, ks, vc, go)):
            h, ks, vc = hist0.clone(), torch.zeros(m["NB"], 16, G, device=DEV), torch.zeros(m["NB"], 16, G, D, device=DEV, dtype=dt)
            q, gate = f(h, ks, vc)
            out.append((q, gate, h, ks, vc))
        (qa, ga, ha, ka, va), (qb, gb, hb, kb, vb) = out
        _close(qa, qb, _tol(dt, 1e-5, 1.2e-2))
        assert torch.equal(ha, hb)
        _close(va, vb, _tol(dt, 1e-5, 8e-3))
        nz = kb != 0
        assert torch.equal(ka != 0, nz)
        _close(ka[nz] / kb[nz], torch.ones_like(kb[nz]), _tol(dt, 1e-5, 1.2e-2))
        if go >= 0:
            assert torch.equal(ga, gb)
        else:
            assert ga is None and gb is None


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D", [(4, 2, 32), (6, 2, 24), (3, 3, 64), (8, 1, 128), (12, 2, 96), (5, 5, 256)])
@pytest.mark.parametrize("lens,starts", [([70], [0]), ([1, 1, 1], [200, 0, 63]), ([33, 1, 2], [5, 130, 64]), ([1], [900]), ([150], [60])])
def test_attention_on_unit_keys(dt, H, G, D, lens, starts):
    """One cached row that is value and, times its factor, key: with and without gate and sink, into columns of wider
    rows; also through a window.  Equal to the attention over separately stored keys."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    m = _stream(lens, starts, 16)
    g = _gen(D + m["T"])
    q = _rand(g, m["T"], H * D, dtype=dt)
    vc = _rand(g, m["NB"], 16, G, D, dtype=dt, scale=2.0)
    ks = torch.rsqrt(vc.float().pow(2).mean(-1) + 1e-6)
    gate, sink = _rand(g, m["T"], H), _rand(g, H)
    at = (m["bt"], m["qs"], m["pos"])
    for gt, sk, window in ((gate, None, 0), (None, sink, 0), (gate, sink, 50)):
        want = ref.window_attention(q, None, vc, *at, sk, gt, D ** -0.5, window, 0, H, torch.float32, ks=ks)
        for left in (0, 24):
            wide = torch.full((m["T"], H * D + left), 7.0, device=DEV, dtype=dt)
            out = wide[:, :H * D]
            got = hops.window_attention(q, None, vc, *at, sk, gt, D ** -0.5, window, 0, H, dt, max(lens), ks=ks, out=out if left else None)
            _close(got, want, _tol(dt, 2e-5, 1.2e-2))
            if left:
                assert got.data_ptr() == wide.data_ptr() and bool((wide[:, H * D:] == 7).all())
        if dt == torch.float32:
            kc = vc * ks[..., None]
            _close(hops.window_attention(q, kc, vc, *at, sk, gt, D ** -0.5, window, 0, H, dt, max(lens)), want, 2e-5)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,G,D,dims", [(4, 2, 24, 8), (2, 1, 64, 0)])
def test_window_prep_temperature_and_unit_keys(dt, H, G, D, dims):
    """The queries' factor by position beside norms and rotation; and unit keys without a convolution."""
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    m = _stream([20, 3], [0, 30], 16)
    g = _gen(D)
    qkv = _rand(g, m["T"], (H + 2 * G) * D, dtype=dt)
    temp = torch.rand(64, device=DEV, generator=g) + 0.5
    cs = rope_cos_sin(1000.0, dims, 64, DEV) if dims else None
    qn, kn = (_rand(g, D) + 1 for _ in range(2)) if dims else (None, None)
    for unit in ((False, True) if not dims else (False,)):
        res = []
        for mod in (hops, ref):
            x = qkv.clone()
            vc = torch.zeros(m["NB"], 16, G, D, device=DEV, dtype=dt)
            kc = None if unit else torch.zeros_like(vc)
            ks = torch.zeros(m["NB"], 16, G, device=DEV) if unit else None
            mod.window_prep(x, H, G, D, D, None, None, m["pos"], m["seq"], m["bt"], qn, kn, 1e-6, cs, dims, kc, vc, False,
                            H * D if unit else -1, None, temp, ks)
            res.append((x[:, :H * D], vc, ks if unit else kc))
        for a, b in zip(*res):
            _close(a, b, _tol(dt, 1e-5, 1e-2))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("H,R,rank", [(2, 16, 32), (6, 16, 128), (3, 8, 40), (16, 64, 512), (5, 4, 130), (8, 32, 64)])
@pytest.mark.parametrize("lens,starts", [([70], [0]), ([1, 1, 1], [200, 0, 63]), ([33, 1, 2], [5, 130, 64]), ([1], [900])])
def test_latent_attention_with_sinks(dt, H, R, rank, lens, starts):
    """Sinks far below, among and far above the scores, with and without a gate and a window, one workgroup per row block
    and key ranges split over several."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    m = _stream(lens, starts, 16)
    g = _gen(rank + m["T"])
    cache = _rand(g, m["NB"], 16, rank + R, dtype=dt)
    qa = _rand(g, m["T"], H, rank + R, dtype=dt)
    gate = _rand(g, m["T"], H)
    scale = (rank + R) ** -0.5
    for sink, gt, window in ((torch.linspace(-30, 12, H, device=DEV), None, 0), (_rand(g, H), gate, 0), (_rand(g, H, scale=3.0), None, 40)):
        want = ref.latent_attention(qa, cache, m["bt"], m["qs"], m["pos"], gt, scale, rank, torch.float32, window, sink)
        got = hops.latent_attention(qa, cache, m["bt"], m["qs"], m["pos"], gt, scale, rank, dt, max(lens), window, True, sink)
        for h in range(H):   # heads under a large sink are small: each against its own size
            _close(got[:, h], want[:, h], _tol(dt, 3e-5, 1.2e-2))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("dims", [0, 6, 8])
def test_latent_prep_on_shared_latents(dt, dims):
    """Without columns of its own a layer rotates its queries and leaves the cache alone."""
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    m = _stream([20, 3], [0, 30], 16)
    g = _gen(dims)
    H, D, R, rank = 3, 10, 8, 24
    q = _rand(g, m["T"], H, D + R, dtype=dt)
    cs = rope_cos_sin(1000.0, dims, 64, DEV, ("ramp", 4.0, 32.0, 8.0, 1.0)) if dims else None
    cache = _rand(g, m["NB"], 16, rank + R, dtype=dt)
    before = cache.clone()
    a, b = (torch.zeros(m["T"], H, rank + R, device=DEV, dtype=dt) for _ in range(2))
    hops.latent_prep(q, None, m["pos"], m["seq"], m["bt"], None, 1e-6, cs, dims, rank, cache, a, True)
    ref.latent_prep(q, None, m["pos"], m["seq"], m["bt"], None, 1e-6, cs, dims, rank, cache, b, True)
    assert torch.equal(cache, before)
    _close(a, b, _tol(dt, 1e-6, 8e-3))
