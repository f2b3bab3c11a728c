"""The kernels of the gated pre-norm stream (Dynamic Tanh, gated join with depth averages, PolyNorm), the per-head products
and the windowed latent attention against their PyTorch references (chronos.ops.hybrid_ref), in both activation dtypes,
at sizes on and off the kernels' tiles."""
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


def _close(a, b, tol):
    a, b = a.float(), b.float()
    err = float((a - b).abs().max())
    ref = float(b.abs().max()) + 1e-6
    assert err <= tol * ref, f"max err {err:.4g} vs magnitude {ref:.4g}"


def _tol(dt, f32=2e-5, bf16=1.5e-2):
    return f32 if dt == torch.float32 else bf16


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,d", [(1, 96), (7, 257), (65, 1000), (3, 4096)])
def test_dyn_tanh(dt, T, d):
    """Slopes from nearly linear to saturated, and values around zero, where a difference of exponentials would cancel."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(T * d)
    for alpha, scale in ((0.7, 1.0), (5.0, 8.0), (0.3, 1e-4), (-1.0, 0.3)):
        wba = torch.cat([_rand(g, d) + 1, _rand(g, d, scale=0.0 if scale < 1e-3 else 0.2), torch.tensor([alpha], device=DEV)])
        x = _rand(g, T, d, scale=scale)
        _close(hops.dyn_tanh(x, wba, dt), ref.dyn_tanh(x, wba, dt), _tol(dt, 3e-6, 8e-3))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,d,pad,off", [(1, 96, 0, 0), (9, 250, 3, 1), (65, 256, 64, 32), (5, 1000, 7, 7), (3, 4096, 512, 512)])
def test_gated_join(dt, T, d, pad, off):
    """With and without a gate, its bias, a depth average (first, middle and last run) and an emitted norm; the gate in
    columns of a wider projection, on and off the vector grid."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(T + d)
    y = _rand(g, T, d, dtype=dt)
    src = _rand(g, T, d + pad, dtype=dt, scale=2.0)
    gb, wba = _rand(g, d), torch.cat([_rand(g, d), _rand(g, d), torch.tensor([0.8], device=DEV)])
    for gate, bias, run, runs, emit in ((True, True, 0, 3, True), (True, True, 2, 3, False), (True, False, 1, 3, True),
                                        (False, False, -1, 0, True), (True, True, -1, 0, True), (True, True, 6, 8, True)):
        x = _rand(g, T, d, scale=3.0)
        hist = _rand(g, runs, T, d) if run >= 0 else None
        dwa = _rand(g, run + 2) if run >= 0 else None
        x2, hist2 = x.clone(), hist.clone() if run >= 0 else None
        args = (src if gate else None, off if gate else -1, gb if bias else None, 0.35, wba if emit else None, dt)
        h = hops.gated_join(y, x, *args, hist, run, dwa, emit)
        h2 = ref.gated_join(y, x2, *args, hist2, run, dwa, emit)
        _close(x, x2, 2e-6)
        if run >= 0:
            _close(hist, hist2, 2e-6)
        assert (h is None) == (not emit)
        if emit:
            _close(h, h2, _tol(dt, 5e-6, 8e-3))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,F,pad", [(1, 40, 0), (9, 250, 3), (5, 384, 256), (3, 1025, 0), (7, 4096, 64), (2, 5000, 8), (3, 14336, 0),
                                     (2, 17000, 4)])
def test_poly_norm(dt, T, F, pad):
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(F)
    z = _rand(g, T, F + pad, dtype=dt, scale=1.3)
    z[0] *= 1e-3   # eps decides
    abce = torch.tensor([0.7, -0.4, 0.3, 0.15], device=DEV)
    _close(hops.poly_norm(z, F, abce, 1e-5, dt), ref.poly_norm(z, F, abce, 1e-5, dt), _tol(dt, 1e-5, 8e-3))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("T,H,N,K,pa,po", [(1, 2, 128, 32, 16, 16), (70, 3, 100, 24, 8, 4), (65, 5, 33, 7, 3, 1), (300, 4, 64, 256, 0, 0),
                                           (300, 3, 200, 136, 8, 8), (130, 2, 512, 128, 64, 64), (257, 6, 32, 512, 0, 0),
                                           (513, 1, 48, 40, 0, 4)])
def test_head_matmul(dt, T, H, N, K, pa, po):
    """Rows that are column ranges of wider ones (which must stay untouched), with and without gate columns."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(T + N + K)
    a = _rand(g, T, H, K + pa, dtype=dt)
    w = _rand(g, H, N, K, dtype=dt, scale=K ** -0.5)
    wide = _rand(g, T, H, N + po, dtype=dt)
    keep = wide[:, :, N:].clone()
    src = _rand(g, T, 24 + H * N, dtype=dt)
    hops.head_matmul(a[:, :, :K], w, wide[:, :, :N])
    _close(wide[:, :, :N], ref.head_matmul(a[:, :, :K], w), _tol(dt, 5e-6, 8e-3))
    assert torch.equal(wide[:, :, N:], keep)
    for off in (24, 8, 5):
        _close(hops.head_matmul(a[:, :, :K], w, None, src, off), ref.head_matmul(a[:, :, :K], w, None, src, off), _tol(dt, 5e-6, 8e-3))


def _stream(lens, starts):
    qs = [0]
    for n in lens:
        qs.append(qs[-1] + n)
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=DEV)  # noqa: E731
    return (i32(qs), i32([s + i for n, s in zip(lens, starts) for i in range(n)]),
            i32([b for b, n in enumerate(lens) for _ in range(n)]))


def _paged(g, lens, starts, BS, DK, dt, width=0):
    nblk = [(s + n + BS - 1) // BS for n, s in zip(lens, starts)]
    perm = torch.randperm(sum(nblk) + 2, generator=torch.Generator().manual_seed(1)).add(1).tolist()
    bt = torch.zeros(len(lens), max(max(nblk) + 1, width), dtype=torch.int32)
    for b, nb in enumerate(nblk):
        for j in range(nb):
            bt[b, j] = perm.pop()
    return _rand(g, sum(nblk) + 3, BS, DK, dtype=dt), bt.to(DEV)


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("inter", [True, False])
@pytest.mark.parametrize("H,D,R,rank,dims", [(2, 24, 32, 32, 16), (3, 5, 6, 40, 6), (6, 32, 16, 128, 16), (70, 8, 32, 96, 32), (2, 8, 4, 8, 0)])
def test_latent_prep_from_one_projection(dt, inter, H, D, R, rank, dims):
    """q | dkv as column ranges of one projection that must stay as it is; rotated query columns land in qa."""
    from chronos.models.hybrid import rope_cos_sin
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(H + D + rank)
    lens, starts = [21, 1, 1, 5], [0, 200, 0, 63]
    q_start, pos, seq = _stream(lens, starts)
    T, DK, nq = sum(lens), rank + R, H * (D + R)
    cache, bt = _paged(g, lens, starts, 16, DK, dt)
    cache2 = cache.clone()
    proj = _rand(g, T, nq + DK + 8, dtype=dt)
    before = proj.clone()
    qa = torch.zeros(T, H, DK, device=DEV, dtype=dt)
    qa2 = qa.clone()
    cs = rope_cos_sin(1e4, dims, 512, DEV) if dims else None
    wn = _rand(g, rank) * 0.1 + 1
    for fn, c, o in ((hops.latent_prep, cache, qa), (ref.latent_prep, cache2, qa2)):
        fn(proj[:, :nq].view(T, H, D + R), proj[:, nq:nq + DK], pos, seq, bt, wn, 1e-6, cs, dims, rank, c, o, inter)
    assert torch.equal(proj, before)
    _close(qa, qa2, _tol(dt, 1e-6, 8e-3))
    _close(cache, cache2, _tol(dt, 1e-6, 8e-3))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("window", [1, 16, 33, 64, 100, 1000])
@pytest.mark.parametrize("H,R,rank", [(2, 16, 32), (6, 16, 128), (3, 8, 40), (16, 64, 512), (5, 4, 130)])
def test_windowed_latent_attention(dt, window, H, R, rank):
    """Portions over a cached prefix, decode rows far beyond the window, first tokens; row widths on and off the 32-column
    step of the matrix-core kernel; a wide block table, so that few-row launches split their keys."""
    from chronos.ops import hybrid as hops, hybrid_ref as ref

    g = _gen(H + rank + window)
    lens, starts = [70, 1, 1, 5, 130, 0, 2], [0, 700, 0, 63, 217, 3, 899]
    q_start, pos, _ = _stream(lens, starts)
    T, DK = sum(lens), rank + R
    cache, bt = _paged(g, lens, starts, 16, DK, dt, 128)
    qa = _rand(g, T, H, DK, dtype=dt, scale=0.3)
    gate = _rand(g, T, H)
    for two in (True, False):
        for gt in (None, gate):
            o = hops.latent_attention(qa, cache, bt, q_start, pos, gt, 0.17, rank, dt, max(lens), window, two)
            o2 = ref.latent_attention(qa, cache, bt, q_start, pos, gt, 0.17, rank, dt, window)
            _close(o, o2, _tol(dt, 2e-5, 1e-2))
    rows = [70, 71, T - 2, T - 1]     # the decode rows and the two-token portion in a launch of their own
    qs = torch.tensor([0, 1, 2, 4], dtype=torch.int32, device=DEV)
    o3 = hops.latent_attention(qa[rows].contiguous(), cache, bt[[1, 2, 6]].contiguous(), qs, pos[rows].contiguous(), None, 0.17,
                               rank, dt, 2, window, True)
    _close(o3, ref.latent_attention(qa, cache, bt, q_start, pos, None, 0.17, rank, dt, window)[rows], _tol(dt, 2e-5, 1e-2))


@pytest.mark.parametrize("dt", DTYPES)
@pytest.mark.parametrize("window", [1, 5, 64, 70])
def test_latent_window_visible_set(dt, window):
    """Zero queries weigh every visible key the same and one-hot latents make a query's output its visibility pattern."""
    from chronos.ops import hybrid as hops

    ctx, R, H = 192, 16, 2
    cache = torch.zeros(ctx // 16 + 1, 16, ctx + R, dtype=dt)
    pages = list(range(ctx // 16, 0, -1))
    for j in range(ctx):
        cache[pages[j // 16], j % 16, j] = 1.0
    bt = torch.tensor([pages], dtype=torch.int32, device=DEV)
    for lo, hi in [(0, 192), (0, 1), (63, 65), (64, 130), (191, 192), (5, 6), (69, 71)]:
        n = hi - lo
        qa = torch.zeros(n, H, ctx + R, dtype=dt, device=DEV)
        i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=DEV)  # noqa: E731
        o = hops.latent_attention(qa, cache.to(DEV), bt, i32([0, n]), i32(list(range(lo, hi))), None, 1.0, ctx, dt, n, window,
                                  True).float().cpu()
        for r, i in enumerate(range(lo, hi)):
            vis = torch.tensor([1.0 if j <= i and i - j < window else 0.0 for j in range(ctx)])
            for h in range(H):
                assert torch.equal(o[r, h] != 0, vis != 0), (lo, hi, i, h)
                assert float((o[r, h] - vis / vis.sum()).abs().max()) <= 4e-3 / float(vis.sum()) + 1e-7
