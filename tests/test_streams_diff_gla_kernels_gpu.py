"""HIP kernels behind the Nosuzen mixers, residual and feed-forward against the PyTorch rendering of
the same ops (CPU tensors), in fp32 and bf16: the pass over parallel residual streams with its
dynamic tanh, the convolved input pass with two maps per head, windows that keep the first tokens,
differential attention, rotations with a magnitude, gated linear attention (matrix-instruction chunks
and the walking kernel), and the router with rescaled weights."""
import pytest
import torch

from p2p_llm_chat_go_amd.ops import seqmix as sm

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
PAGE = 64


def _tol(dt):
    return dict(rtol=2e-2, atol=2e-2) if dt == torch.bfloat16 else dict(rtol=2e-4, atol=3e-5)


def _d(*ts):
    return [None if t is None else t.to(DEV) for t in ts]


def _step(lens, starts, slots=None):
    ent, r0 = [], 0
    for i, (n, s) in enumerate(zip(lens, starts)):
        ent.append((r0, n, s, i if slots is None else slots[i]))
        r0 += n
    row_ent = torch.tensor([i for i, e in enumerate(ent) for _ in range(e[1])], dtype=torch.int32)
    pos = torch.tensor([s + i for n, s in zip(lens, starts) for i in range(n)], dtype=torch.int32)
    return ent, torch.tensor(ent, dtype=torch.int32), row_ent, pos, r0


# decode only / short portions / long portions (chunks) beside short ones and single tokens
STEPS = {"decode": ([1, 1, 1], [0, 5, 77]), "short": ([5, 1, 2, 30], [0, 3, 1, 64]),
         "long": ([150, 1, 64, 129, 2, 16, 17], [0, 9, 0, 33, 2, 0, 70]), "one_long": ([200], [0])}


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("R,n", [(3, 200), (300, 1028), (9, 37), (270, 33)])   # four channels per thread / one
@pytest.mark.parametrize("NS", [1, 2, 3, 4, 7])
def test_stream_pass(dt, R, n, NS):
    g = torch.Generator().manual_seed(0)
    x0 = torch.randn(R, NS, n, generator=g)
    table, ids = torch.randn(50, n, generator=g).to(dt), torch.randint(0, 50, (R,), generator=g, dtype=torch.int32)
    a, b = (torch.randn(R, n + 4, generator=g).to(dt)[:, 4:] for _ in range(2))
    mix, out, read = (torch.randn(*s, generator=g) for s in ((NS, NS), (NS,), (NS,)))
    dyt = (0.7, torch.randn(n, generator=g), torch.randn(n, generator=g))
    top = 3
    routed = (torch.randn(R * top, n, generator=g).to(dt), torch.rand(R, top, generator=g))
    rows = torch.randperm(R, generator=g)[:max(1, R // 2)].to(torch.int32)
    full = dict(mix=mix, out=out)
    cases = [dict(embed=(table, ids, 1.7), read=read, dyt=dyt), dict(embed=(table, ids, 0.5)),
             dict(a=a, read=read, dyt=dyt, **full), dict(a=a, b=b, routed=routed, read=read, **full),
             dict(routed=routed, dyt=dyt, **full), dict(a=a, routed=routed, **full), dict(a=a, nothing=True, **full),
             dict(dyt=dyt, rows=rows, write=False), dict(a=a, routed=routed, dyt=dyt, rows=rows, write=False, **full)]
    up = lambda v, dev: tuple(t.to(dev) if torch.is_tensor(t) else t for t in v) if isinstance(v, tuple) else \
        v.to(dev) if torch.is_tensor(v) else v
    for kw in cases:
        kw = dict(kw)
        quiet = kw.pop("nothing", False)            # no sublayer follows: only the streams are updated
        res = []
        for dev in ("cpu", DEV):
            x = x0.clone().to(dev)
            h = None if quiet else torch.zeros(R, n, dtype=dt, device=dev)
            sm.stream_mix(x, h=h, **{k: up(v, dev) for k, v in kw.items()})
            res.append((x.cpu(), None if h is None else h.cpu().float()))
        torch.testing.assert_close(res[1][0], res[0][0], rtol=1e-5, atol=2e-5)
        if kw.get("write") is False:
            assert torch.equal(res[1][0], x0)
        if not quiet:
            torch.testing.assert_close(res[1][1], res[0][1], **(_tol(dt) if dt == torch.bfloat16
                                                                else dict(rtol=1e-5, atol=2e-5)))


def test_stream_norm_is_precise():
    """The dynamic tanh in fp32 over small, middling and saturated arguments."""
    n = 4096
    u = torch.cat([torch.linspace(-12, 12, n // 2), torch.logspace(-7, 0, n // 2)]).view(1, 1, n)
    dyt = (1.0, torch.ones(n), torch.zeros(n))
    h = torch.zeros(1, n, device=DEV)
    sm.stream_mix(u.to(DEV), dyt=(1.0, *_d(*dyt[1:])), h=h, write=False)
    ref = torch.tanh(u.double()).view(1, n)
    assert float(((h.cpu().double() - ref).abs() / ref.abs().clamp(min=1e-30)).max()) < 5e-7


PREP = [
    # heads, value heads, D, V, taps, rotated
    (6, 2, 24, 40, 4, 16), (4, 4, 16, 8, 3, 16), (8, 2, 128, 112, 4, 64), (3, 1, 7, 5, 2, 0), (2, 1, 70, 300, 4, 20),
    (2, 2, 12, 12, 1, 6)]


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,V,K,dims", PREP)
@pytest.mark.parametrize("step", sorted(STEPS))
def test_two_map_input_pass(dt, H, G, D, V, K, dims, step):
    g = torch.Generator().manual_seed(4)
    lens, starts = STEPS[step]
    ent, entt, row_ent, pos, R = _step(lens, starts)
    E, mp = len(lens), 4
    pages = (torch.randperm(E * mp, generator=g) + 1).to(torch.int32).view(E, mp)
    rows = torch.tensor([int(pages[e, p // PAGE]) * PAGE + p % PAGE for e, p in zip(row_ent.tolist(), pos.tolist())],
                        dtype=torch.int32)
    inv = sm.rope_inv_freq(500.0, dims, "cpu")
    for own in (True, False):
        C, W = (2 * H + (2 * G if own else 0)) * D + (G * V if own else 0), G * (2 * D + V)
        proj, cw = torch.randn(R, C + 6, generator=g).to(dt), torch.randn(C, K, generator=g)
        pool0, tail0 = torch.randn((E * mp + 1) * PAGE, W, generator=g).to(dt), torch.randn(E, K - 1, C, generator=g)
        res = []
        for dev in ("cpu", DEV):
            pool, tail, q = pool0.clone().to(dev), tail0.clone().to(dev), torch.empty(R, 2 * H * D, dtype=dt, device=dev)
            sm.conv_rope_norm_store(proj.to(dev), H, G, D, V, cw.to(dev), tail, inv.to(dev), None, pos.to(dev),
                                    rows.to(dev), pool if own else None, 1e-3, q, entt.to(dev), ent, row_ent.to(dev),
                                    pages.to(dev), PAGE, maps=2, norm=False, rm=1.2)
            res.append((q.cpu(), pool.cpu(), tail.cpu()))
        torch.testing.assert_close(res[1][0].float(), res[0][0].float(), **_tol(dt))
        torch.testing.assert_close(res[1][1].float(), res[0][1].float(), **_tol(dt))
        assert torch.equal(res[1][2], res[0][2]) and torch.equal(res[0][1], pool0) != own


ATTN = [
    # H, G, D, V
    (6, 2, 24, 40),      # three heads per key/value head
    (4, 4, 16, 8),       # one head per key/value head
    (16, 2, 128, 112),   # eight heads per key/value head
    (34, 2, 8, 16),      # more heads per key/value head than a wavefront's pairs
    (4, 2, 136, 200),    # wide heads
    (3, 1, 7, 5),        # sizes off the matrix cores' grid
]


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,V", ATTN)
@pytest.mark.parametrize("win,keep", [(20, 6), (1, 1), (64, 130), (7, 0), (33, 32), (500, 3)])
@pytest.mark.parametrize("two", [False, True])
def test_kept_tokens_and_two_maps(dt, H, G, D, V, win, keep, two):
    g = torch.Generator().manual_seed(5)
    lens, starts = [70, 9, 1, 1], [0, 150, 131, 0]
    ent, _entt, row_ent, pos, R = _step(lens, starts)
    M = 2 if two else 1
    bt = torch.tensor([[3, 5, 0], [7, 2, 9], [1, 4, 8], [6, 0, 0]], dtype=torch.int32)
    pool = torch.randn(12 * PAGE, G * (M * D + V), generator=g).to(dt)
    q = torch.randn(R, H * M * D, generator=g).to(dt)
    kw = dict(keep=keep, diff=(0.37, 1e-4) if two else None, out_scale=0.6)
    scale = 1.2 / D ** 0.5
    o1 = torch.empty(R, H * V, dtype=dt)
    sm.window_attn(q, pool, bt, row_ent, pos, None, scale, win, o1, PAGE, H, G, D, V, **kw)
    q2, pool2 = _d(q, pool)
    for mfma in ([False, True] if dt == torch.bfloat16 else [False]):
        for max_keys in (None, 160):    # whole key lists / lists cut into runs
            units = None
            if mfma:
                if not sm.window_mfma_ok(q2, pool2, D, V):
                    assert D % 8 or V % 8
                    continue
                units = sm.make_units(ent, sm.window_rows_per_wave(H // G)).to(DEV)
            o2 = torch.full((R, H * V + 8), 7.0, dtype=dt, device=DEV)
            sm.window_attn(q2, pool2, *_d(bt, row_ent, pos), None, scale, win, o2[:, :H * V], PAGE, H, G, D, V,
                           units=units, max_keys=max_keys, **kw)
            torch.testing.assert_close(o2[:, :H * V].cpu().float(), o1.float(), **_tol(dt))
            assert bool((o2[:, H * V:] == 7.0).all())
    # the kept tokens are at work wherever some row's window has left one behind
    o3 = torch.empty(R, H * V, dtype=dt)
    sm.window_attn(q, pool, bt, row_ent, pos, None, scale, win, o3, PAGE, H, G, D, V, **dict(kw, keep=0))
    assert ((o3.float() - o1.float()).abs().max() > 1e-3) == bool(keep > 0 and (pos - win + 1 > 0).any())


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
def test_rotation_magnitude(dt):
    g = torch.Generator().manual_seed(1)
    sc = {"factor": 6.0, "original": 300, "fast": 16.0, "slow": 1.0}
    rm, R = sm.rope_magnitude(sc), 19
    assert abs(rm - 1.1791759) < 1e-6 and sm.rope_magnitude(None) == 1.0
    inv = sm.rope_inv_freq(900.0, 12, "cpu", sc)
    pos = torch.randint(0, 2000, (R,), generator=g, dtype=torch.int32)
    src = torch.randn(R, 60, generator=g).to(dt)
    d1, d2 = torch.zeros(R, 60, dtype=dt), torch.zeros(R, 60, dtype=dt, device=DEV)
    sm.rope_rows(src, 3, 20, inv, pos, d1, 20, rm=rm)
    sm.rope_rows(src.to(DEV), 3, 20, inv.to(DEV), pos.to(DEV), d2, 20, rm=rm)
    torch.testing.assert_close(d2.cpu().float(), d1.float(), **_tol(dt))
    # latent and key part without a query latent
    rows = torch.randperm(40, generator=g)[:R].to(torch.int32)
    cw = torch.randn(40, generator=g)
    p1, p2 = torch.zeros(40, 54, dtype=dt), torch.zeros(40, 54, dtype=dt, device=DEV)
    proj = torch.randn(R, 60, generator=g).to(dt)
    sm.latent_prep(proj[:, 4:], 0, 40, 14, None, cw, inv, pos, rows, p1, 1e-5, None, rm=rm)
    sm.latent_prep(proj.to(DEV)[:, 4:], 0, 40, 14, None, *_d(cw, inv, pos, rows), p2, 1e-5, None, rm=rm)
    torch.testing.assert_close(p2.cpu().float(), p1.float(), **_tol(dt))
    # per-head norm, rotation, store
    H, G, D, V = 3, 1, 16, 8
    proj, qw, kw = torch.randn(R, 72, generator=g).to(dt), torch.randn(D, generator=g), torch.randn(D, generator=g)
    outs = []
    for dev in ("cpu", DEV):
        q, pool = torch.zeros(R, H * D, dtype=dt, device=dev), torch.zeros(40, G * (D + V), dtype=dt, device=dev)
        sm.qk_norm_rope_store(proj.to(dev), H, G, D, V, *(t.to(dev) for t in (qw, kw, inv, pos, rows)), pool, 1e-5, q,
                              per_head=True, half=True, rm=rm)
        outs.append((q.cpu().float(), pool.cpu().float()))
    for a, b in zip(*outs):
        torch.testing.assert_close(b, a, **_tol(dt))


GLA = [
    # H, D, V, rank, tau
    (2, 16, 16, 16, 16.0), (3, 48, 32, 16, 16.0), (2, 128, 128, 16, 8.0), (1, 7, 5, 3, 1.0), (2, 20, 100, 8, 4.0),
    (1, 128, 36, 1, 2.0), (4, 64, 64, 40, 0.5), (1, 160, 24, 16, 16.0), (2, 24, 200, 4, 3.0)]


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,D,V,rank,tau", GLA)
@pytest.mark.parametrize("step", sorted(STEPS))
def test_gla_scan(dt, H, D, V, rank, tau, step):
    g = torch.Generator().manual_seed(7)
    lens, starts = STEPS[step]
    ent, entt, _re, _pos, R = _step(lens, starts, slots=list(range(len(lens)))[::-1])
    low0 = 2 * H * D + 2 * H * V
    proj = torch.randn(R, low0 + rank + 1, generator=g).to(dt)
    wa2 = (torch.randn(H * D, rank, generator=g) / rank ** 0.5).to(dt)
    normw = 1 + 0.1 * torch.randn(V, generator=g)
    # decays near 1, mixed, and so strong that a quotient of running products would overflow
    for shift in (4.0, 0.0, -12.0):
        za = torch.randn(H * D, generator=g) * 2 + shift
        s0 = torch.randn(len(lens) + 1, H, D, V, generator=g)
        res = []
        for dev in ("cpu", DEV):
            st, o = s0.clone().to(dev), torch.full((R, H * V + 8), 7.0, dtype=dt, device=dev)
            sm.gla_scan(proj.to(dev), low0, rank, wa2.to(dev), za.to(dev), 1.0 / tau, normw.to(dev), st, entt.to(dev),
                        ent, o[:, :H * V], H, D, V, 1e-5, out_scale=0.5)
            res.append((o.cpu().float(), st.cpu()))
        (o1, s1), (o2, s2) = res
        if dt == torch.float32:
            torch.testing.assert_close(s2, s1, rtol=1e-4, atol=2e-5 * float(s1.abs().max()))
            torch.testing.assert_close(o2, o1, rtol=2e-3, atol=2e-4)
        else:      # the rounding of the decay logits shows in the states
            torch.testing.assert_close(s2, s1, rtol=2e-2, atol=5e-3 * float(s1.abs().max()))
            d = (o2 - o1).pow(2).mean().sqrt() / o1.pow(2).mean().sqrt()
            assert float(d) < 0.02


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("E,top,groups,keep", [(12, 2, 2, 1), (8, 3, 4, 2), (6, 1, 1, 1), (70, 5, 7, 3), (4, 4, 2, 2)])
def test_router_rescaled(dt, E, top, groups, keep):
    g = torch.Generator().manual_seed(9)
    R, W = 37, 72
    h, wr = torch.randn(R, W, generator=g).to(dt), torch.randn(E, W, generator=g) * 0.3
    for scale in (1.0, 2.5):
        res = []
        for dev in ("cpu", DEV):
            ids, wts = torch.zeros(R, top, dtype=torch.int32, device=dev), torch.zeros(R, top, device=dev)
            cnt, rows = torch.zeros(E, dtype=torch.int32, device=dev), torch.zeros(E, R * top, dtype=torch.int32, device=dev)
            sm.group_route(h.to(dev), wr.to(dev), top, groups, keep, ids, wts, cnt, rows, score="softmax",
                           group_score="max", renorm=True, scale=scale)
            res.append((ids.cpu(), wts.cpu(), cnt.cpu()))
        assert torch.equal(res[0][0], res[1][0]) and torch.equal(res[0][2], res[1][2])
        torch.testing.assert_close(res[1][1], res[0][1], rtol=1e-4, atol=1e-6)
        torch.testing.assert_close(res[1][1].sum(1), torch.full((R,), scale), rtol=1e-5, atol=1e-5)
