"""HIP kernels behind the Rasepel mixers against the PyTorch rendering of the same ops (CPU
tensors), in fp32 and bf16: the residual pass that hands on the rows themselves, the gated norm of a
whole row, short convolutions with their tails, the selective scan (portions, chunks, the fused
single-token step), lightning attention (matrix-instruction chunks and the walking kernel), the
convolved attention input pass with its blocks, and attention over blocks and tokens with a gate
per channel."""
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
         "long": ([150, 1, 64, 129, 2], [0, 9, 0, 33, 2]), "one_long": ([200], [0])}


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [200, 1500, 4200])
def test_post_norm_pass_and_norm_gate(dt, n):
    g = torch.Generator().manual_seed(0)
    R = 21
    x, y = torch.randn(R, n, generator=g), torch.randn(R, n + 3, generator=g).to(dt)[:, 3:]
    w = 1 + 0.1 * torch.randn(n, generator=g)
    h1, h2 = torch.zeros(R, n, dtype=dt), torch.zeros(R, n, dtype=dt, device=DEV)
    x1 = sm.norm_scale_add(x.clone(), y, w, None, 1e-5, next_out=h1)
    x2 = sm.norm_scale_add(x.to(DEV), y.to(DEV), w.to(DEV), None, 1e-5, next_out=h2)
    torch.testing.assert_close(x2.cpu(), x1, rtol=1e-5, atol=1e-5)
    assert torch.equal(h2.cpu(), x2.cpu().to(dt)) and torch.equal(h1, x1.to(dt))
    x3 = sm.norm_scale_add(x.to(DEV), y.to(DEV), w.to(DEV), None, 1e-5)
    assert torch.equal(x3, x2)
    gate = torch.randn(R, n + 8, generator=g).to(dt)[:, 8:]
    a = sm.norm_gate(x, w, gate, 1e-5, torch.empty(R, n, dtype=dt))
    b = sm.norm_gate(x.to(DEV), w.to(DEV), gate.to(DEV), 1e-5, torch.empty(R, n, dtype=dt, device=DEV))
    torch.testing.assert_close(b.cpu().float(), a.float(), **_tol(dt))


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("K", [1, 2, 3, 4, 7])
@pytest.mark.parametrize("step", sorted(STEPS))
def test_short_convolution(dt, K, step):
    g = torch.Generator().manual_seed(1)
    lens, starts = STEPS[step]
    ent, entt, row_ent, _pos, R = _step(lens, starts)
    C = 70
    zx = torch.randn(R, C + 9, generator=g).to(dt)
    cw, cb = torch.randn(C, K, generator=g), torch.randn(C, generator=g)
    tail0 = torch.randn(len(lens), K - 1, C, generator=g)
    for roll in (True, False):
        for odt in {dt, torch.float32}:
            t1, t2 = tail0.clone(), tail0.to(DEV)
            o1, o2 = torch.empty(R, C, dtype=odt), torch.empty(R, C, dtype=odt, device=DEV)
            sm.mamba_conv(zx, 5, cw, cb, t1, entt, ent, row_ent, o1, roll=roll)
            sm.mamba_conv(zx.to(DEV), 5, cw.to(DEV), cb.to(DEV), t2, entt.to(DEV), ent, row_ent.to(DEV), o2, roll=roll)
            torch.testing.assert_close(o2.cpu().float(), o1.float(), **_tol(odt))
            assert torch.equal(t2.cpu(), t1) and (torch.equal(t1, tail0) == (not roll or K == 1))


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("I,N,rank", [(70, 16, 6), (256, 24, 12), (65, 3, 1), (40, 70, 9), (130, 130, 33), (64, 8, 40)])
@pytest.mark.parametrize("step", sorted(STEPS))
def test_selective_scan(dt, I, N, rank, step):
    g = torch.Generator().manual_seed(2)
    lens, starts = STEPS[step]
    ent, entt, _re, _pos, R = _step(lens, starts, slots=list(range(len(lens)))[::-1])
    x = (torch.randn(R, I, generator=g)).to(dt)
    xp = (torch.randn(R, rank + 2 * N, generator=g) * 0.7).to(dt)
    wdt = (torch.randn(rank, I, generator=g) / rank ** 0.5).to(dt)
    z = torch.randn(R, I + 3, generator=g).to(dt)[:, 3:]
    bias, Dp = torch.randn(I, generator=g) * 2 - 2, torch.randn(I, generator=g)
    A2 = -torch.exp(torch.rand(N, I, generator=g) * 4 - 2) * sm.LOG2E
    s0 = torch.randn(len(lens) + 1, N, I, generator=g)
    s1, s2 = s0.clone(), s0.to(DEV)
    y1, y2 = torch.empty(R, I, dtype=dt), torch.empty(R, I, dtype=dt, device=DEV)
    sm.selective_scan(x, xp, rank, wdt, bias, A2, Dp, z, s1, entt, ent, y1)
    sm.selective_scan(*_d(x, xp), rank, *_d(wdt, bias, A2, Dp, z), s2, entt.to(DEV), ent, y2)
    # the projected step sizes are rounded in bf16 portions; everything after is fp32
    tol = dict(rtol=5e-4, atol=5e-4) if dt == torch.float32 else dict(rtol=5e-2, atol=8e-2 * max(1.0, float(y1.float().abs().mean())))
    torch.testing.assert_close(y2.cpu().float(), y1.float(), **tol)
    torch.testing.assert_close(s2.cpu(), s1, **tol)


@pytest.mark.parametrize("step", ["decode", "long"])
def test_selective_scan_step_sizes(step):
    """Step sizes from 1e-8 to 30 keep their relative accuracy (D = 0, a fresh state, one token: y is
    dt x B C silu(z))."""
    I, N = 64, 4
    lens, starts = ([1, 1], [0, 0]) if step == "decode" else ([2, 130], [0, 0])
    ent, entt, _re, _pos, R = _step(lens, starts)
    bias = torch.linspace(-18.0, 30.0, I)
    one = torch.ones(R, I)
    xp = torch.cat([torch.zeros(R, 1), torch.ones(R, 2 * N)], 1)
    A2 = torch.full((N, I), -0.1)
    y = torch.empty(R, I, device=DEV)
    sm.selective_scan(*_d(one, xp), 1, *_d(torch.zeros(1, I), bias, A2, torch.zeros(I), one),
                      torch.zeros(3, N, I, device=DEV), entt.to(DEV), ent, y)
    want = torch.nn.functional.softplus(bias.double(), threshold=1e9) * N / (1 + torch.exp(torch.tensor(-1.0)).double())
    for row0, _n, _s, _sl in ent:
        torch.testing.assert_close(y[row0].cpu().double(), want, rtol=2e-6, atol=0)


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,D,V", [(3, 32, 48), (2, 128, 128), (1, 7, 5), (2, 20, 136), (1, 256, 256), (4, 16, 16), (2, 200, 30)])
@pytest.mark.parametrize("step", sorted(STEPS))
def test_lightning_scan(dt, H, D, V, step):
    g = torch.Generator().manual_seed(3)
    lens, starts = STEPS[step]
    ent, entt, _re, _pos, R = _step(lens, starts, slots=list(range(len(lens)))[::-1])
    proj = torch.randn(R, 2 * H * D + 2 * H * V + 4, generator=g).to(dt)
    for decay in ([0.5, 0.9, 0.99, 0.999][:H], [1.0, 0.0, 0.999, 0.3][:H]):
        pw = sm.decay_powers(decay, "cpu")
        assert float(pw[0, 0]) == 1.0 and pw.shape == (H, 65)
        s0 = torch.randn(len(lens) + 1, H, D, V, generator=g)
        s1, s2 = s0.clone(), s0.to(DEV)
        o1, o2 = torch.empty(R, H * V), torch.empty(R, H * V, device=DEV)
        sm.lightning_scan(proj, pw, s1, entt, ent, o1, H, D, V)
        sm.lightning_scan(proj.to(DEV), pw.to(DEV), s2, entt.to(DEV), ent, o2, H, D, V)
        # fp32 sums in another order, in both formats
        torch.testing.assert_close(o2.cpu(), o1, rtol=1e-4, atol=2e-5 * float(o1.abs().max()))
        torch.testing.assert_close(s2.cpu(), s1, rtol=1e-4, atol=2e-5 * float(s1.abs().max()))


PREP = [
    # H, G, D, V, taps, rotated, block
    (6, 2, 24, 40, 4, 16, 7),
    (4, 4, 16, 8, 3, 16, 64),
    (16, 2, 128, 112, 4, 64, 16),
    (3, 1, 7, 5, 2, 0, 3),
    (2, 1, 70, 300, 4, 20, 1),       # a value size beyond the rows kernel
    (5, 5, 130, 66, 3, 128, 100),    # blocks longer than a page
    (2, 2, 12, 12, 1, 6, None),
]


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,V,K,dims,P", PREP)
@pytest.mark.parametrize("step", sorted(STEPS))
def test_conv_rope_norm_store(dt, H, G, D, V, K, dims, P, step):
    g = torch.Generator().manual_seed(4)
    lens, starts = STEPS[step]
    ent, entt, row_ent, pos, R = _step(lens, starts)
    E, mp = len(lens), 4
    pages = (torch.randperm(E * mp, generator=g) + 1).to(torch.int32).view(E, mp)
    rows = torch.tensor([int(pages[e, p // PAGE]) * PAGE + p % PAGE for e, p in zip(row_ent.tolist(), pos.tolist())],
                        dtype=torch.int32)
    C, W = (H + G) * D + G * V, G * (D + V)
    proj = torch.randn(R, C + 6, generator=g).to(dt)
    cw = torch.randn(C, K, generator=g)
    temp = torch.randn(H, generator=g)
    inv = sm.rope_inv_freq(500.0, dims, "cpu")
    pool0 = torch.randn((E * mp + 1) * PAGE, W, generator=g).to(dt)
    blk0 = torch.zeros((E * mp + 1) * sm.blocks_per_page(PAGE, P), W, dtype=dt) if P else None
    tail0 = torch.randn(E, K - 1, C, generator=g)
    res = []
    for dev in ("cpu", DEV):
        pool, tail, q = pool0.clone().to(dev), tail0.clone().to(dev), torch.empty(R, H * D, dtype=dt, device=dev)
        blk = blk0.clone().to(dev) if P else None
        args = [t.to(dev) for t in (cw, tail, inv, temp, pos, rows)]
        args[1] = tail
        sm.conv_rope_norm_store(proj.to(dev), H, G, D, V, *args, pool, 1e-3, q, entt.to(dev), ent, row_ent.to(dev),
                                pages.to(dev), PAGE, blk=blk, every=P or 0)
        res.append((q, pool, tail, blk))
    (q1, p1, t1, b1), (q2, p2, t2, b2) = res
    torch.testing.assert_close(q2.cpu().float(), q1.float(), **_tol(dt))
    torch.testing.assert_close(p2.cpu().float(), p1.float(), **_tol(dt))
    assert torch.equal(t2.cpu(), t1)
    if P:
        torch.testing.assert_close(b2.cpu().float(), b1.float(), **_tol(dt))
        done = sum((s + n) // P - s // P for n, s in zip(lens, starts))
        assert int((b1.float().abs().sum(1) > 0).sum()) == done


ATTN = [
    # H, G, D, V
    (6, 2, 24, 40),      # three heads per key/value head
    (4, 4, 16, 8),       # one head per key/value head
    (16, 2, 128, 112),   # eight heads per key/value head
    (34, 2, 8, 16),      # more heads per key/value head than a wavefront's pairs
    (3, 1, 7, 5),        # sizes off the matrix cores' grid
]


@pytest.mark.parametrize("dt", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,V", ATTN)
@pytest.mark.parametrize("win,P", [(20, 6), (1, 1), (64, 16), (7, 70), (150, 3), (500, 8)])
def test_attention_over_blocks(dt, H, G, D, V, win, P):
    g = torch.Generator().manual_seed(5)
    lens, starts = [70, 9, 1, 1], [0, 150, 131, 0]
    ent, _entt, row_ent, pos, R = _step(lens, starts)
    bt = torch.tensor([[3, 5, 0], [7, 2, 9], [1, 4, 8], [6, 0, 0]], dtype=torch.int32)
    pool = torch.randn(12 * PAGE, G * (D + V), generator=g).to(dt)
    blk = torch.randn(12 * sm.blocks_per_page(PAGE, P), G * (D + V), generator=g).to(dt)
    q = torch.randn(R, H * D, generator=g).to(dt)
    gate = torch.randn(R, H * V + 5, generator=g).to(dt)[:, 5:]
    kw = dict(gate_channels=True, every=P)
    o1 = torch.empty(R, H * V, dtype=dt)
    sm.window_attn(q, pool, bt, row_ent, pos, None, 0.4, win, o1, PAGE, H, G, D, V, gate=gate, blk=blk, **kw)
    q2, pool2, blk2, gate2 = _d(q, pool, blk, gate)
    for mfma in ([False, True] if dt == torch.bfloat16 else [False]):
        for max_keys in (None, 160):    # whole key lists / lists cut into runs
            units = None
            if mfma:
                if not sm.window_mfma_ok(q2, pool2, D, V):
                    assert D % 8 or V % 8
                    continue
                units = sm.make_units(ent, sm.window_rows_per_wave(H // G)).to(DEV)
            o2 = torch.empty(R, H * V, dtype=dt, device=DEV)
            sm.window_attn(q2, pool2, *_d(bt, row_ent, pos), None, 0.4, win, o2, PAGE, H, G, D, V, units=units,
                           max_keys=max_keys, gate=gate2, blk=blk2, **kw)
            torch.testing.assert_close(o2.cpu().float(), o1.float(), **_tol(dt))
    # the blocks are at work wherever some row sees one
    o3 = torch.empty(R, H * V, dtype=dt)
    sm.window_attn(q, pool, bt, row_ent, pos, None, 0.4, win, o3, PAGE, H, G, D, V, gate=gate, gate_channels=True)
    sees = bool(((pos - win + 1).clamp(min=0) // P > 0).any())
    assert ((o3.float() - o1.float()).abs().max() > 1e-3) == sees
