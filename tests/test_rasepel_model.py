"""The Rasepel hybrid model on the engine against the plain oracle (tests/rasepel_oracle.py).

Every test builds its own small configuration and random checkpoint, runs the oracle once
over whole sequences in float64, and drives the engine's step function / generate / server
in float32 (and bfloat16 with a loose bound).  The CPU variants exercise the model, cache,
batching and scheduling code with the ops' PyTorch rendering; the ``gpu`` variants run the
same cases on the HIP kernels.
"""
import copy
import math

import pytest
import torch

import rasepel_oracle as O
from p2p_llm_chat_go_amd.engine.hybrid import HybridEngine
from p2p_llm_chat_go_amd.models import hybrid as Hy
from p2p_llm_chat_go_amd.ops import PAGE

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]

FF = {"kind": "dense", "ff": 56, "limit": 1.2}
MB = {"type": "mamba1", "mixer": {"inner": 40, "state": 10, "dt_rank": 6, "conv": 3}, "mlp": None}
LG = {"type": "lightning", "mixer": {"heads": 3, "dim": 20, "vdim": 12, "decay": [0.6, 0.93, 0.995]}, "mlp": None}
AT = {"type": "attention",
      "mixer": {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 24, "conv": 3, "scale": 0.7,
                "mask": {"size": 21, "pool": 5}, "rot": {"base": 400.0, "dims": 8}},
      "mlp": None}


def layer(base, mlp=None, **mixer):
    L = copy.deepcopy(base)
    L["mlp"] = copy.deepcopy(mlp)
    L["mixer"].update(copy.deepcopy(mixer))
    return L


def window(size, pool):
    return {"mask": {"size": size, "pool": pool}}


def make(layers, width=48, vocab=83, seed=0, eps=1e-5, scale=1.7):
    c = {"architecture": "Rasepel", "width": width, "vocab": vocab, "norm": {"eps": eps},
         "embedding": {"scale": scale}, "layers": copy.deepcopy(layers)}
    cfg = Hy.HybridConfig.from_dict(c)
    return c, cfg, Hy.random_state_dict(cfg, seed)


def engine(cfg, sd, dev, dtype=torch.float32, pages=24, slots=4, **kw):
    return HybridEngine(cfg, Hy.HybridWeights(cfg, sd, dev, dtype), dev, kv_pages=pages,
                        num_slots=slots, max_batch=slots, **kw)


def toks(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def close(got, ref, tol=2e-4):
    """Difference of logits rows, mean removed, RMS over the vocabulary, relative to the RMS of
    the reference logits."""
    got, ref = got.detach().cpu().double(), ref.double()
    d = got - ref
    d = d - d.mean(-1, keepdim=True)
    scale = (ref - ref.mean(-1, keepdim=True)).pow(2).mean().sqrt()
    err = d.pow(2).mean(-1).sqrt() / scale
    worst = int(err.argmax())
    assert float(err[worst]) < tol, "row %d of %d: relative logits error %.3g" % (worst, len(err), err[worst])


def run_whole(eng, key, t):
    out = eng.step([(key, t, list(range(len(t))))])
    eng.release(key)
    return out


def run_cuts(eng, key, t, cuts):
    at, outs = 0, []
    for n in cuts:
        n = min(n, len(t) - at)
        if n <= 0:
            break
        outs.append(eng.step([(key, t[at:at + n], list(range(n)))]))
        at += n
    if at < len(t):
        outs.append(eng.step([(key, t[at:], list(range(len(t) - at)))]))
    eng.release(key)
    return torch.cat(outs)


# ------------------------------------------------------------------ the oracle's own pieces
def test_oracle_pieces():
    """The oracle's building blocks on cases that can be worked out by hand."""
    f = lambda *x: torch.tensor(x, dtype=torch.float64)
    # convolution: the last tap meets the current token, nothing before the start
    u = f([1.0], [2.0], [4.0])
    torch.testing.assert_close(O.short_conv(u, f([10.0, 1.0])), f([1.0], [12.0], [24.0]))
    # visibility: size 3, blocks of 2 -> position 5 sees tokens 3..5 and block 0 (tokens 0, 1: ends at
    # 1 <= 5 - 3); token 2 is seen by nobody until block 1 (2, 3) has left the window of position 6
    assert O.visible(5, 3, 2) == ([3, 4, 5], [0])
    assert O.visible(4, 3, 2) == ([2, 3, 4], [0])
    assert O.visible(3, 3, 2) == ([1, 2, 3], [])
    assert O.visible(6, 3, 2) == ([4, 5, 6], [0, 1])
    # decayed memory with one channel: a geometric sum
    q = torch.ones(3, 1, 1, dtype=torch.float64)
    torch.testing.assert_close(O.decayed_memory(q, q, q, [0.5]).reshape(-1), f(1.0, 1.5, 1.75))
    # selective scan, one channel and state, dt = 1, A = -ln 2: the state halves
    one = torch.ones(3, 1, dtype=torch.float64)
    y = O.selective_scan(one, one, f([-math.log(2.0)]), one, one, f(10.0))
    torch.testing.assert_close(y.reshape(-1), f(11.0, 11.5, 11.75))
    # rotation: base 1 -> angle = position; channel 0 pairs with channel 2, channel 4 passes
    x = torch.zeros(3, 1, 5, dtype=torch.float64)
    x[:, 0, 0], x[:, 0, 4] = 1.0, 7.0
    z = O.rotate_halves(x, 4, 1.0)
    torch.testing.assert_close(z[2, 0, [0, 2]], f(math.cos(2.0), math.sin(2.0)))
    assert float(z[2, 0, 4]) == 7.0 and float(z[2, 0, 1]) == 0.0
    # clamped unit: both sides of the gate's limit, the up part's two limits
    eye = torch.eye(1, dtype=torch.float64)
    t = {"gate": eye, "up": eye, "down": eye}
    for v in (-5.0, 0.5, 5.0):
        g, up = min(v, 2.0), max(-2.0, min(v, 2.0))
        torch.testing.assert_close(O.clamped_unit(f([v]), t, "", 2.0)[0, 0],
                                   f(g / (1 + math.exp(-1.702 * g)) * (up + 1))[0])


# ------------------------------------------------------------------ each mechanism alone
ALONE = {
    "mamba1": [MB],
    "lightning": [LG],
    "attention": [AT],
    "attention_no_blocks": [layer(AT, None, mask={"size": 9})],
    "attention_unrotated": [layer(AT, None, rot=None)],
    "dense_ff": [layer(LG, FF)],
}


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", sorted(ALONE))
def test_single_mechanism(dev, name):
    c, cfg, sd = make(ALONE[name], seed=3)
    t = toks(90, cfg.vocab, 1)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev)
    close(run_whole(eng, "a", t), ref)
    close(run_cuts(eng, "b", t, [30, 1, 2, 1, 40]), ref)


@pytest.mark.parametrize("dev", DEVICES)
def test_layers_match_oracle(dev):
    c, cfg, sd = make([layer(MB, FF), layer(AT, FF), LG, layer(AT, None), layer(LG, FF)], seed=4)
    t = toks(40, cfg.vocab, 2)
    lay = []
    ref = O.forward(c, sd, t, layers_out=lay)
    eng = engine(cfg, sd, dev)
    got = []
    out = eng.step([("a", t, list(range(len(t))))], return_layers=got)
    assert len(got) == len(lay) == 5
    for i, x in enumerate(got):
        torch.testing.assert_close(x.cpu().double(), lay[i], rtol=1e-4, atol=2e-4, msg="layer %d" % i)
    close(out, ref)


@pytest.mark.parametrize("dev", DEVICES)
def test_post_norm_reads_residual(dev):
    """The norm sits on what a sublayer produces: weights near -1 silence a sublayer, and the next
    one still reads the residual itself, whatever its size."""
    c, cfg, sd = make([layer(LG, FF), layer(MB, FF)], seed=30, scale=6.0)
    for k in ("l0.norm1", "l0.norm2"):
        sd[k] = torch.full_like(sd[k], -1.0)
    t = toks(50, cfg.vocab, 31)
    lay = []
    ref = O.forward(c, sd, t, layers_out=lay)
    torch.testing.assert_close(lay[0], sd["embed"].double()[torch.tensor(t)] * 6.0)
    close(run_cuts(engine(cfg, sd, dev), "a", t, [20, 1, 1]), ref)


# ------------------------------------------------------------------ other sizes
VARIANTS = {
    # one head, one tap, one state, rank one, blocks of one token, a window of one token
    "ones": ([layer(MB, {"kind": "dense", "ff": 8, "limit": 0.5}, inner=8, state=1, dt_rank=1, conv=1),
              layer(AT, None, heads=1, kv_heads=1, dim=8, vdim=8, conv=1, mask={"size": 1, "pool": 1},
                    rot={"base": 10.0, "dims": 2}),
              layer(LG, None, heads=1, dim=8, vdim=8, decay=[0.5])], 40),
    # sizes that are not multiples of 8, as many kv heads as heads, every channel rotated, 5 taps, blocks as
    # long as the window, decays 0 and 1
    "odd": ([layer(AT, {"kind": "dense", "ff": 50, "limit": 3.0}, heads=5, kv_heads=5, dim=6, vdim=10, conv=5,
                   scale=1.3, mask={"size": 7, "pool": 7}, rot={"base": 40000.0, "dims": 6}),
             layer(MB, FF, inner=37, state=7, dt_rank=5, conv=2),
             layer(LG, None, heads=2, dim=9, vdim=11, decay=[0.0, 1.0]),
             layer(MB, None, inner=33, state=13, dt_rank=3, conv=6)], 36),
    # wide heads and states, blocks longer than a page and than the window, four taps
    "wide": ([layer(AT, None, heads=6, kv_heads=1, dim=72, vdim=40, conv=4, mask={"size": 10, "pool": 70},
                    rot={"base": 1000.0, "dims": 40}),
              layer(MB, FF, inner=130, state=40, dt_rank=20, conv=4),
              layer(LG, None, heads=2, dim=136, vdim=72, decay=[0.8, 0.99]),
              layer(MB, None, inner=64, state=130, dt_rank=40, conv=4)], 100),
}


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("name", sorted(VARIANTS))
def test_other_sizes(dev, name):
    layers, width = VARIANTS[name]
    c, cfg, sd = make(layers, width=width, vocab=61, seed=5, eps=1e-3, scale=1.0 if name == "ones" else 0.4)
    t = toks(150, cfg.vocab, 3)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev)
    # first part as a prompt, the rest in portions of 1, 2 and 5 tokens
    close(run_cuts(eng, "a", t, [70, 1, 2, 5, 1, 1, 2, 40, 1, 2, 1, 1]), ref)
    close(run_whole(eng, "b", t), ref)


# ------------------------------------------------------------------ prefill vs decode, portions
@pytest.mark.parametrize("dev", DEVICES)
def test_prefill_decode_and_portions(dev):
    c, cfg, sd = make([layer(MB, FF), layer(AT, FF), layer(LG, None), layer(AT, None, **window(33, 12))], seed=6)
    n = 2 * PAGE + 21                      # crosses two page borders
    t = toks(n, cfg.vocab, 4)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev)
    close(run_whole(eng, "w", t), ref)
    # token by token from the first token on: the first tokens stand on zeros before the start
    close(run_cuts(eng, "d", t, [1] * n), ref)
    # portions of changing size, down to two tokens and one, cut inside pages, windows, blocks
    for sizes in ([2] * 20 + [63, 1, 1, 2, 40, 3], [5, 59, 1, 64, 7, 2, 3, 8], [129, 2, 1, 17], [1, 2, 1, 3, 70, 31, 32, 1]):
        close(run_cuts(eng, "p", t, sizes), ref)


@pytest.mark.parametrize("dev", DEVICES)
def test_long_sequence_chunks(dev):
    """A prompt of several chunks of every scan, continued by portions on both sides of the length
    from which the scans run in chunks, then decoded."""
    c, cfg, sd = make([layer(MB, None, conv=4), layer(LG, FF), layer(AT, None, conv=4, **window(50, 9))], seed=9)
    n = 5 * PAGE + 30
    t = toks(n, cfg.vocab, 14)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev)
    close(run_whole(eng, "w", t), ref)
    close(run_cuts(eng, "p", t, [129, 31, 32, 33, 65, 1, 1, 2, 3]), ref)


@pytest.mark.parametrize("dev", DEVICES)
def test_long_decoding(dev):
    """Many single tokens: states, tails and blocks written by decode steps only."""
    c, cfg, sd = make([layer(AT, None, **window(13, 4)), MB, LG, layer(AT, FF, conv=4, **window(40, 16))], seed=10)
    n = 3 * PAGE + 5
    t = toks(n, cfg.vocab, 15)
    ref = O.forward(c, sd, t)
    close(run_cuts(engine(cfg, sd, dev), "d", t, [2] + [1] * n), ref)


# ------------------------------------------------------------------ batches, reuse of pages and slots
@pytest.mark.parametrize("dev", DEVICES)
def test_mixed_batches_and_reuse(dev):
    c, cfg, sd = make([layer(AT, FF), MB, layer(LG, None), layer(AT, None, conv=4, **window(30, 8)), layer(MB, FF)],
                      seed=7)
    lens = [150, 9, 70, 1, 33, 130, 64, 65]
    reqs = {i: toks(n, cfg.vocab, 10 + i) for i, n in enumerate(lens)}
    refs = {i: O.forward(c, sd, t) for i, t in reqs.items()}
    # a pool that holds three of the long requests at most: pages and slots must come back
    eng = engine(cfg, sd, dev, pages=8, slots=3)
    got = {i: [] for i in reqs}
    at = {i: 0 for i in reqs}
    waiting, live, step = sorted(reqs), [], 0
    sizes = [7, 1, 30, 2, 1, 64, 3, 1, 1, 19]
    while waiting or live:
        while waiting and len(live) < 3:
            need = sum(-(-len(reqs[i]) // PAGE) for i in live) + -(-len(reqs[waiting[0]]) // PAGE)
            if need > 7:
                break
            live.append(waiting.pop(0))
        entries = []
        for j, i in enumerate(live):
            if (step + j) % 4 == 3 and len(live) > 1:
                continue                      # a request may sit a step out
            n = min(sizes[(step + 3 * j) % len(sizes)], len(reqs[i]) - at[i])
            entries.append((i, reqs[i][at[i]:at[i] + n], list(range(n))))
            at[i] += n
        out = eng.step(entries)
        o = 0
        for i, tk, w in entries:
            got[i].append(out[o:o + len(w)])
            o += len(w)
        for i in [i for i in live if at[i] == len(reqs[i])]:
            eng.release(i)
            live.remove(i)
        step += 1
    assert eng.cache.live == 0 and eng.cache.allocator.free_pages == 7 and eng.cache.slots.free_slots == 3
    for i in reqs:
        close(torch.cat(got[i]), refs[i])


@pytest.mark.parametrize("dev", DEVICES)
def test_big_batch_beside_decode(dev):
    """Portions long enough for the row-grouped and chunked kernels beside single tokens and a
    two-token portion, starting and continuing, in one step."""
    c, cfg, sd = make([layer(AT, FF, conv=4, **window(18, 6)), layer(MB, None, conv=4), layer(LG, FF)], seed=17)
    ts = {k: toks(n, cfg.vocab, 200 + i) for i, (k, n) in enumerate((("a", 200), ("b", 37), ("c", 90), ("d", 150)))}
    refs = {k: O.forward(c, sd, t) for k, t in ts.items()}
    eng = engine(cfg, sd, dev)
    at = dict.fromkeys(ts, 0)
    got = {k: [] for k in ts}
    for step in ({"a": 70, "b": 35}, {"b": 1, "a": 60, "c": 17, "d": 1}, {"d": 100, "c": 2, "b": 1, "a": 1},
                 {"a": 69, "c": 71, "d": 49}):
        ent = [(k, ts[k][at[k]:at[k] + n], list(range(n))) for k, n in step.items()]
        out, o = eng.step(ent), 0
        for k, n in step.items():
            got[k].append(out[o:o + n])
            o, at[k] = o + n, at[k] + n
    for k in ts:
        close(torch.cat(got[k]), refs[k])


@pytest.mark.parametrize("dev", DEVICES)
def test_first_tokens_in_used_pages_and_slots(dev):
    """A sequence that starts in the pages and the slot another one left behind sees none of it:
    no keys, blocks, convolution inputs or states from before position 0."""
    c, cfg, sd = make([layer(AT, None, **window(4, 2)), MB, LG], seed=8)
    eng = engine(cfg, sd, dev, pages=3, slots=1)
    b = toks(11, cfg.vocab, 21)
    ref = O.forward(c, sd, b)
    for cuts in ([1, 2, 1, 1, 2, 1, 3], [11], [2, 9], [1] * 11):
        eng.step([("a", toks(100, cfg.vocab, 20), [])])
        eng.release("a")
        close(run_cuts(eng, "b", b, cuts), ref)


# ------------------------------------------------------------------ far keys, windows, blocks
FILL = list(range(20, 28))   # the tokens around the hot one


def spike(hot, qtok, mask, beta=40.0, seed=11, conv=1, rot=None):
    """Attention alone whose query projection is rebuilt so that every query of token ``qtok`` points
    along the part of token ``hot``'s key that is orthogonal to the keys of the tokens ``FILL``, and
    whose scale makes that score stand out: among those tokens (score 0) ``hot``, or a block that
    holds it, takes nearly all the softmax weight where it is visible.  The convolution keeps the
    current token only."""
    mx = {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 8, "conv": conv, "scale": 1.0, "mask": mask, "rot": rot}
    c, cfg, sd = make([{"type": "attention", "mixer": mx, "mlp": None}], width=32, vocab=50, seed=seed)
    H, G, D = mx["heads"], mx["kv_heads"], mx["dim"]
    for b in ("q", "k", "v"):
        sd["l0.mix.%s.b" % b] = torch.zeros_like(sd["l0.mix.%s.b" % b])
        w = torch.zeros_like(sd["l0.mix.%s.conv" % b])
        w[:, -1] = 1.0
        sd["l0.mix.%s.conv" % b] = w
    sd["l0.mix.temp"] = torch.tensor([1.0, 1.5, 0.75, 1.25]).to(torch.bfloat16)
    u = sd["embed"].double() * c["embedding"]["scale"]
    keys = (u @ sd["l0.mix.k"].double().T).view(-1, G, D)
    k = torch.stack([keys[hot, g] - (b := torch.linalg.qr(keys[FILL, g].T)[0]) @ (b.T @ keys[hot, g])
                     for g in range(G)])
    target = k.repeat_interleave(H // G, 0).reshape(-1)                  # [H * D]
    sd["l0.mix.q"] = (target[:, None] * u[qtok][None, :] / (u[qtok] @ u[qtok])).to(torch.bfloat16)
    c["layers"][0]["mixer"]["scale"] = beta / D                          # unit-RMS heads: q . k = D at best
    return c, Hy.HybridConfig.from_dict(c), sd


def spiked_tokens(vocab, n, hot, qtok, where, at, seed):
    t = [FILL[x % len(FILL)] for x in toks(n, vocab, seed)]
    t[at] = qtok
    if where is not None:
        t[where] = hot
    return t


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("size,pool", [(16, 4), (PAGE, 12), (7, 7), (33, 1), (5, 70)])
def test_window_and_block_edges(dev, size, pool):
    """A key that stands out just inside and just outside the window, in the newest visible block and
    in the one after it (which nobody sees), at a block's first and last token, in prompts, portions
    of two and decoding.  The oracle tells which of them show."""
    hot, qtok = 7, 11
    c, cfg, sd = spike(hot, qtok, {"size": size, "pool": pool}, beta=40.0 * min(pool, 12))
    n = 2 * PAGE + 19
    at = n - 3                               # the query's place
    nb = max(0, at - size + 1) // pool       # blocks it sees
    places = {"self_edge": at - 1, "inside": at - size + 1, "outside": at - size, "block_end": nb * pool - 1,
              "block_start": (nb - 1) * pool, "after_blocks": nb * pool, "first": 0, "page": PAGE, "page_end": PAGE - 1}
    base = O.forward(c, sd, spiked_tokens(cfg.vocab, n, hot, qtok, None, at, 5))
    shows = {}
    eng = engine(cfg, sd, dev)
    for name, w in sorted(places.items()):
        if not 0 <= w < at:
            continue
        t = spiked_tokens(cfg.vocab, n, hot, qtok, w, at, 5)
        ref = O.forward(c, sd, t)
        shows[name] = float((ref[at] - base[at]).abs().max())
        close(run_whole(eng, "w", t), ref)
        close(run_cuts(eng, "d", t, [at - 2] + [1] * 6), ref)
        close(run_cuts(eng, "e", t, [max(1, w), 1] + [2] * n), ref)
    assert shows["inside"] > 0.05
    if nb * pool < at - size + 1:            # tokens between the blocks and the window
        assert shows["outside"] < 1e-9 and shows["after_blocks"] < 1e-9
    elif size > 1:
        assert shows["outside"] > 1e-4       # it ends a block
    if nb and pool <= 12:
        assert shows["block_end"] > 1e-4 and shows["block_start"] > 1e-4


@pytest.mark.parametrize("dev", DEVICES)
@pytest.mark.parametrize("n,where", [(3 * PAGE + 9, 0), (3 * PAGE + 9, PAGE - 1), (3 * PAGE + 9, PAGE),
                                     (2 * PAGE + 1, 2 * PAGE - 1), (2 * PAGE + 1, 2 * PAGE)])
def test_far_keys_and_page_borders(dev, n, where):
    """One key among hundreds, far back inside a long window, on both sides of page borders."""
    hot, qtok = 7, 11
    c, cfg, sd = spike(hot, qtok, {"size": 4 * PAGE, "pool": 16})
    t = spiked_tokens(cfg.vocab, n, hot, qtok, where if where < n - 1 else None, n - 1, n + where)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev)
    close(run_whole(eng, "w", t), ref)
    close(run_cuts(eng, "d", t, [n - 5] + [1] * 5), ref)
    close(run_cuts(eng, "e", t, [max(1, where), 1] + [2] * n), ref)


@pytest.mark.parametrize("dev", DEVICES)
def test_blocks_across_cuts(dev):
    """Blocks whose tokens come in different steps and lie on two pages; blocks completed by the first,
    an inner or the last token of a portion, or by a decoded token."""
    hot, qtok = 7, 11
    c, cfg, sd = spike(hot, qtok, {"size": 6, "pool": 9}, beta=360.0)
    n = 2 * PAGE + 10
    eng = engine(cfg, sd, dev)
    for where in (PAGE - 1, PAGE, PAGE + 5, 2 * PAGE - 2, 8, 9):
        t = spiked_tokens(cfg.vocab, n, hot, qtok, where, n - 2, 77)
        ref = O.forward(c, sd, t)
        for cuts in ([9] * 30, [8, 1] * 20, [1, 8] * 20, [PAGE - 1, 2, 2, 2, 2, 1, 1, 1, 40], [64, 5, 68]):
            close(run_cuts(eng, "a", t, cuts), ref)


@pytest.mark.parametrize("dev", DEVICES)
def test_convolution_window_and_temperature(dev):
    """Convolutions that read only their oldest tap, across portions' edges; score factors of either
    sign; a rotation that turns far keys away."""
    c, cfg, sd = make([layer(AT, None, conv=4, scale=1.5, **window(12, 3)), layer(MB, None, conv=4)], seed=40)
    for k in list(sd):
        if k.endswith(".conv"):
            w = torch.zeros_like(sd[k])
            w[:, 0] = 1.0
            w[:, -1] = 0.25
            sd[k] = w
    sd["l0.mix.temp"] = torch.tensor([2.0, -1.0, 0.0, 0.5]).to(torch.bfloat16)
    t = toks(PAGE + 11, cfg.vocab, 42)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev)
    close(run_whole(eng, "w", t), ref)
    close(run_cuts(eng, "a", t, [1, 1, 1, 1, 2, 2, 3, 1, 5, 1, 1, PAGE - 15, 1, 2, 1]), ref)
    other = copy.deepcopy(c)
    other["layers"][0]["mixer"]["rot"]["base"] = 3.0
    assert (O.forward(other, sd, t) - ref).abs().max() > 1e-3


@pytest.mark.parametrize("dev", DEVICES)
def test_slow_and_fast_states(dev):
    """A decay near one keeps the first token alive for hundreds of tokens; step sizes from tiny to
    large and decay rates over three orders of magnitude."""
    c, cfg, sd = make([layer(LG, None, heads=2, decay=[0.9999, 0.01]), layer(MB, None)], seed=45)
    A = torch.linspace(-4.0, 3.0, sd["l1.mix.A_log"].numel()).reshape(sd["l1.mix.A_log"].shape)
    sd["l1.mix.A_log"] = A.to(torch.bfloat16)
    sd["l1.mix.dt.b"] = torch.linspace(-9.0, 3.0, sd["l1.mix.dt.b"].numel()).to(torch.bfloat16)
    n = 4 * PAGE + 3
    t = toks(n, cfg.vocab, 46)
    t2 = [(t[0] + 1) % cfg.vocab] + t[1:]
    ref, ref2 = O.forward(c, sd, t), O.forward(c, sd, t2)
    assert (ref[-1] - ref2[-1]).abs().max() > 1e-4
    eng = engine(cfg, sd, dev)
    close(run_whole(eng, "a", t), ref)
    close(run_cuts(eng, "b", t2, [100, 20, 1, 1, 130]), ref2)


# ------------------------------------------------------------------ bf16 serving precision
@pytest.mark.parametrize("dev", DEVICES)
def test_bfloat16(dev):
    c, cfg, sd = make([layer(MB, FF, inner=96, state=16, dt_rank=8, conv=4),
                       layer(AT, FF, heads=8, kv_heads=2, dim=32, vdim=48, conv=4, scale=0.2, **window(40, 8)),
                       layer(LG, FF, heads=4, dim=32, vdim=24, decay=[0.5, 0.9, 0.97, 0.99]),
                       layer(AT, None, heads=4, kv_heads=4, dim=20, vdim=12, scale=0.3)],
                      width=128, vocab=200, seed=13, scale=0.8)
    t = toks(PAGE + 90, cfg.vocab, 50)
    ref = O.forward(c, sd, t)
    eng = engine(cfg, sd, dev, dtype=torch.bfloat16)
    close(run_whole(eng, "a", t), ref, tol=0.06)
    close(run_cuts(eng, "b", t, [50, 64] + [1] * 40), ref, tol=0.06)


# ------------------------------------------------------------------ generation
def near_tie(c, sd, prompt, got, n):
    """Greedy tokens equal the oracle's, or differ only where its top two logits tie."""
    lg = O.forward(c, sd, list(prompt) + got[:n - 1])
    for i, tkn in enumerate(got[:n]):
        row = lg[len(prompt) - 1 + i]
        assert tkn == int(row.argmax()) or float(row.max() - row[tkn]) < 1e-3 * float(row.abs().max())


@pytest.mark.parametrize("dev", DEVICES)
def test_generate_greedy(dev):
    c, cfg, sd = make([layer(AT, FF), MB, layer(LG, FF)], seed=14)
    prompts = [toks(n, cfg.vocab, 60 + n) for n in (12, 70, 3)]
    eng = engine(cfg, sd, dev, max_prefill_tokens=32)      # prompts are cut into portions
    res = eng.generate(prompts, max_new_tokens=30, stop_on_eos=False)
    for p, r in zip(prompts, res):
        assert len(r.tokens) == 30 and r.prompt_eval_count == len(p)
        near_tie(c, sd, p, r.tokens, 30)
    assert eng.cache.live == 0 and eng.cache.slots.free_slots == 4


@pytest.mark.parametrize("dev", DEVICES)
def test_server_scheduler_greedy(dev):
    """Through the continuous-batching server: the native scheduler owns the pages, requests
    arrive while others decode, pages are handed back and used again."""
    native = pytest.importorskip("p2p_llm_chat_go_amd.native")
    try:
        native.load()
    except Exception as e:  # noqa: BLE001
        pytest.skip("native runtime not built: %s" % e)
    from p2p_llm_chat_go_amd.engine.sampling import SamplingParams
    from p2p_llm_chat_go_amd.engine.server import EngineServer

    c, cfg, sd = make([layer(LG, FF), layer(AT, FF), MB], seed=15)
    eng = engine(cfg, sd, dev, pages=40, slots=2, max_prefill_tokens=48)
    srv = EngineServer(eng, max_batch=2, decode_chunk=4)
    try:
        prompts = [toks(n, cfg.vocab, 80 + n) for n in (20, 5, 66, 9, 31)]
        futs = [srv.submit(p, SamplingParams(max_tokens=10, stop_on_eos=False)) for p in prompts]
        for p, f in zip(prompts, futs):
            r = f.result(timeout=120)
            assert len(r["tokens"]) == 10
            near_tie(c, sd, p, r["tokens"], 10)
        assert eng.cache.slots.free_slots == 2
    finally:
        srv.close()


@pytest.mark.gpu
def test_decode_graph_matches_eager():
    """Greedy decoding through the captured step graph, replayed many times with eager steps
    of other requests in between, gives the tokens of the eager engine."""
    c, cfg, sd = make([layer(AT, FF, conv=4, dim=16, vdim=16, **window(24, 8)), layer(MB, FF), layer(LG, FF)], width=64,
                      seed=16)
    prompts = [toks(n, cfg.vocab, 90 + n) for n in (70, 5, 33)]
    w = Hy.HybridWeights(cfg, sd, "cuda:0", torch.bfloat16)
    outs = []
    for graph in (True, False):
        eng = HybridEngine(cfg, w, "cuda:0", kv_pages=24, num_slots=4, max_batch=4, use_graph=graph)
        res = eng.generate(prompts, max_new_tokens=40, stop_on_eos=False)
        res2 = eng.generate(prompts[:2], max_new_tokens=70, stop_on_eos=False)
        outs.append([r.tokens for r in res + res2])
        assert bool(eng._graphs) == graph
    # the split of a captured step's keys is fixed while an eager step's follows the position, so the
    # two may round a near tie differently: their tokens agree up to the first one of a request
    same = sum(a == b for a, b in zip(*outs))
    assert same >= 4, outs
    for p, t in zip(prompts, outs[0]):
        assert len(t) == 40


def test_trace_runner_cli(tmp_path):
    """bin/trace_run on a saved checkpoint: steps on stdin, logits files and 'done' lines out,
    finished requests hand their pages and slot back (the pool is smaller than the sum)."""
    import json
    import os
    import subprocess

    import numpy as np
    from safetensors.torch import save_file

    c, cfg, sd = make([layer(AT, FF), layer(MB, None), layer(LG, FF)], seed=17)
    model = tmp_path / "model"
    model.mkdir()
    (model / "config.json").write_text(json.dumps(c))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(model / "model.safetensors"))
    a, b, d = toks(90, cfg.vocab, 1), toks(40, cfg.vocab, 2), toks(100, cfg.vocab, 3)
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:50], "want": [0, 49]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[50:88], "want": []},
                                {"id": "b", "tokens": b[:39], "want": [38]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[39:], "want": [0]},
                                {"id": "a", "tokens": a[88:], "want": [0, 1]}], "end": ["a", "b"]},
        {"step": 3, "entries": [{"id": "d", "tokens": d, "want": [99]}], "end": ["d"]},
    ]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    r = subprocess.run([os.path.join(root, "bin", "trace_run"), "--model", str(model), "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "192", "--device", "cpu"],
                       input="".join(json.dumps(x) + "\n" for x in steps), capture_output=True, text=True,
                       timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [ln for ln in r.stdout.split("\n") if ln.startswith("done")] == ["done %d" % i for i in range(4)]
    ra, rb, rd = (O.forward(c, sd, t) for t in (a, b, d))
    got = {i: torch.from_numpy(np.fromfile(out / ("%d.f32" % i), dtype="<f4").reshape(-1, cfg.vocab))
           for i in (0, 1, 2, 3)}
    close(got[0], ra[[0, 49]])
    close(got[1], rb[[38]])
    close(got[2], torch.stack([rb[39], ra[88], ra[89]]))
    close(got[3], rd[[99]])


def test_preset_through_registry(tmp_path):
    """The preset and a saved checkpoint both reach the hybrid engine through the registry."""
    import json

    from safetensors.torch import save_file

    from p2p_llm_chat_go_amd.models import registry
    from p2p_llm_chat_go_amd.models.config import get_config

    cfg = get_config("tiny-rasepel")
    assert cfg.design == "Rasepel" and not cfg.is_moe and not cfg.traits.positions and cfg.embed_scale == 4.0
    sd = Hy.random_state_dict(cfg, 3)
    (tmp_path / "config.json").write_text(json.dumps(cfg.to_dict()))
    save_file({k: v.contiguous() for k, v in sd.items()}, str(tmp_path / "model.safetensors"))
    assert registry.is_hybrid_dir(str(tmp_path)) and registry.supports_dtype(str(tmp_path), torch.float32)
    cfg2, w = registry.load_checkpoint(str(tmp_path), "cpu", torch.float32)
    assert cfg2.layers == cfg.layers and cfg2.embed_scale == cfg.embed_scale
    assert w.head is w.embed
    eng = registry.make_engine(cfg2, w, "cpu", kv_pages=6, num_slots=2, max_batch=2, dtype=torch.float32)
    p = toks(9, cfg.vocab, 5)
    r = eng.generate([p], max_new_tokens=4, stop_on_eos=False)[0]
    near_tie(cfg.to_dict(), sd, p, r.tokens, 4)


def test_config_roundtrip_and_errors():
    c, cfg, sd = make([layer(AT, FF), layer(MB, None), layer(LG, FF)])
    again = Hy.HybridConfig.from_dict(cfg.to_dict())
    assert again.layers == cfg.layers and again.design == "Rasepel" and again.embed_scale == cfg.embed_scale
    assert set(Hy.tensor_shapes(cfg)) == set(sd) and "head" not in sd and "pos" not in sd
    assert "l1.norm2" not in sd and "l0.norm2" in sd and sd["l0.mix.g"].shape == (4 * 24, cfg.width)
    assert sd["l0.mix.k.conv"].shape == (2 * 16, 3) and sd["l1.mix.A_log"].shape == (40, 10)
    # attention keeps tokens, blocks and the convolution's inputs; the recurrences their states
    w = Hy.HybridWeights(cfg, sd, "cpu", torch.float32)
    at, mb, lg = w.cache_specs()
    assert at == [("paged", 80), ("state", {"tail": (2, 4 * 16 + 2 * 16 + 2 * 24)}), ("pooled", (80, 5))]
    assert mb == ("state", {"S": (10, 40), "tail": (2, 40)}) and lg == ("state", {"S": (3, 20, 12)})
    eng = engine(cfg, sd, "cpu", pages=6)
    assert eng.cache.pooled[0].shape == (6 * 13, 80)        # 13 blocks of 5 tokens end in a page of 64 at most
    assert eng.cache.bytes_per_page() == (PAGE + 13) * 80 * 4
    bad = dict(sd)
    bad["l0.mix.temp"] = bad["l0.mix.temp"][:2]
    with pytest.raises(ValueError):
        Hy.HybridWeights(cfg, bad, "cpu", torch.float32)
    with pytest.raises(KeyError):
        Hy.HybridWeights(cfg, {k: v for k, v in sd.items() if k != "l0.mix.o.b"}, "cpu", torch.float32)
    for L in (layer(AT, None, heads=5, kv_heads=2), layer(AT, None, mask={"size": 0, "pool": 4}),
              layer(AT, None, rot={"base": 10.0, "dims": 18}), layer(LG, None, decay=[0.5]), layer(MB, None, state=0)):
        with pytest.raises(ValueError):
            make([L])
    eng = engine(cfg, sd, "cpu", pages=2, slots=1)
    eng.step([("a", [1, 2, 3], [2])])
    with pytest.raises(MemoryError):
        eng.step([("b", [1], [0])])          # no second state slot
    with pytest.raises(MemoryError):
        eng.step([("a", [1] * PAGE, [])])    # no second page
