"""Bugapel's mechanisms one at a time against the plain oracle of tests/bugapel_oracle.py: the new and extended
operators directly, and every mixer alone through the model's own methods with hand-made batches (portions,
pages in any order, decode rows, slots taken over), on inputs made so that a fault shows: keys that tower over
the others just inside and just outside windows and the kept tokens, at page borders and far back.
"""
import math

import numpy as np
import pytest
import torch

import bugapel_oracle as oracle
from localai_amd import ops
from localai_amd.models.bugapel import BugapelModel
from localai_amd.models.decoder import ForwardBatch
from localai_amd.models.hf_checkpoint import open_model
from localai_amd.models.layered import RoutedExperts
from test_bugapel import SCALING, attention, attention_2, bare, config, gla, make_weights, write_checkpoint

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
MODES = [("cpu", "float32"), pytest.param("cuda:0", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda:0", "bfloat16", marks=pytest.mark.gpu)]


def rel(got, want):
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    return float((got - want).norm() / want.norm().clamp_min(1e-12))


def row_err(got, want):
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    return (got - want).norm(dim=-1) / want.norm(dim=-1).clamp_min(1e-9)


def i32(v, dev="cpu"):
    return torch.tensor(np.asarray(v), dtype=torch.int32, device=dev)


def results(g, T, N, device):
    """(what an operator is given, its value): one fp32 / bf16 matrix, fp32 slabs, all without and with a bias."""
    b = torch.randn(T, N, generator=g)
    bias = torch.randn(N, generator=g)
    for S in (3, 6):
        sl = torch.randn(S, T, N, generator=g)
        yield ops.Partial(sl.to(device)), sl.sum(0)
        yield ops.Partial(sl.to(device), bias.to(device)), sl.sum(0) + bias
    yield ops.Partial(b.to(torch.bfloat16).to(device), bias.to(device)), b.to(torch.bfloat16).float() + bias
    yield b.to(device), b
    yield b.to(torch.bfloat16).to(device), b.to(torch.bfloat16).float()


# ------------------------------------------------------------------------------------------- streams
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("n,T,D", [(1, 5, 48), (2, 5, 35), (3, 4, 1028), (4, 2, 4100), (2, 3, 8200), (5, 6, 64), (16, 3, 1032), (2, 520, 1032),
                                   (3, 2, 33), (16, 2, 41)])
def test_streams_exchange_weighted_sum_and_norm(device, n, T, D):
    """Few and many rows (both workgroup sizes), widths beyond what a thread keeps in registers, stream counts of
    every instance; a mix matrix that is far from symmetric, so that from and to cannot be taken for one another."""
    g = torch.Generator().manual_seed(n * 10000 + D)
    X0 = torch.randn(T, n, D, generator=g) * 3 + 1
    mix = torch.randn(n, n, generator=g).triu() + 0.1
    out_w, in_w = torch.randn(n, generator=g), torch.randn(n, generator=g) + 1
    w, b = 1 + 0.3 * torch.randn(D, generator=g), torch.randn(D, generator=g)
    dev = lambda *t: [x.to(device) for x in t]  # noqa: E731
    dm, do, di, dw, db = dev(mix, out_w, in_w, w, b)
    for br, val in results(g, T, D, device):
        X = X0.clone().to(device)
        out = ops.hyper_streams(X, br, dm, do, di, (dw, db, 1e-2), out_dtype=torch.float32)
        want = oracle.streams_out(X0.double(), val.double(), mix.double(), out_w.double())
        assert rel(X, want) < 2e-6
        u = oracle.streams_in(want, in_w.double())
        assert float(row_err(out, oracle.layer_norm(u, w.double(), b.double(), 1e-2)).max()) < 2e-5
    # the plain sum, in 16 bits; no output; nothing but the norm
    out = ops.hyper_streams(X, None, norm=(dw, db, 1e-3))
    assert out.dtype == torch.bfloat16 and rel(out, oracle.layer_norm(want.sum(1), w.double(), b.double(), 1e-3)) < 5e-3
    assert rel(X, want) < 2e-6
    assert ops.hyper_streams(X, val.to(device), dm, do) is None
    # streams that start as one row each, with and without a first result
    x0 = torch.randn(T, D, generator=g)
    X = torch.full((T, n, D), float("nan"), device=device)
    out = ops.hyper_streams(X, None, in_w=di, norm=(dw, db, 1e-2), init=x0.to(device), out_dtype=torch.float32)
    copies = x0.double().unsqueeze(1).repeat(1, n, 1)
    assert rel(X, copies) < 1e-7
    assert float(row_err(out, oracle.layer_norm(oracle.streams_in(copies, in_w.double()), w.double(), b.double(), 1e-2)).max()) < 5e-5
    X = torch.full((T, n, D), float("nan"), device=device)
    ops.hyper_streams(X, val.to(device), dm, do, init=x0.to(device))
    assert rel(X, oracle.streams_out(copies, val.double(), mix.double(), out_w.double())) < 2e-6


# ------------------------------------------------------------------------------------------- rotated heads
@pytest.mark.parametrize("scaling", [None, SCALING, {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192},
                                     {"factor": 3.0, "low": 2.0, "high": 9.0, "original": 500}])
@pytest.mark.parametrize("dims,base", [(2, 100.0), (8, 50.0), (64, 500000.0), (96, 10000.0)])
def test_rotation_frequencies(dims, base, scaling):
    f, mag = ops.rot_freqs(dims, base, scaling)
    want = oracle.frequencies(dims, base, scaling)
    assert mag == 1.0 and np.allclose(f.numpy(), want, rtol=1e-6)
    if scaling and scaling["original"] == 8192 and dims > 60:      # all three ranges occur
        plain = np.array(oracle.frequencies(dims, base))
        r = f.numpy() / plain
        assert (r > 0.999).any() and (np.abs(r * 8 - 1) < 1e-3).any() and ((r < 0.99) & (r * 8 > 1.01)).any()


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("interleaved", [False, True])
@pytest.mark.parametrize("H,G,D,Dv,rot", [(4, 2, 12, 8, 8), (3, 1, 7, 5, 2), (5, 5, 10, 6, 0), (2, 2, 64, 64, 64), (8, 2, 64, 32, 32), (4, 1, 80, 16, 80),
                                          (4, 4, 24, 40, 16), (16, 4, 128, 128, 128), (2, 1, 200, 8, 24), (1, 1, 256, 4, 256), (3, 0, 20, 0, 12)])
def test_rotated_heads_into_pages(device, interleaved, H, G, D, Dv, rot):
    """Both pair layouts, with and without the unit norm, biases, slabs and a wider row; pages with leftovers, a row
    without a slot, far positions."""
    g = torch.Generator().manual_seed(H * 100 + D)
    T, BS, W = 9, 8, H * D + G * (D + Dv)
    pos = [0, 1, 2, 3, 40, 41, 1000, 7, 8]
    slots = [16, 17, 18, 19, 0, 1, 9, -1, 31]
    fr = oracle.frequencies(rot, 50.0, SCALING)
    fq, _ = ops.rot_freqs(rot, 50.0, SCALING, device)
    wide = torch.randn(T, W + 8, generator=g)
    sources = list(results(g, T, W, device)) + [(wide.to(device)[:, :W], wide[:, :W])]
    for k, (src, val) in enumerate(sources):
        dt, tol = ((torch.float32, 2e-4) if k % 2 else (torch.bfloat16, 8e-3))      # fp32 angles: position 1000 rounds at 6e-5 rad
        unit = 1e-3 if k % 3 else None
        kc = torch.full((4, G, BS, D), 7.0, dtype=dt).to(device) if G else None
        vc = torch.full((4, G, BS // 8, Dv, 8), 7.0, dtype=dt).to(device) if G else None
        q = ops.head_rope_pages(src, H, D, G, D, Dv, i32(pos, device), i32(slots, device), fq, rot, interleaved, kc, vc,
                                unit_eps=unit, dtype=dt)
        assert q.dtype == dt
        s64 = val.double()
        turn = lambda x, t: (lambda y: y if unit is None else oracle.unit_rms(y, unit))(oracle.rotate(x, pos[t], fr, interleaved))  # noqa: E731
        for t in range(T):
            assert rel(q[t].view(H, D), turn(s64[t, :H * D].view(H, D), t)) < tol
            if slots[t] < 0 or not G:
                continue
            b, o = slots[t] // BS, slots[t] % BS
            assert rel(kc[b, :, o], turn(s64[t, H * D:(H + G) * D].view(G, D), t)) < tol
            assert rel(vc[b, :, o // 8, :, o % 8], s64[t, (H + G) * D:].view(G, Dv)) < (1e-6 if dt == torch.float32 else 4e-3)
        if G:
            assert float(kc[1, :, 2:].float().min()) == 7.0 and float(vc[3, :, 0, :, :7].float().min()) == 7.0


@pytest.mark.parametrize("device", DEVICES)
def test_rotated_heads_of_many_rows(device):
    """More rows than the few that get large workgroups: the same numbers as row by row."""
    H, G, D, Dv, rot, T, BS = 8, 2, 64, 32, 32, 530, 16
    g = torch.Generator().manual_seed(3)
    src = torch.randn(T, H * D + G * (D + Dv), generator=g).to(device)
    fq, _ = ops.rot_freqs(rot, 50.0, None, device)
    pools = [(torch.zeros(34, G, BS, D, device=device), torch.zeros(34, G, BS // 8, Dv, 8, device=device)) for _ in range(2)]
    pos, slots = i32(range(T), device), i32(range(T), device)
    q = ops.head_rope_pages(src, H, D, G, D, Dv, pos, slots, fq, rot, True, *pools[0], unit_eps=1e-4, dtype=torch.float32)
    parts = [ops.head_rope_pages(src[a:a + 53], H, D, G, D, Dv, pos[a:a + 53], slots[a:a + 53], fq, rot, True, *pools[1], unit_eps=1e-4,
                                 dtype=torch.float32) for a in range(0, T, 53)]
    assert rel(q, torch.cat(parts)) < 1e-6 and rel(pools[0][0], pools[1][0]) < 1e-6 and rel(pools[0][1], pools[1][1]) == 0.0
    t = 511
    want = oracle.unit_rms(oracle.rotate(src[t, :H * D].cpu().double().view(H, D), t, oracle.frequencies(rot, 50.0), True), 1e-4)
    assert rel(q[t].view(H, D), want) < 1e-4


@pytest.mark.parametrize("device", DEVICES)
def test_slab_sums_with_a_soft_cap(device):
    g = torch.Generator().manual_seed(4)
    for src, val in results(g, 5, 40, device):
        if isinstance(src, ops.Partial):
            for dt, tol in ((torch.float32, 1e-6), (torch.bfloat16, 5e-3)):
                assert rel(ops.reduce(src, dt, softcap=1.5), 1.5 * torch.tanh(val.double() / 1.5)) < tol


# ------------------------------------------------------------------------------------------- kept first tokens, a one in the denominator
def paged(rows_k, rows_v, perm, BS, nb, dt, dev):
    """Pages (leftovers of 50 elsewhere) holding every sequence's keys and values, and the block tables."""
    G, D = rows_k[0].shape[1:]
    Dv = rows_v[0].shape[2]
    kc = torch.full((nb, G, BS, D), 50.0, dtype=dt)
    vc = torch.full((nb, G, BS // 8, Dv, 8), 50.0, dtype=dt)
    bt = np.zeros((len(rows_k), max(-(-k.shape[0] // BS) for k in rows_k)), dtype=np.int32)
    used = 0
    for b, (k, v) in enumerate(zip(rows_k, rows_v)):
        n = -(-k.shape[0] // BS)
        bt[b, :n] = perm[used:used + n]
        used += n
        for t in range(k.shape[0]):
            blk, o = int(bt[b, t // BS]), t % BS
            kc[blk, :, o] = k[t].to(dt)
            vc[blk, :, o // 8, :, o % 8] = v[t].to(dt)
    return kc.to(dev), vc.to(dev), i32(bt, dev)


def attention_case(H, G, D, Dv, lens, hot, seed):
    """Per sequence q, k, v (bf16-exact) where the keys at the positions `hot` point the way every query does, each a
    little longer than the next: whichever of them is visible and first takes nearly all the weight."""
    g = torch.Generator().manual_seed(seed)
    r16 = lambda x: x.to(torch.bfloat16).float()  # noqa: E731
    u = torch.nn.functional.normalize(torch.randn(G, D, generator=g), dim=-1)
    out = []
    for n in lens:
        k = r16(torch.randn(n, G, D, generator=g) * 0.3)
        q = r16(torch.randn(n, H, D, generator=g) * 0.3 + 4 * u.repeat_interleave(H // G, 0))
        for i, t in enumerate(hot):
            if t < n:
                k[t] = r16((9 + 2 * (len(hot) - i) / len(hot)) * u)
        out.append((q, k, r16(torch.randn(n, G, Dv, generator=g))))
    return out


def hots(window, keep, n):
    """The last kept token and the one after it, page borders, and tokens that queries see just inside and just outside
    their windows."""
    ts = [keep - 1, keep, 15, 16, 31, 32] + list(range(keep + 3, n, max(window - 1, 1)))
    return sorted({t for t in ts if 0 <= t < n})


SHAPES = [(4, 1, 64, 64), (8, 2, 128, 64), (6, 6, 80, 80), (16, 1, 96, 32), (4, 4, 32, 48), (3, 1, 24, 16), (5, 5, 10, 7), (12, 4, 64, 128)]
WINDOWS = [(7, 0), (7, 1), (20, 5), (40, 37), (16, 33), (200, 4), (1, 2), (0, 0)]


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("H,G,D,Dv", SHAPES)
@pytest.mark.parametrize("window,keep", WINDOWS)
def test_kept_tokens_on_the_row_and_tile_kernels(device, dtype, H, G, D, Dv, window, keep):
    """attn_mix: portions (tiles on the GPU in bf16 where the widths allow), then single rows with key splits; with and
    without the one in the denominator."""
    if device == "cpu" and H * D > 400:
        pytest.skip("the widest shapes run on the GPU")
    dt, BS, lens = getattr(torch, dtype), 16, [90, 37]
    seqs = attention_case(H, G, D, Dv, lens, hots(window, keep, 90), H + D)
    scale = 0.12
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(0).permutation(12), BS, 12, dt, device)
    q = torch.cat([s[0] for s in seqs]).view(-1, H * D).to(device=device, dtype=dt)
    T = q.shape[0]
    pos = i32(np.concatenate([np.arange(n) for n in lens]), device)
    tol = 2e-5 if dtype == "float32" else 1.5e-2
    gpu = device != "cpu"
    for one in (False, True):
        sc = scale * (0.1 if one else 1.0)      # small scores: the one counts
        want = torch.cat([oracle.softmax_attention(a.double(), k.double(), v.double(), sc, window, keep, one) for a, k, v in seqs]).view(T, -1)
        kw = dict(window=window, keep=keep, sink=torch.zeros(H, device=device) if one else None)
        tiles, rows = ops.attn_mix_tiles(lens, device) if gpu else (None, 0)
        rs = i32([0] * 90 + [1] * 37, device)
        out = ops.attn_mix(q, kc, vc, rs, pos, bt, H, sc, tiles=tiles, tile_rows=rows, cu_q=i32([0, 90, 127], device), **kw)
        err = row_err(out, want)
        assert float(err.max()) < tol, (int(err.argmax()), float(err.max()))
        # the last row of each sequence alone, its keys dealt to several workgroups
        last = torch.tensor([89, 126], device=device)
        tl = torch.tensor([[0, 0], [1, 0]], dtype=torch.int32, device=device)
        for splits in (1, 3):
            out = ops.attn_mix(q[last].contiguous(), kc, vc, i32([0, 1], device), pos[last].contiguous(), bt, H, sc, tiles=tl if gpu else None,
                               tile_rows=2 if gpu else 0, cu_q=i32([0, 1, 2], device), key_splits=splits, **kw)
            assert rel(out, want[last.cpu()]) < tol


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D", [(4, 1, 64), (8, 2, 128), (6, 6, 80), (16, 1, 96), (4, 2, 192), (2, 1, 256)])
@pytest.mark.parametrize("window,keep,BS", [(40, 4, 16), (200, 37, 32), (333, 1, 16), (65, 130, 32), (0, 0, 32), (7, 500, 64), (100, 32, 128)])
def test_kept_tokens_on_the_decode_kernel(H, G, D, window, keep, BS):
    """The newest row of sequences of 1 .. 700 keys as a decode batch: lengths around the window and the kept tokens,
    several partitions and their merge, more kept tokens than a page and than the window, few and many sequences."""
    dev, dt = "cuda:0", torch.bfloat16
    w = window or 350
    lens = sorted({n for n in (1, 2, 17, keep, keep + 1, w - 1, w, w + 1, w + keep, w + keep + 1, 2 * w + 1, 700) if n > 0})
    # what the longest rows see: the last kept token, the first dropped one, both sides of the window's edge
    hot = sorted({t for t in (keep - 1, keep, 700 - w, 699 - w, 31, 32, 650) if 0 <= t < 700})
    seqs = attention_case(H, G, D, D, lens, hot, H * D)
    nb = sum(-(-n // BS) for n in lens) + 2
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(1).permutation(nb), BS, nb, dt, dev)
    q = torch.stack([s[0][-1] for s in seqs]).to(device=dev, dtype=dt)
    for one, sc in ((False, 0.12), (True, 0.01)):
        sink = torch.zeros(H, device=dev) if one else None
        out = ops.attn_decode(q, kc, vc, bt, i32(lens, dev), sc, 700, window=window, keep=keep, sink=sink)
        # the same rows many times over: one-wave workgroups
        many = 300 // len(lens) + 1
        out2 = ops.attn_decode(q.repeat(many, 1, 1), kc, vc, bt.repeat(many, 1), i32(lens * many, dev), sc, 700, window=window, keep=keep,
                               sink=sink)
        for b, (qq, k, v) in enumerate(seqs):
            n = k.shape[0]
            js = oracle.visible(n - 1, window, keep)
            want = oracle.attend(qq[-1].double(), k[js].double(), v[js].double(), sc, one).view(-1)
            assert rel(out[b].view(-1), want) < 1.5e-2, (n, one)
            assert rel(out2[b + len(lens) * (many - 1)].view(-1), want) < 1.5e-2, (n, one)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D", [(4, 1, 64), (4, 2, 128), (3, 3, 96)])
@pytest.mark.parametrize("window,keep", [(23, 4), (64, 33), (100, 1), (40, 0), (0, 0), (30, 70)])
def test_kept_tokens_on_the_prefill_kernel(H, G, D, window, keep):
    """Three portions: one continuing after cached rows, one from position 0, one of a single row."""
    dev, dt, BS = "cuda:0", torch.bfloat16, 16
    spans = [(50, 190), (0, 70), (20, 21)]
    seqs = attention_case(H, G, D, D, [e for _, e in spans], hots(window, keep, 190), H + D)
    nb = sum(-(-e // BS) for _, e in spans) + 2
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(2).permutation(nb), BS, nb, dt, dev)
    q = torch.cat([s[0][a:] for s, (a, _) in zip(seqs, spans)]).to(device=dev, dtype=dt)
    qlens = [e - a for a, e in spans]
    for one, sc in ((False, 0.12), (True, 0.01)):
        want = torch.cat([oracle.softmax_attention(s[0].double(), s[1].double(), s[2].double(), sc, window, keep, one)[a:]
                          for s, (a, _) in zip(seqs, spans)]).view(q.shape[0], -1)
        out = ops.attn_prefill(q, kc, vc, i32(np.cumsum([0] + qlens), dev), i32([e for _, e in spans], dev), bt, sc,
                               tiles=ops.prefill_tiles(qlens, dev), window=window, keep=keep, sink=torch.zeros(H, device=dev) if one else None)
        err = row_err(out.view(q.shape[0], -1), want)
        assert float(err.max()) < 1.5e-2, (one, int(err.argmax()), float(err.max()))


# ------------------------------------------------------------------------------------------- gated linear attention
GLA = [(3, 8, 6), (1, 5, 7), (2, 64, 64), (5, 40, 72), (1, 200, 16), (8, 16, 8), (2, 128, 130), (4, 96, 48), (1, 1, 1), (2, 250, 33), (1, 256, 256)]


def gla_case(H, Dk, Dv, T, nseq, seed, shift=0.0):
    g = torch.Generator().manual_seed(seed)
    r16 = lambda x: x.to(torch.bfloat16).float()  # noqa: E731
    N = 2 * H * (Dk + Dv)
    src = r16(torch.randn(nseq, T, N + 8, generator=g))
    src[:, 0] *= 8                                        # a write that every later read-out sees
    z, zb = r16(torch.randn(nseq, T, H * Dk, generator=g) * 3), torch.randn(H * Dk, generator=g) + shift
    return src, z, zb, 1 + 0.3 * torch.randn(Dv, generator=g)


def gla_want(src, z, zb, w, tau, H, Dk, Dv, eps):
    T = src.shape[0]
    x = src.double()
    q, k = x[:, :H * Dk].view(T, H, Dk) * Dk ** -0.5, x[:, H * Dk:2 * H * Dk].view(T, H, Dk)
    v, g = x[:, 2 * H * Dk:2 * H * Dk + H * Dv].view(T, H, Dv), x[:, 2 * H * Dk + H * Dv:2 * H * (Dk + Dv)]
    al = torch.exp(oracle.log_sigmoid(z.double() + zb.double()) / tau).view(T, H, Dk)
    o = oracle.unit_rms(oracle.gla_scan(q, k, v, al), eps) * w.double()
    return o.reshape(T, -1) * g * oracle.sigmoid(g)


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("H,Dk,Dv", GLA)
@pytest.mark.parametrize("tau,shift", [(16.0, 0.0), (0.3, -2.0), (1.0, 8.0)])
def test_gla_portions_slots_and_decays(device, dtype, H, Dk, Dv, tau, shift):
    """Two sequences side by side (unequal portions in the last split), whole, in portions down to one row, around the
    chunks of 16, token by token; slots that hold leftovers; decays that forget within a token or two, where running
    products over a chunk would overflow or vanish, and decays near one."""
    if device == "cpu" and (Dk > 64 or H * Dk * Dv > 5000):
        pytest.skip("the widest shapes run on the GPU")
    T = 53
    src, z, zb, w = gla_case(H, Dk, Dv, T, 2, H * 1000 + Dk, shift)
    want = [gla_want(src[s], z[s], zb, w, tau, H, Dk, Dv, 1e-5) for s in range(2)]
    dt = getattr(torch, dtype)
    for cuts in ([T], [1] * T, [2] * 26 + [1], [15, 1, 1, 16, 17, 3], [16, 16, 16, 5], [30, 1, 22]):
        state = torch.full((3, H, Dv, Dk), 9.0).to(device)
        at, got = 0, [[], []]
        for c in cuts:
            rows = torch.cat([src[s, at:at + c] for s in range(2)]).to(device=device, dtype=dt)
            zz = torch.cat([z[s, at:at + c] for s in range(2)]).to(device=device, dtype=dt)
            out = ops.gla(rows, zz, zb.to(device), tau, H, Dk, Dv, i32(list(range(at, at + c)) * 2, device), i32([0, c, 2 * c], device),
                          i32([2, 0], device), state, w.to(device), 1e-5, max_rows=c)
            assert out.dtype == dt
            got[0].append(out[:c])
            got[1].append(out[c:])
            at += c
        for s in range(2):
            err = row_err(torch.cat(got[s]), want[s])
            assert float(err.max()) < (2e-4 if dtype == "float32" else 1e-2), (cuts[:3], s, int(err.argmax()), float(err.max()))
        assert float(state[1].min()) == 9.0 and float(state[1].max()) == 9.0      # nobody's slot


@pytest.mark.parametrize("device,dtype", MODES)
def test_gla_unequal_portions_beside_single_rows(device, dtype):
    """One batch: a long portion, a single row that continues a sequence, a short portion that continues, a new one-row
    sequence, a row without a slot."""
    H, Dk, Dv, T, dt = 3, 24, 20, 60, getattr(torch, dtype)
    src, z, zb, w = gla_case(H, Dk, Dv, T, 5, 77)
    want = [gla_want(src[s], z[s], zb, w, 4.0, H, Dk, Dv, 1e-5) for s in range(5)]
    state = torch.full((5, H, Dv, Dk), 9.0).to(device)
    args = (zb.to(device), 4.0, H, Dk, Dv)

    def run(spans, slots):
        rows = torch.cat([src[s, a:b] for s, a, b in spans]).to(device=device, dtype=dt)
        zz = torch.cat([z[s, a:b] for s, a, b in spans]).to(device=device, dtype=dt)
        pos = i32(np.concatenate([np.arange(a, b) for _, a, b in spans]), device)
        cu = np.cumsum([0] + [b - a for _, a, b in spans])
        out = ops.gla(rows, zz, *args, pos, i32(cu, device), i32(slots, device), state, w.to(device), 1e-5,
                      max_rows=max(b - a for _, a, b in spans))
        for k, (s, a, b) in enumerate(spans):
            err = row_err(out[cu[k]:cu[k + 1]], want[s][a:b])
            assert float(err.max()) < (2e-4 if dtype == "float32" else 1e-2), (s, a, b, float(err.max()))
    run([(1, 0, 20), (2, 0, 33)], [4, 1])
    run([(0, 0, 50), (1, 20, 21), (2, 33, 39), (3, 0, 1), (4, 0, 1)], [3, 4, 1, 0, -1])
    run([(0, 50, 51), (1, 21, 22), (2, 39, 40), (3, 1, 2)], [3, 4, 1, 0])
    run([(3, 2, 60), (0, 51, 60), (1, 22, 24)], [0, 3, 4])
    assert float(state[2].min()) == 9.0


@pytest.mark.parametrize("device,dtype", MODES)
def test_gla_remembers_over_a_long_run(device, dtype):
    """900 rows with decays so near one that the first row's write still shows at the end."""
    H, Dk, Dv, T, dt = 2, 32, 32, 900, getattr(torch, dtype)
    src, z, zb, w = gla_case(H, Dk, Dv, T, 1, 5, shift=6.0)
    src[0, 0] *= 4
    want = gla_want(src[0], z[0], zb, w, 64.0, H, Dk, Dv, 1e-5)
    state = torch.full((1, H, Dv, Dk), 9.0).to(device)
    got, at = [], 0
    for c in [700, 150, 1, 1, 2, 46]:
        out = ops.gla(src[0, at:at + c].to(device=device, dtype=dt), z[0, at:at + c].to(device=device, dtype=dt), zb.to(device), 64.0, H, Dk,
                      Dv, i32(range(at, at + c), device), i32([0, c], device), i32([0], device), state, w.to(device), 1e-5, max_rows=c)
        got.append(out)
        at += c
    err = row_err(torch.cat(got), want)
    assert float(err.max()) < (2e-4 if dtype == "float32" else 1e-2), (int(err.argmax()), float(err.max()))


# ------------------------------------------------------------------------------------------- experts
@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("E,groups,keep,top,D", [(12, 3, 2, 3, 40), (6, 1, 1, 2, 35), (8, 8, 3, 3, 64), (200, 20, 4, 8, 64), (9, 3, 1, 3, 33), (4, 2, 2, 4, 128),
                                                 (256, 128, 5, 6, 32)])
@pytest.mark.parametrize("T", [37, 600])
def test_router_takes_the_best_groups_first(device, dtype, E, groups, keep, top, D, T):
    """Few rows (a workgroup each) and many (four a workgroup)."""
    g = torch.Generator().manual_seed(E)
    x = torch.randn(T, D, generator=g).to(torch.bfloat16).float()
    w = torch.randn(E, D, generator=g)
    ids, wts = ops.router_softmax(x.to(device=device, dtype=getattr(torch, dtype)), w.to(device), None, top, groups, keep, 2.5)
    other = 0
    for t in range(0, T, 1 if T < 100 else 13):
        z = w.double() @ x[t].double()
        want_i, want_w = oracle.route(z, top, groups, keep, 2.5)
        assert ids[t].tolist() == want_i
        assert np.allclose(wts.view(T, top)[t].cpu().numpy(), want_w, rtol=2e-4, atol=1e-7)
        other += want_i != oracle.route(z, top, 1, 1, 2.5)[0]
    assert other > 0 or top <= keep or keep == groups      # else the groups do change the choice
    with pytest.raises(ValueError):
        ops.router_softmax(x.to(device), w.to(device), None, 2, E, 1)


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("E,top,D,F", [(5, 2, 40, 24), (4, 3, 35, 13), (6, 2, 256, 256), (3, 1, 64, 48)])
@pytest.mark.parametrize("T", [1, 2, 7, 33, 80])
def test_ungated_experts_on_every_path(device, dtype, E, top, D, F, T):
    """Pair GEMVs, the grouped expert GEMMs (widths % 256 in bf16) and library GEMMs by batch size; an expert nobody chose."""
    g = torch.Generator().manual_seed(D + T)
    dt = getattr(torch, dtype)
    up, down = (torch.randn(E, F, D, generator=g) * D ** -0.5).to(torch.bfloat16).float(), (torch.randn(E, D, F, generator=g) * F ** -0.5).to(torch.bfloat16).float()
    x = torch.randn(T, D, generator=g).to(torch.bfloat16).float()
    ids = torch.stack([torch.randperm(E - 1 if E > top else E, generator=g)[:top] for _ in range(T)]).to(torch.int32)
    wts = torch.rand(T, top, generator=g) + 0.1
    ex = RoutedExperts([(None, up[e], down[e]) for e in range(E)], torch.device(device), dt, "relu2")
    y = ex(x.to(device=device, dtype=dt), ids.to(device), wts.reshape(-1).to(device))
    y = y.dense() if isinstance(y, ops.Partial) else y
    want = torch.stack([sum(float(wts[t, k]) * (down[e].double() @ torch.relu(up[e].double() @ x[t].double()) ** 2)
                            for k, e in enumerate(ids[t].tolist())) for t in range(T)])
    err = row_err(y, want)
    assert float(err.max()) < (1e-5 if dtype == "float32" else 1.5e-2), float(err.max())


# ------------------------------------------------------------------------------------------- mixers alone
def build(layer, D, tmp_path, device, dtype, seed=0, edit=None):
    """A one-layer checkpoint and its model: (model, the layer's config, float64 weights)."""
    cfg = config([layer], 11, D, 2)
    W = make_weights(cfg, seed)
    if edit:
        edit(W)
    path = str(tmp_path / f"m{seed}")
    write_checkpoint(path, cfg, W)
    return BugapelModel(open_model(path), torch.device(device), dtype=getattr(torch, dtype)), layer, {k: v.double() for k, v in W.items()}


def run_mixer(model, kv, table, slot, h, cuts, bs):
    """Feed rows h (the mixer's input) of one sequence in portions through layer 0's mixer and output
    projection, single rows as decode batches.  fp32 [T, D]."""
    dev, L, m = model.device, model.layers[0], model.hp.mixers[0]
    outs, at = [], 0
    tab = i32([list(table)], dev)
    for c in cuts:
        pos = np.arange(at, at + c)
        dec = c == 1 and at > 0
        fb = ForwardBatch(tokens=i32([0] * c, dev), pos=i32(pos, dev), slots=i32([table[p // bs] * bs + p % bs for p in pos], dev),
                          decode=dec, block_tables=tab, sslots=i32([slot], dev))
        if dec:
            fb.seq_lens, fb.max_len = i32([at + 1], dev), at + 1
        else:
            fb.cu_q, fb.ctx_lens, fb.row_seq, fb.max_q = i32([0, c], dev), i32([at + c], dev), i32([0] * c, dev), c
            fb.tiles, fb.tile_rows = model.prefill_tiles([c], dev)
        b = model._batch_rows(fb)
        x = h[at:at + c].to(model.dtype).to(dev).contiguous()
        a = model._gla(L, m, x, fb, kv, 0, b) if m.kind == "gla" else model._attention(L, m, x, fb, kv, 0, b)
        outs.append(ops.reduce(ops.linear(a, L.wo, L.wo_b)).cpu() if dev.type == "cuda" and model.hp.n_embd % 4 == 0
                    else ops.linear(a, L.wo, L.wo_b).dense().cpu())
        at += c
    return torch.cat(outs, 0)


def check_mixer(model, layer, W, h, cuts_list, bs, nblocks, dtype):
    want = oracle.MIXERS[layer["type"]](W, "l0.mix.", layer["mixer"], h.double(), 1e-5)
    kv = model.new_kv_cache(nblocks, bs, state_slots=3)
    T = h.shape[0]
    for n, cuts in enumerate(cuts_list):
        # pages in another order every time, slots in turn: leftovers of the run before lie in both
        table = [int(b) for b in np.random.default_rng(n).permutation(nblocks)[:-(-T // bs)]]
        err = row_err(run_mixer(model, kv, table, n % 3, h, cuts, bs), want)
        where = (n, int(err.argmax()), float(err.max()), float(err.median()))
        assert float(err.max()) < (2e-4 if dtype == "float32" else 0.1) and float(err.median()) < (5e-5 if dtype == "float32" else 2e-2), where


def inputs(T, D, seed, hot=()):
    """Rows of unit size; the rows listed in `hot` tower over the others."""
    g = torch.Generator().manual_seed(seed)
    h = torch.randn(T, D, generator=g)
    for t in hot:
        h[t] = h[t] * 6
    return h.to(torch.bfloat16).float()


def cuts_of(T, *sizes):
    out, i, k = [], 0, 0
    while i < T:
        s = min(sizes[k % len(sizes)], T - i)
        out.append(s)
        i += s
        k += 1
    return out


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("spec", [dict(), dict(heads=1, dim=5, vdim=7, tau=1.0, rank=1), dict(heads=2, dim=64, vdim=64, tau=0.25, rank=8),
                                  dict(heads=5, dim=40, vdim=72, rank=16), dict(heads=4, dim=128, vdim=130, tau=100.0, rank=5)])
def test_gla_mixer_alone(tmp_path, device, dtype, spec):
    model, layer, W = build(bare(gla(**spec)), 32, tmp_path, device, dtype)
    T = 45
    check_mixer(model, layer, W, inputs(T, 32, 1, hot=(0, 17)), [[T], cuts_of(T, 2), cuts_of(T, 1), cuts_of(T, 7, 1, 2, 16), [30] + [1] * 15], 16, 6, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("spec", [dict(), dict(heads=3, kv=1, dim=10, vdim=6, rot=2, scaling=SCALING), dict(heads=5, kv=5, dim=7, vdim=9, rot=6),
                                  dict(heads=4, kv=2, dim=64, vdim=64, rot=32, scaling=SCALING), dict(heads=8, kv=2, dim=64, vdim=32, rot=64),
                                  dict(heads=4, kv=1, dim=128, vdim=128, rot=128), dict(heads=2, kv=2, dim=16, vdim=16, rot=0)])
def test_attention_mixer_alone(tmp_path, device, dtype, spec):
    """Whole, in portions, token by token (the split-KV decode kernel where the widths allow); one query and key that meet
    over a long distance."""
    model, layer, W = build(bare(attention(**spec)), 32, tmp_path, device, dtype)
    T = 100
    h = inputs(T, 32, 4, hot=(0, 16))
    h[97] = h[3]
    check_mixer(model, layer, W, h, [[T], cuts_of(T, 2), [40] + [1] * 60, cuts_of(T, 33, 1, 9)], 16, 8, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("spec", [dict(), dict(heads=3, kv=1, dim=10, vdim=6, rot=2, window=33, keep=0), dict(heads=5, kv=5, dim=7, vdim=9, rot=6, window=1, keep=1),
                                  dict(heads=4, kv=2, dim=64, vdim=64, rot=32, window=24, keep=4), dict(heads=8, kv=2, dim=64, vdim=32, rot=64, window=17, keep=20),
                                  dict(heads=4, kv=1, dim=128, vdim=128, rot=128, window=40, keep=33), dict(heads=2, kv=2, dim=32, vdim=16, rot=0, window=300, keep=2),
                                  dict(heads=17, kv=1, dim=64, vdim=64, rot=8, window=48, keep=3)])
def test_attention_2_mixer_alone(tmp_path, device, dtype, spec):
    """Towering keys at the last kept position, the first dropped one and around the window's edge; biases larger than
    the projections."""
    def edit(W):
        for n in ("q.b", "k.b", "v.b", "o.b"):
            W["l0.mix." + n] *= 3
    model, layer, W = build(bare(attention_2(**spec)), 32, tmp_path, device, dtype, edit=edit)
    w, kp = layer["mixer"]["mask"]["size"], layer["mixer"]["mask"]["keep_first"]
    T = 100
    h = inputs(T, 32, 4, hot=hots(w, kp, T)[:10])
    c = min(w + kp, 60)
    check_mixer(model, layer, W, h, [[T], cuts_of(T, 2), [c] + [1] * (T - c), cuts_of(T, 33, 1, 9)], 16, 8, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_a_far_key_among_hundreds_kept_or_not(tmp_path, device, dtype):
    """The keys at 3 (kept) and 4 (not kept) stand out for the queries far outside the window."""
    def edit(W):
        for n in ("q.b", "k.b"):
            W["l0.mix." + n] *= 0
        W["l0.mix.k"] = W["l0.mix.q"][:32].clone()      # queries of equal rows meet keys of equal rows
    model, layer, W = build(bare(attention_2(heads=4, kv=2, dim=16, vdim=8, rot=0, window=50, keep=4, scale=1.0)), 32, tmp_path, device, dtype, edit=edit)
    T = 310
    h = inputs(T, 32, 9)
    for i, t in enumerate((290, 295, 300, 305)):
        h[t] = h[3 + i % 2] * 1.5
    check_mixer(model, layer, W, h, [[T], [280] + [1] * 30, cuts_of(T, 77, 2)], 16, 24, dtype)


def test_one_in_the_denominator_shrinks_weak_rows():
    """A lone key of score s weighs e^s / (1 + e^s), far from 1 when s is small."""
    q, k, v = torch.zeros(1, 1, 4), torch.zeros(1, 1, 4), torch.ones(1, 1, 4)
    assert math.isclose(float(oracle.softmax_attention(q.double(), k.double(), v.double(), 1.0, one=True)[0, 0, 0]), 0.5)
