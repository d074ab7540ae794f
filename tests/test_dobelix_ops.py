"""Dobelix's mechanisms one at a time against the plain oracle of tests/dobelix_oracle.py: the new and
extended operators directly, and both mixers alone through the model's own methods with hand-made
batches (portions, pages in any order, decode rows, slots taken over), on inputs made so that a fault
shows: keys that tower over the others at both ends of a chunk, at page borders and far back.
"""
import numpy as np
import pytest
import torch

import dobelix_oracle as oracle
from localai_amd import ops
from localai_amd.models.decoder import ForwardBatch
from localai_amd.models.dobelix import DobelixModel
from localai_amd.models.hf_checkpoint import open_model
from test_dobelix import attention, config, ff, lightning, make_weights, write_checkpoint

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
MODES = [("cpu", "float32"), pytest.param("cuda:0", "float32", marks=pytest.mark.gpu),
         pytest.param("cuda:0", "bfloat16", marks=pytest.mark.gpu)]
F64 = torch.float64


def rel(got, want):
    got, want = got.detach().double().cpu(), want.detach().double().cpu()
    return float((got - want).norm() / want.norm().clamp_min(1e-12))


def i32(v, dev="cpu"):
    return torch.tensor(np.asarray(v), dtype=torch.int32, device=dev)


def branches(g, T, D, device):
    """(what an operator is given, its value): nothing, one fp32 / bf16 matrix, fp32 slabs."""
    b = torch.randn(T, D, generator=g)
    yield None, None
    yield b.to(device), b
    yield b.to(torch.bfloat16).to(device), b.to(torch.bfloat16).float()
    for S in (3, 6):
        sl = torch.randn(S, T, D, generator=g)
        yield ops.Partial(sl.to(device)), sl.sum(0)


# ------------------------------------------------------------------------------------------- sublayer boundaries
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("T,D", [(5, 48), (5, 35), (3, 1028), (2, 4100), (2, 8200), (520, 1032), (520, 4104)])
def test_rms_norm_on_a_branch_and_on_the_stream(device, T, D):
    """Few and many rows (both workgroup sizes), widths beyond what a thread keeps in registers."""
    g = torch.Generator().manual_seed(D)
    res0 = torch.randn(T, D, generator=g) * 3
    w1, w2 = 1 + 0.3 * torch.randn(D, generator=g), 1 + 0.3 * torch.randn(D, generator=g)
    for br, val in branches(g, T, D, device):
        for pre in (("cast",), ("rms", w2.to(device), 1e-3), None):
            res = res0.clone().to(device)
            post = ("rms", w1.to(device), 1e-2) if br is not None else None
            out = ops.norm_chain(res, br, post, pre, out_dtype=torch.float32)
            want = res0.double()
            if val is not None:
                want = want + oracle.rms_norm(val.double(), w1.double(), 1e-2)
            assert rel(res, want) < 1e-6
            if pre is None:
                assert out is None
            else:
                assert rel(out, want if pre[0] == "cast" else oracle.rms_norm(want, w2.double(), 1e-3)) < 2e-6
    out16 = ops.norm_chain(res0.clone().to(device), None, None, ("rms", w2.to(device), 1e-3))
    assert out16.dtype == torch.bfloat16 and rel(out16, oracle.rms_norm(res0.double(), w2.double(), 1e-3)) < 5e-3


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("taps,D", [(1, 24), (2, 35), (3, 40), (4, 256), (5, 33), (4, 2048), (3, 4100)])
def test_stream_convolution_portions_tails_and_slots(device, taps, D):
    """Two sequences in one batch, portions down to one row, single-row batches (norm, add, convolution and
    tail in one launch), slots that hold another sequence's leftovers, a row without a slot."""
    g = torch.Generator().manual_seed(taps * 1000 + D)
    T = 23
    xs = [torch.randn(T, D, generator=g), torch.randn(T, D, generator=g)]
    w = torch.randn(D, taps, generator=g) * 0.5
    nw = 1 + 0.3 * torch.randn(D, generator=g)
    wt = w.t().contiguous().to(device)
    want = [x.double() + oracle.causal_conv(x.double(), w.double()) for x in xs]
    for cuts in ([T], [1] * T, [2] * 11 + [1], [7, 1, 3, 12], [1, 1, 2, 19]):
        tail = torch.full((3, taps - 1, D), 9.0).to(device)
        at, got = 0, [[], []]
        for c in cuts:
            single = c == 1
            base = [x[at:at + c] for x in xs]
            pos = i32(list(range(at, at + c)) * 2, device)
            cu, rs, ss = i32([0, c, 2 * c], device), i32([0] * c + [1] * c, device), i32([2, 0], device)
            # the rows reach the stream as branch + residual (a branch whose unit norm is known)
            br = torch.randn(2 * c, D, generator=g)
            add = oracle.rms_norm(br.double(), nw.double(), 1e-3).float()
            res = (torch.cat(base) - add).to(device)
            out = ops.stream_conv(res, br.to(device), ("rms", nw.to(device), 1e-3), wt, rs, cu, pos, ss, tail, single=single,
                                  out_dtype=torch.float32)
            assert rel(res, torch.cat(base)) < 1e-6
            got[0].append(out[:c].cpu())
            got[1].append(out[c:].cpu())
            at += c
        for s in range(2):
            assert rel(torch.cat(got[s]), want[s]) < 3e-6, (cuts, s)
            if taps > 1:
                assert rel(tail[2 - 2 * s], xs[s][-(taps - 1):]) < 1e-6
        if taps > 1:
            assert float(tail[1].min()) == 9.0      # nobody's slot
    # slabs and bf16 as the branch of a single-row batch without a norm, 16-bit output, a row without a slot
    for br, val in branches(g, 2, D, device):
        res = torch.stack([xs[0][0], xs[1][0]]).to(device)
        tail = torch.full((2, taps - 1, D), 9.0).to(device)
        out = ops.stream_conv(res, br, None, wt, None, None, i32([0, 5], device), i32([1, -1], device), tail, single=True)
        x = torch.stack([xs[0][0], xs[1][0]]).double() + (0 if val is None else val.double())
        assert out.dtype == torch.bfloat16 and rel(out, x * (1 + w[:, -1].double())) < 5e-3
        assert taps == 1 or float(tail[0].min()) == 9.0


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("F", [13, 40, 1000])
def test_gated_units(device, F):
    g = torch.Generator().manual_seed(F)
    z = (torch.randn(6, 2 * F, generator=g) * 3).to(torch.bfloat16)
    for mode, fn in ((ops.ACT_GEGLU, oracle.gelu_tanh), (ops.ACT_SWIGLU, oracle.silu)):
        want = fn(z[:, :F].double()) * z[:, F:].double()
        for src in (z.to(device), z.float().to(device), ops.Partial(torch.stack([z.float() * 0.25, z.float() * 0.75]).to(device))):
            assert rel(ops.glu_act(src, F, mode, torch.float32), want) < 3e-6
        out = ops.glu_act(ops.Partial(z.to(device)), F, mode)
        assert out.dtype == torch.bfloat16 and rel(out, want) < 5e-3


# ------------------------------------------------------------------------------------------- keys that are values
@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("H,G,D,rot", [(4, 2, 12, 8), (3, 1, 7, 2), (5, 5, 10, 0), (2, 2, 64, 64), (8, 2, 64, 32), (4, 1, 80, 80),
                                       (4, 4, 24, 16), (16, 4, 128, 128)])
def test_row_normed_rotated_pages_with_raw_keys_as_values(device, H, G, D, rot):
    """One root mean square over all query heads and one over all key heads, weights per channel, rotation of the
    first dims, a number per query head; pages with leftovers, a row without a slot, far positions."""
    g = torch.Generator().manual_seed(H * 100 + D)
    T, BS = 9, 8
    src = torch.randn(T, (H + G) * D + 8, generator=g)           # columns to spare: a wider projection
    src[:, :D] *= 5                                             # heads of unequal size: a norm per head would show
    src[:, H * D:H * D + D] *= 0.2
    src = src.to(torch.bfloat16).float()
    qw, kw = 1 + 0.3 * torch.randn(H * D, generator=g), 1 + 0.3 * torch.randn(G * D, generator=g)
    temp = torch.randn(H, generator=g)
    pos = [0, 1, 2, 3, 40, 41, 1000, 7, 8]
    slots = [16, 17, 18, 19, 0, 1, 9, -1, 31]
    fq = ops.linear_rot_freqs(rot, 50.0, 1.0, device)
    for dt, tol in ((torch.float32, 5e-5), (torch.bfloat16, 6e-3)):     # fp32 angles: position 1000 rounds at 6e-5 rad
        kc = torch.full((4, G, BS, D), 7.0, dtype=dt).to(device)
        vc = torch.full((4, G, BS // 8, D, 8), 7.0, dtype=dt).to(device)
        q = ops.qk_row_norm_rope_pages(src.to(device=device, dtype=dt), H, D, G, i32(pos, device), i32(slots, device),
                                       qw.to(device), kw.to(device), 1e-5, fq, rot, kc, vc, head_scale=temp.to(device))
        plain = ops.qk_row_norm_rope_pages(src.to(device=device, dtype=dt), H, D, G, i32(pos, device), i32([-1] * T, device),
                                           qw.to(device), kw.to(device), 1e-5, fq, rot, kc, vc)
        s64 = src.double()
        for t in range(T):
            qq = oracle.rms_norm(s64[t, :H * D], qw.double(), 1e-5).view(H, D)
            qq = oracle.rotate_halves(qq, pos[t], rot, 50.0)
            assert rel(plain[t].view(H, D), qq) < tol
            assert rel(q[t].view(H, D), qq * temp.double().view(H, 1)) < tol
            if slots[t] < 0:
                continue
            b, o = slots[t] // BS, slots[t] % BS
            raw = s64[t, H * D:(H + G) * D]
            kk = oracle.rotate_halves(oracle.rms_norm(raw, kw.double(), 1e-5).view(G, D), pos[t], rot, 50.0)
            assert rel(kc[b, :, o], kk) < tol
            assert rel(vc[b, :, o // 8, :, o % 8], raw.view(G, D)) < 1e-7
        assert float(kc[1, :, 2:].float().min()) == 7.0 and float(vc[3, :, 0, :, :7].float().min()) == 7.0


# ------------------------------------------------------------------------------------------- sigmoid attention
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


def attention_case(H, G, D, lens, chunk, hot, seed):
    """Per sequence q, k, v (bf16-exact) where the keys at the positions `hot` point the way every query does: their
    weight is near 1 beside a few hundredths for the others, so that one wrongly seen or missed shows."""
    g = torch.Generator().manual_seed(seed)
    r16 = lambda x: x.to(torch.bfloat16).float()  # noqa: E731
    u = torch.nn.functional.normalize(torch.randn(G, D, generator=g), dim=-1)
    out = []
    for n in lens:
        k = r16(torch.randn(n, G, D, generator=g) * 0.3)
        q = r16(torch.randn(n, H, D, generator=g) * 0.3 + 4 * u.repeat_interleave(H // G, 0))
        for t in hot:
            if t < n:
                k[t] = r16(10 * u)
        out.append((q, k, r16(torch.randn(n, G, D, generator=g))))
    return out


def hots(chunk, n):
    """Both ends of the chunks, page borders, the first position."""
    edges = [c for e in range(0, n, chunk or n) for c in (e, e + (chunk or n) - 1)]
    return sorted({t for t in edges + [0, 15, 16, 31, 32] if t < n})


SHAPES = [(4, 1, 64), (8, 2, 128), (6, 6, 80), (16, 1, 96), (4, 4, 32), (3, 1, 24), (5, 5, 10)]


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("H,G,D", SHAPES)
@pytest.mark.parametrize("chunk", [7, 40, 0])
def test_sigmoid_attention_on_the_row_and_tile_kernels(device, dtype, H, G, D, chunk):
    """attn_mix: portions (tiles on the GPU in bf16 where the widths allow), then single rows with key splits; a
    gate per head and per channel."""
    if device == "cpu" and H * D > 400:
        pytest.skip("the widest shapes run on the GPU")
    dt, BS, lens = getattr(torch, dtype), 16, [90, 37]
    seqs = attention_case(H, G, D, lens, chunk, hots(chunk, 90), H + D)
    g = torch.Generator().manual_seed(1)
    pb, scale = torch.randn(H, generator=g) * 0.5 - 3.0, 0.12
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(0).permutation(12), BS, 12, dt, device)
    want = [oracle.sigmoid_attention(q.double(), k.double(), v.double(), scale, [1.0] * H, pb.double(), chunk) for q, k, v in seqs]
    q = torch.cat([s[0] for s in seqs]).view(-1, H * D).to(device=device, dtype=dt)
    T = q.shape[0]
    pos = i32(np.concatenate([np.arange(n) for n in lens]), device)
    tol = 1e-5 if dtype == "float32" else 1.5e-2
    w = torch.cat(want)
    for gw in (0, H, H * D):
        gate = (torch.randn(T, gw + 3, generator=g) * 2).to(dt).to(device)[:, 3:] if gw else None
        ww = w if not gw else w * oracle.sigmoid(gate.cpu().double()).view(T, H, gw // H)
        tiles, rows = ops.attn_mix_tiles(lens, device) if device != "cpu" else (None, 0)
        kw = dict(chunk=chunk, sigmoid_bias=pb.to(device), gate=gate, cu_q=i32([0, 90, 127], device))
        rs = i32([0] * 90 + [1] * 37, device)
        out = ops.attn_mix(q, kc, vc, rs, pos, bt, H, scale, tiles=tiles, tile_rows=rows, **kw)
        err = (out.cpu().double().view(T, -1) - ww.view(T, -1)).norm(dim=-1) / ww.view(T, -1).norm(dim=-1)
        assert float(err.max()) < tol, (int(err.argmax()), float(err.max()))
        # the last row of each sequence alone, its keys dealt to several workgroups
        last = torch.tensor([89, 126], device=device)
        one = torch.tensor([[0, 0], [1, 0]], dtype=torch.int32, device=device)
        kw.update(cu_q=i32([0, 1, 2], device), gate=None if gate is None else gate[last].contiguous())
        out = ops.attn_mix(q[last].contiguous(), kc, vc, i32([0, 1], device), pos[last].contiguous(), bt, H, scale,
                           tiles=one if device != "cpu" else None, tile_rows=2 if device != "cpu" else 0, key_splits=3, **kw)
        assert rel(out, ww[last.cpu()].reshape(2, -1)) < tol


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D", [(4, 1, 64), (8, 2, 128), (6, 6, 80), (16, 1, 96), (4, 2, 192), (2, 1, 256)])
@pytest.mark.parametrize("chunk,BS", [(40, 16), (200, 32), (333, 16), (0, 32)])
def test_sigmoid_attention_on_the_decode_kernel(H, G, D, chunk, BS):
    """The newest row of sequences of 1 .. 700 keys as a decode batch: lengths around chunk edges, several partitions
    and their merge, one-wave and four-wave workgroups by batch size; the gate per channel read from a wider row."""
    dev, dt = "cuda:0", torch.bfloat16
    c = chunk or 350
    lens = sorted({1, 2, 17, c - 1, c, c + 1, 2 * c, 2 * c + 1, 700})
    seqs = attention_case(H, G, D, lens, chunk, hots(chunk, 701), H * D)
    g = torch.Generator().manual_seed(2)
    pb, scale = torch.randn(H, generator=g) * 0.5 - 4.0, 0.12
    nb = sum(-(-n // BS) for n in lens) + 2
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(1).permutation(nb), BS, nb, dt, dev)
    q = torch.stack([s[0][-1] for s in seqs]).to(device=dev, dtype=dt)
    gate = (torch.randn(len(lens), H * D + 16, generator=g) * 2).to(dt).to(dev)[:, 8:8 + H * D]
    out = ops.attn_decode(q, kc, vc, bt, i32(lens, dev), scale, 700, sigmoid_bias=pb.to(dev), chunk=chunk, gate=gate)
    plain = ops.attn_decode(q, kc, vc, bt, i32(lens, dev), scale, 700, sigmoid_bias=pb.to(dev), chunk=chunk)
    for b, (qq, k, v) in enumerate(seqs):
        n = k.shape[0]
        lo = (n - 1) // chunk * chunk if chunk else 0
        want = oracle.sigmoid_attention(torch.cat([torch.zeros(n - lo - 1, H, D), qq[-1:]]).double(), k[lo:].double(), v[lo:].double(),
                                        scale, [1.0] * H, pb.double(), 0)[-1].view(-1)
        assert rel(plain[b].view(-1), want) < 1.5e-2, (lens[b], chunk)
        assert rel(out[b].view(-1), want * oracle.sigmoid(gate[b].cpu().double())) < 1.5e-2, (lens[b], chunk)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,D", [(4, 1, 64), (4, 2, 128), (3, 3, 96)])
@pytest.mark.parametrize("chunk", [23, 64, 100, 0])
def test_sigmoid_attention_on_the_prefill_kernel(H, G, D, chunk):
    """Three portions: one continuing after cached rows in the middle of a chunk, one from position 0, one of a single row."""
    dev, dt, BS = "cuda:0", torch.bfloat16, 16
    spans = [(50, 190), (0, 70), (20, 21)]
    seqs = attention_case(H, G, D, [e for _, e in spans], chunk, hots(chunk, 190), H + D)
    g = torch.Generator().manual_seed(3)
    pb, scale = torch.randn(H, generator=g) * 0.5 - 4.0, 0.12
    nb = sum(-(-e // BS) for _, e in spans) + 2
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(2).permutation(nb), BS, nb, dt, dev)
    q = torch.cat([s[0][a:] for s, (a, _) in zip(seqs, spans)]).to(device=dev, dtype=dt)
    want = torch.cat([oracle.sigmoid_attention(s[0].double(), s[1].double(), s[2].double(), scale, [1.0] * H, pb.double(), chunk)[a:]
                      for s, (a, _) in zip(seqs, spans)]).view(q.shape[0], -1)
    gate = (torch.randn(q.shape[0], H * D + 8, generator=g) * 2).to(dt).to(dev)[:, :H * D]
    qlens = [e - a for a, e in spans]
    out = ops.attn_prefill(q, kc, vc, i32(np.cumsum([0] + qlens), dev), i32([e for _, e in spans], dev), bt, scale,
                           tiles=ops.prefill_tiles(qlens, dev), sigmoid_bias=pb.to(dev), chunk=chunk, gate=gate)
    want = want * oracle.sigmoid(gate.cpu().double())
    err = (out.cpu().double().view(q.shape[0], -1) - want).norm(dim=-1) / want.norm(dim=-1)
    assert float(err.max()) < 1.5e-2, (int(err.argmax()), float(err.max()))


@pytest.mark.gpu
@pytest.mark.parametrize("window,chunk", [(40, 0), (130, 0), (0, 100)])
def test_softmax_kernels_start_at_the_first_visible_key(window, chunk):
    """The decode and prefill kernels skip what lies before the window or the chunk; softmax weights as attn_mix gives them."""
    dev, dt, BS, H, G, D = "cuda:0", torch.bfloat16, 32, 4, 2, 128
    lens = [1, 39, 40, 41, 101, 300, 700]
    seqs = attention_case(H, G, D, lens, 0, [0, 60, 299, 560, 600, 659], 5)
    nb = sum(-(-n // BS) for n in lens) + 2
    kc, vc, bt = paged([s[1] for s in seqs], [s[2] for s in seqs], np.random.default_rng(3).permutation(nb), BS, nb, dt, dev)
    q = torch.stack([s[0][-1] for s in seqs]).to(device=dev, dtype=dt)
    r = torch.arange(len(lens), dtype=torch.int32, device=dev)
    want = ops.attn_mix(q.view(len(lens), -1), kc, vc, r, i32([n - 1 for n in lens], dev), bt, H, 0.05, window=window, chunk=chunk)
    out = ops.attn_decode(q, kc, vc, bt, i32(lens, dev), 0.05, 700, window=window, chunk=chunk)
    assert rel(out.view(len(lens), -1), want) < 1e-2
    k = 6
    qp = seqs[k][0][500:].to(device=dev, dtype=dt)
    want = ops.attn_mix(qp.view(200, -1), kc, vc, i32([k] * 200, dev), i32(range(500, 700), dev), bt, H, 0.05, window=window, chunk=chunk)
    out = ops.attn_prefill(qp, kc, vc, i32([0, 200], dev), i32([700], dev), bt[k:k + 1].contiguous(), 0.05,
                           tiles=ops.prefill_tiles([200], dev), window=window, chunk=chunk)
    assert rel(out.view(200, -1), want) < 1e-2


# ------------------------------------------------------------------------------------------- mixers alone
def build(layer, D, tmp_path, device, dtype, seed=0, edit=None):
    """A one-layer checkpoint and its model: (model, the layer's config, float64 weights)."""
    cfg = config([layer], 11, D, 1)
    W = make_weights(cfg, seed)
    if edit:
        edit(W)
    path = str(tmp_path / f"m{seed}")
    write_checkpoint(path, cfg, W)
    return DobelixModel(open_model(path), torch.device(device), dtype=getattr(torch, dtype)), layer, {k: v.double() for k, v in W.items()}


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
            row_seq, cu_q, tiles = model._single_rows(1)
            tile_rows, splits = (1 if (not model.f32 and dev.type == "cuda") else 0), 2
        else:
            fb.cu_q, fb.ctx_lens, fb.row_seq, fb.max_q = i32([0, c], dev), i32([at + c], dev), i32([0] * c, dev), c
            tiles, tile_rows = model.prefill_tiles([c], dev)
            row_seq, cu_q, splits = fb.row_seq, fb.cu_q, 1
        x = h[at:at + c].to(model.dtype).to(dev).contiguous()
        if m.kind == "lightning":
            a = model._lightning(L, m, x, fb, kv, 0, cu_q)
        else:
            a = model._attention(L, m, x, fb, kv, 0, row_seq, cu_q, tiles, tile_rows, splits)
        outs.append(model._dense(ops.linear(a, L.wo)).float().cpu())
        at += c
    return torch.cat(outs, 0)


def check_mixer(model, layer, W, h, cuts_list, bs, nblocks, dtype, tables=None):
    want = oracle.MIXERS[layer["type"]](W, "l0.mix.", layer["mixer"], h.double(), 1e-5)
    kv = model.new_kv_cache(nblocks, bs, state_slots=3)
    T = h.shape[0]
    for n, cuts in enumerate(cuts_list):
        # pages in another order every time, slots in turn: leftovers of the run before lie in both
        table = tables[n] if tables else [int(b) for b in np.random.default_rng(n).permutation(nblocks)[:-(-T // bs)]]
        got = run_mixer(model, kv, table, n % 3, h, cuts, bs)
        err = (got.double() - want).norm(dim=-1) / want.norm(dim=-1).clamp_min(1e-9)
        where = (n, int(err.argmax()), float(err.max()), float(err.median()))
        assert float(err.max()) < (1e-4 if dtype == "float32" else 0.1) and float(err.median()) < (3e-5 if dtype == "float32" else 2e-2), where


def inputs(T, D, seed, hot=()):
    """Rows of unit size; the rows listed in `hot` tower over the others."""
    g = torch.Generator().manual_seed(seed)
    h = torch.randn(T, D, generator=g)
    for t in hot:
        h[t] = h[t] * 12
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
@pytest.mark.parametrize("spec", [dict(heads=3, dim=8, vdim=6), dict(heads=1, dim=5, vdim=7, decay=[1.0]),
                                  dict(heads=2, dim=64, vdim=64, decay=[0.2, 0.999]), dict(heads=5, dim=40, vdim=72),
                                  dict(heads=1, dim=200, vdim=16), dict(heads=8, dim=16, vdim=8), dict(heads=4, dim=128, vdim=130)])
def test_lightning_alone(tmp_path, device, dtype, spec):
    """Whole, in portions down to two rows and one, token by token; hot rows whose write every later read-out sees."""
    model, layer, W = build(ff(lightning(**spec), 0), 32, tmp_path, device, dtype)
    T = 45
    h = inputs(T, 32, 1, hot=(0, 17))
    check_mixer(model, layer, W, h, [[T], cuts_of(T, 2), cuts_of(T, 1), cuts_of(T, 7, 1, 2, 16), [30] + [1] * 15], 16, 6, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_lightning_long_rows_in_segments(tmp_path, device, dtype):
    """1100 rows in one portion (scanned in segments on the GPU), then portions and single rows from the slot; a head
    that forgets nothing, one that forgets at once, the state of a slot taken over from another sequence."""
    model, layer, W = build(ff(lightning(heads=4, dim=24, vdim=64, decay=[1.0, 0.05, 0.999, 0.9]), 0), 40, tmp_path, device, dtype)
    T = 1160
    h = inputs(T, 40, 6, hot=(0, 500))
    check_mixer(model, layer, W, h, [[1100, 30, 2, 1, 1] + [13, 13], [T], [600, 560]], 16, 80, dtype,
                tables=[list(range(73)), list(range(79, 6, -1)), list(range(73))])


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("spec", [dict(chunk=12), dict(heads=3, kv=1, dim=10, rot=2, chunk=33), dict(heads=5, kv=5, dim=7, rot=6, chunk=1),
                                  dict(heads=4, kv=2, dim=64, rot=32, chunk=24), dict(heads=8, kv=2, dim=64, rot=64, chunk=17),
                                  dict(heads=2, kv=2, dim=32, rot=16, chunk=0), dict(heads=4, kv=1, dim=128, rot=64, chunk=40),
                                  dict(heads=6, kv=3, dim=96, rot=96, chunk=19), dict(heads=2, kv=2, dim=80, rot=40, chunk=70),
                                  dict(heads=36, kv=4, dim=32, rot=32, chunk=25), dict(heads=17, kv=1, dim=64, rot=8, chunk=48)])
def test_attention_alone(tmp_path, device, dtype, spec):
    """Towering values (the raw keys) at both ends of the chunks, at page borders and far back; portions, decode
    rows (the split-KV decode kernel where the widths allow, more than 16 heads a group and more than 32 heads elsewhere)."""
    model, layer, W = build(ff(attention(**spec), 0), 32, tmp_path, device, dtype)
    c = spec.get("chunk") or 1000
    T = 100
    h = inputs(T, 32, 4, hot=hots(c, T)[:12])
    cuts = [[T], cuts_of(T, 2), ([c - 1, 1, 1, 1] if 1 < c < 90 else [50, 1]), [40] + [1] * 60]
    cuts[2] = cuts[2] + cuts_of(T - sum(cuts[2]), 9, 1)
    check_mixer(model, layer, W, h, cuts, 16, 8, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_a_far_key_among_hundreds(tmp_path, device, dtype):
    """Heads whose bias hides nearly every key (weights of some 1e-3) and one query-key direction that stands out, 280
    rows back within the same chunk and just across a chunk's edge."""
    def edit(W):
        W["l0.mix.pb"][:] = -7.0
        W["l0.mix.temp"][:] = 3.0
    model, layer, W = build(ff(attention(heads=4, kv=2, dim=16, rot=4, chunk=290, scale=1.0), 0), 32, tmp_path, device, dtype, edit=edit)
    T = 310
    h = inputs(T, 32, 9)
    h[285] = h[289] = h[5] * 1.5       # the queries at 285 and 289 meet the key at 5 ...
    h[295] = h[5] * 1.5                # ... the one at 295 is in the next chunk
    check_mixer(model, layer, W, h, [[T], [280] + [1] * 30, cuts_of(T, 77, 2)], 16, 24, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("n", [13, 40, 512])
def test_feed_forward_alone(tmp_path, device, dtype, n):
    model, layer, W = build(ff(lightning(), n), 32, tmp_path, device, dtype)
    L = model.layers[0]
    h = inputs(12, 32, 8)
    want = oracle.dense_ff(W, "l0.mlp.", h.double())
    y = ops.linear(ops.glu_act(ops.linear(h.to(model.dtype).to(device), L.gate_up), n, ops.ACT_GEGLU, model.dtype), L.down)
    assert rel(model._dense(y).float(), want) < (1e-5 if dtype == "float32" else 3e-2)
