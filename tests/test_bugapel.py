"""Bugapel through the framework (reader, model class, K/V pools, recurrent state slots, native scheduler, schedule replay, generation) against the plain oracle of
tests/bugapel_oracle.py.

Every test builds its own small random checkpoint.  The CPU runs use the operator layer's PyTorch
paths; the `gpu` runs put the same engine on the HIP kernels, in bf16 and in fp32.
"""
import json
import os

import numpy as np
import pytest
import torch

import bugapel_oracle as oracle
from localai_amd.engine.llm_engine import EngineConfig, LLMEngine
from localai_amd.engine.sampling_params import SamplingParams

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
MODES = [("cpu", "float32"), ("cpu", "bfloat16"),
         pytest.param("cuda:0", "float32", marks=pytest.mark.gpu), pytest.param("cuda:0", "bfloat16", marks=pytest.mark.gpu)]


def gla(heads=3, dim=8, vdim=6, tau=16.0, rank=4):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}, "rank": rank}


SCALING = {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 24}


def attention(heads=4, kv=2, dim=12, vdim=8, rot=8, base=100.0, scale=0.5, scaling=None):
    r = {"dims": rot, "base": base}
    if scaling:
        r["scaling"] = scaling
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": r}}


def attention_2(heads=4, kv=2, dim=12, vdim=8, rot=8, base=100.0, scale=0.3, window=20, keep=3):
    return {"type": "attention_2", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale,
                                             "rot": {"dims": rot, "base": base}, "mask": {"size": window, "keep_first": keep}}}


def moe(layer, experts=6, top=2, ff=20, groups=3, keep=2, scale=1.5):
    r = {"experts": experts, "top": top, "scale": scale, "groups": {"count": groups, "keep": keep}}
    return dict(layer, mlp={"kind": "moe", "expert": {"ff": ff}, "router": r})


def bare(layer):
    return dict(layer, mlp=None)


def config(layers, vocab, width, streams, eps=1e-5, es=1.5, cap=25.0):
    return {"vocab": vocab, "width": width, "norm": {"eps": eps}, "streams": streams, "embedding": {"scale": es},
            "logit_softcap": cap, "layers": layers}


# layer orders and sizes unlike one another: every mixer first, last and alone, 1 to 5 streams, windows shorter than a
# page / several pages / odd / longer than the prompts, kept tokens 0 / 1 / a few / more than a page, kv heads 1 /
# several / = heads, rotation over a part / the whole / none of a head, scaled frequencies of all three ranges and
# unscaled ones, key widths above, below and equal to value widths, decays that forget at once (small tau) and
# hardly at all, ranks 1 and others, one group, one kept group, all groups kept, top 1, layers without a feed-forward
CONFIGS = {
    "small": config([moe(gla()), moe(attention(scaling=SCALING)), moe(attention_2()), bare(gla(heads=2, dim=10, vdim=14, tau=1.0)),
                     moe(attention_2(heads=3, kv=3, dim=8, vdim=10, rot=8, window=7, keep=5), top=1, keep=1)], 61, 48, 2),
    "varied": config([moe(attention(heads=6, kv=1, dim=10, vdim=10, rot=4, base=10000.0, scale=1.0), experts=5, top=3, ff=24, groups=1,
                          keep=1, scale=1.0),
                      bare(attention_2(heads=2, kv=1, dim=6, vdim=12, rot=6, window=33, keep=0)),
                      moe(gla(heads=5, dim=4, vdim=12, tau=0.5, rank=1), experts=8, top=4, groups=4, keep=3, scale=0.7),
                      bare(attention_2(heads=4, kv=4, dim=14, vdim=4, rot=0, window=200, keep=1)),
                      bare(attention(heads=2, kv=2, dim=16, vdim=6, rot=16, scaling=dict(SCALING, factor=8.0, original=60)))],
                     83, 40, 3, eps=1e-6, es=3.0, cap=0.0),
    "scan": config([moe(gla(heads=1, dim=16, vdim=4, tau=8.0), experts=2, top=2, groups=2, keep=2), bare(gla(heads=4, dim=6, vdim=6, tau=64.0))],
                   50, 32, 1, es=1.0),
    # sizes no vector load likes (odd width, odd head widths and counts)
    "odd": config([moe(attention(heads=5, kv=5, dim=7, vdim=5, rot=2), ff=13, scale=2.0), moe(gla(heads=3, dim=5, vdim=7, rank=3), ff=17),
                   bare(attention_2(heads=3, kv=1, dim=9, vdim=11, rot=6, window=18, keep=17))], 51, 35, 5, eps=1e-6),
    # widths the GPU's specialised paths take: split-KV decode and prefill kernels, matrix-core tiles, the vectorised
    # page append, the grouped expert GEMMs, several blocks of key channels
    "wide": config([moe(attention(heads=8, kv=2, dim=64, vdim=64, rot=32, scale=0.12, scaling=SCALING), ff=256),
                    moe(attention_2(heads=4, kv=1, dim=128, vdim=128, rot=128, scale=0.1, window=37, keep=4), ff=256, groups=1, keep=1),
                    bare(gla(heads=4, dim=64, vdim=96, rank=16)), moe(gla(heads=2, dim=80, vdim=32, rank=8), ff=64),
                    bare(attention_2(heads=4, kv=2, dim=32, vdim=64, rot=32, scale=0.2, window=24, keep=20)),
                    moe(attention(heads=4, kv=4, dim=96, vdim=32, rot=96, scale=0.1), ff=256)], 97, 256, 2),
}


def make_weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    D, n = cfg["width"], cfg["streams"]

    def rnd(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(torch.bfloat16)

    def lin(n, k, s=1.0):
        return rnd(n, k, s=s * k ** -0.5)

    def norm(W, name, n):
        W[name] = (1.0 + 0.2 * torch.randn(n, generator=g)).to(torch.bfloat16)

    W = {"embed": rnd(cfg["vocab"], D, s=0.7)}
    norm(W, "final.norm", D)
    W["final.norm.b"] = rnd(D, s=0.2)
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", L["mixer"]
        for q in (1, 2) if L["mlp"] else (1,):
            norm(W, f"l{i}.norm{q}", D)
            W[f"l{i}.norm{q}.b"] = rnd(D, s=0.2)
            h = f"l{i}.hc{q}."
            W[h + "in"] = (1.0 / n + 0.15 / n * torch.randn(n, generator=g)).to(torch.bfloat16)
            W[h + "out"] = (0.7 + 0.2 * torch.randn(n, generator=g)).to(torch.bfloat16)
            W[h + "mix"] = (0.8 * torch.eye(n) + 0.2 / n + 0.1 * torch.randn(n, n, generator=g)).to(torch.bfloat16)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        W[p + "q"], W[p + "o"] = lin(H * d, D), lin(D, H * dv)
        if L["type"] == "gla":
            W[p + "k"], W[p + "v"], W[p + "g"] = lin(H * d, D), lin(H * dv, D), lin(H * dv, D, 2.0)
            W[p + "a1"], W[p + "a2"] = lin(L["rank"], D), lin(H * d, L["rank"], 2.0)
            W[p + "a2.b"] = rnd(H * d)
            norm(W, p + "norm", dv)
        else:
            G = m["kv_heads"]
            W[p + "k"], W[p + "v"] = lin(G * d, D), lin(G * dv, D)
            if L["type"] == "attention_2":
                for t, k in (("q", H * d), ("k", G * d), ("v", G * dv), ("o", D)):
                    W[f"{p}{t}.b"] = rnd(k, s=0.5)
        if L["mlp"]:
            p, f, E = f"l{i}.mlp.", L["mlp"]["expert"]["ff"], L["mlp"]["router"]["experts"]
            W[p + "router"] = lin(E, D, 2.0)
            for e in range(E):
                W[p + f"e{e}.up"], W[p + f"e{e}.down"] = lin(f, D, 0.8), lin(D, f, 1.2)
    return W


def config_file(cfg):
    """What config.json holds (the tests' layer entries also carry the decay rank, which tensors give)."""
    return dict(cfg, layers=[{k: v for k, v in L.items() if k != "rank"} for L in cfg["layers"]])


def write_checkpoint(path, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(dict(config_file(cfg), architecture="Bugapel"), f)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))


_CKPT = {}


@pytest.fixture(scope="module")
def ckpt(tmp_path_factory):
    def get(name, seed=0):
        key = (name, seed)
        if key not in _CKPT:
            cfg = CONFIGS[name]
            W = make_weights(cfg, seed)
            path = str(tmp_path_factory.mktemp(f"bugapel_{name}_{seed}"))
            write_checkpoint(path, cfg, W)
            _CKPT[key] = (path, cfg, {k: v.double() for k, v in W.items()})
        return _CKPT[key]
    return get


def engine(path, device, dtype="float32", tokens=256, slots=4, bs=16, graphs=False):
    return LLMEngine(EngineConfig(model_path=path, device=device, context_size=tokens, max_num_seqs=slots,
                                  max_batched_tokens=tokens, block_size=bs, max_kv_tokens=tokens, kv_pool_exact=True,
                                  use_graphs=graphs, dtype=dtype, state_slots=slots, record_tokens=True))


MARGIN = 0.08     # of router logits: below it 16-bit rounding may choose other experts than the oracle


class Want:
    """The oracle's logits of a sequence and, per position, its smallest router margin."""

    def __init__(self, logits, margins):
        self.logits, self.margins = logits, torch.as_tensor(margins, dtype=torch.float64)

    def __getitem__(self, idx):
        return Want(self.logits[idx], self.margins[idx])


def close(got, want, dtype):
    """Every position, its mean taken off, in units of the wanted logits' spread.  fp32: to rounding.  bf16: to 16-bit
    rounding; a position whose routing is a close call, or that of one of the 6 before it (whose change it reads),
    counts in the median only, and of the others one in ten may stand out."""
    got, logits = got.detach().double().cpu(), want.logits.double()
    d = got - logits
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / logits.std(-1).clamp_min(1e-6)
    if dtype == "float32":
        assert float(err.max()) < 4e-4 and float(err.median()) < 1e-5, (int(err.argmax()), float(err.max()), float(err.median()))
        return
    m = want.margins
    sure = err[torch.stack([m[max(0, t - 6):t + 1].min() for t in range(m.shape[0])]) > MARGIN]
    out = int((sure > 0.12).sum())
    assert out <= max(1, sure.numel() // 10) and (err.numel() < 10 or float(err.median()) < 0.04), (out, sure.numel(), float(err.max()), float(err.median()))


def portions(n, sizes):
    out, i, k = [], 0, 0
    while i < n:
        s = min(sizes[k % len(sizes)], n - i)
        out.append(s)
        i += s
        k += 1
    return out


def replay_alone(eng, rid, toks, cuts):
    """Feed `toks` in the given portion sizes; logits of every position."""
    rows, i = [], 0
    for c in cuts:
        rows.append(eng.replay_step([(rid, toks[i:i + c], list(range(c)))], [rid] if i + c == len(toks) else []))
        i += c
    return torch.cat(rows, 0)


def rand_tokens(cfg, n, seed):
    return np.random.default_rng(seed).integers(0, cfg["vocab"], size=n).tolist()


_ORACLE = {}


def fwd(cfg, W, toks):
    """The oracle on one sequence (kept per configuration and token list: several tests ask for the same)."""
    key = (json.dumps(cfg, sort_keys=True), tuple(toks))
    if key not in _ORACLE:
        margins = [float("inf")] * len(toks)
        _ORACLE[key] = Want(oracle.forward(cfg, W, toks, margins=margins), margins)
    return _ORACLE[key]


def skip_slow_cpu(name, device, dtype, whole=False):
    """The configuration made for the GPU's specialised paths is slow on the CPU: it runs there once, as a whole prompt in fp32."""
    if name == "wide" and device == "cpu" and not (whole and dtype == "float32"):
        pytest.skip("the wide configuration runs on the GPU")


# --------------------------------------------------------------------------------------- whole prompts
@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_matches_oracle(ckpt, name, device, dtype):
    skip_slow_cpu(name, device, dtype, whole=True)
    path, cfg, W = ckpt(name)
    toks = rand_tokens(cfg, 75, 1)            # past most windows, pages of 16
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype)
    close(replay_alone(eng, 1, toks, [len(toks)]), want, dtype)
    # the very first tokens: a one-token prompt, then two (zero state)
    close(replay_alone(eng, 2, toks[:1], [1]), want[:1], dtype)
    close(replay_alone(eng, 3, toks[:2], [2]), want[:2], dtype)


@pytest.mark.parametrize("device", DEVICES)
@pytest.mark.parametrize("name", ["small", "varied", "odd", "wide"])
def test_residual_stream_after_every_layer(ckpt, name, device):
    skip_slow_cpu(name, device, "float32")
    from localai_amd.models.decoder import ForwardBatch
    path, cfg, W = ckpt(name)
    toks = rand_tokens(cfg, 29, 2)
    want, got = [], []
    oracle.forward(cfg, W, toks, want)
    eng = engine(path, device, "float32")
    eng.sched.add(1, toks, 0)
    plan = eng.sched.schedule_explicit([(1, len(toks))])
    fb = ForwardBatch(tokens=eng._dev(plan["p_tokens"]), pos=eng._dev(plan["p_pos"]), slots=eng._dev(plan["p_slots"]),
                      decode=False, block_tables=eng._dev(plan["p_bt"]), cu_q=eng._dev(plan["p_cu"]),
                      ctx_lens=eng._dev(plan["p_ctx"]), sslots=eng._dev(plan["p_sslot"]),
                      row_seq=eng._dev(np.zeros(len(toks), dtype=np.int32)))
    eng.model.forward(fb, eng.kv, layer_out=got)
    assert len(got) == len(want) == len(cfg["layers"])
    for a, b in zip(got, want):
        assert float((a.cpu() - b).abs().max()) < 1e-4 * max(1.0, float(b.abs().max()))


# --------------------------------------------------------------------------------------- portions, decoding
@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_portions_and_token_by_token_decoding(ckpt, name, device, dtype):
    skip_slow_cpu(name, device, dtype)
    path, cfg, W = ckpt(name)
    toks = rand_tokens(cfg, 75, 1)
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype)
    # cuts in the middle of pages, windows and chunks of 16 tokens, at their edges, and single tokens throughout
    for rid, cuts in enumerate([portions(75, [2]), portions(75, [5, 2, 17, 3, 31]), portions(75, [34, 1, 1, 7]),
                                [25] + [1] * 50, [1] * 75, portions(75, [20, 13, 7, 10])], 1):
        close(replay_alone(eng, rid, toks, cuts), want, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_long_decoding_over_windows_and_pages(ckpt, device, dtype):
    path, cfg, W = ckpt("small")
    toks = rand_tokens(cfg, 170, 4)           # windows of 20 and 7, pages of 16
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype)
    close(replay_alone(eng, 1, toks, [10] + [1] * 160), want, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_long_prompt_then_decoding(ckpt, device, dtype):
    """600 tokens in one step (37 chunks and a half of the recurrence), then decoding."""
    path, cfg, W = ckpt("scan")
    toks = rand_tokens(cfg, 610, 6)
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype, tokens=640)
    close(replay_alone(eng, 1, toks, [600] + [1] * 10), want, dtype)


# --------------------------------------------------------------------------------------- batches, reuse
@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches_of_unequal_requests_with_page_and_slot_reuse(ckpt, name, device, dtype):
    """Four live requests at most in a pool of 160 tokens with 4 state slots, ten requests in all:
    portions of some beside single tokens of others, every finished request's pages and slot taken
    over by the next (whose recurrent state must start from zero, not from the leftovers).  Every position must equal the request run alone (the oracle)."""
    skip_slow_cpu(name, device, dtype)
    path, cfg, W = ckpt(name)
    rng = np.random.default_rng(5)
    lens = [33, 7, 48, 2, 21, 40, 1, 17, 30, 9]
    reqs = {i + 1: rand_tokens(cfg, n, 100 + i) for i, n in enumerate(lens)}
    want = {i: fwd(cfg, W, t) for i, t in reqs.items()}
    eng = engine(path, device, dtype, tokens=160, slots=4, bs=16)
    pending = list(reqs)
    live, at = [], {}
    got = {i: [] for i in reqs}
    while pending or live:
        while pending and len(live) < 4 and sum(-(-len(reqs[i]) // 16) * 16 for i in live + pending[:1]) <= 160:
            live.append(pending.pop(0))
            at[live[-1]] = 0
        entries = []
        for i in live:
            if rng.random() < 0.2 and len(live) > 1:
                continue                       # rests this step
            left = len(reqs[i]) - at[i]
            n = min(left, int(rng.choice([1, 1, 2, 3, 8, 19])))
            entries.append((i, reqs[i][at[i]:at[i] + n], list(range(n))))
        if not entries:
            continue
        end = [i for i, t, _ in entries if at[i] + len(t) == len(reqs[i])]
        lg = eng.replay_step(entries, end)
        o = 0
        for i, t, _ in entries:
            got[i].append(lg[o:o + len(t)])
            o += len(t)
            at[i] += len(t)
        for i in end:
            live.remove(i)
    assert eng.sched.num_free_state_slots == 4 and eng.sched.blocks().num_free == 10
    for i in reqs:
        close(torch.cat(got[i], 0), want[i], dtype)


@pytest.mark.parametrize("device", DEVICES)
def test_pools_follow_the_layers(ckpt, device):
    """A gla layer holds an fp32 state per slot, an attention layer K / V pages of the serving dtype and its widths."""
    path, cfg, W = ckpt("small")
    kv = engine(path, device, "bfloat16", tokens=64, slots=2, bs=16).kv
    assert len(kv.k) == len(kv.state) == 5
    for i, (shape, G, dk, dv) in enumerate([((2, 3, 6, 8), 0, 0, 0), (None, 2, 12, 8), (None, 2, 12, 8), ((2, 2, 14, 10), 0, 0, 0),
                                            (None, 3, 8, 10)]):
        if shape:
            assert kv.k[i] is None and kv.state[i][0].dtype == torch.float32 and tuple(kv.state[i][0].shape) == shape
        else:
            assert kv.state[i] is None and kv.k[i].dtype == torch.bfloat16
            assert tuple(kv.k[i].shape[1:]) == (G, 16, dk) and tuple(kv.v[i].shape[1:]) == (G, 2, dv, 8)


# --------------------------------------------------------------------------------------- generation
@pytest.mark.parametrize("device,dtype,graphs,name", [
    ("cpu", "float32", False, "small"),
    pytest.param("cuda:0", "float32", False, "small", marks=pytest.mark.gpu),
    pytest.param("cuda:0", "bfloat16", True, "small", marks=pytest.mark.gpu),
    pytest.param("cuda:0", "float32", True, "varied", marks=pytest.mark.gpu),
    pytest.param("cuda:0", "bfloat16", True, "odd", marks=pytest.mark.gpu),
    pytest.param("cuda:0", "bfloat16", True, "wide", marks=pytest.mark.gpu),
    pytest.param("cuda:0", "bfloat16", False, "wide", marks=pytest.mark.gpu)])
def test_greedy_generation_through_the_engine(ckpt, device, dtype, graphs, name):
    """engine.add_request / step: scheduler-planned chunked prefill, (graph-replayed multi-step)
    decode with the device sampler, several requests at once; every emitted token is the oracle's
    argmax at its position unless the oracle's top-2 margin is within rounding."""
    path, cfg, W = ckpt(name)
    eng = LLMEngine(EngineConfig(model_path=path, device=device, context_size=128, max_num_seqs=4,
                                 max_batched_tokens=24, block_size=16, use_graphs=graphs, dtype=dtype,
                                 record_tokens=True, decode_steps=4, decode_steps_wide=4))
    prompts = [rand_tokens(cfg, n, 200 + n) for n in (5, 30, 47)]
    done = {}
    for k, p in enumerate(prompts):
        def cb(ev, k=k):
            if ev.finished:
                done[k] = ev
        eng.add_request(p, SamplingParams(max_tokens=20, temperature=0.0, ignore_eos=True), cb)
    for _ in range(400):
        if len(done) == len(prompts):
            break
        eng.step()
    assert len(done) == len(prompts)
    for k, p in enumerate(prompts):
        gen = done[k].token_ids
        assert len(gen) == 20
        ref = fwd(cfg, W, p + gen[:-1])
        for j, t in enumerate(gen):
            row = ref.logits[len(p) - 1 + j]
            if dtype != "float32" and float(ref.margins[:len(p) + j].min()) < 0.02:
                break       # a very close router call upstream: from here on the oracle may follow other experts
            margin_ok = (1e-3 if dtype == "float32" else 0.3) * float(row.std())
            assert t == int(row.argmax()) or float(row.max() - row[t]) <= margin_ok, (k, j)
    assert eng.sched.num_free_state_slots == 4


def test_registry_reader_and_configuration(ckpt):
    from localai_amd.models import model_class
    from localai_amd.models.bugapel import BugapelModel
    from localai_amd.models.hf_checkpoint import open_model
    path, cfg, W = ckpt("varied")
    r = open_model(path)
    assert r.architecture == "bugapel" and model_class(r.architecture) is BugapelModel
    m = BugapelModel(r, torch.device("cpu"), dtype=torch.float32)
    hp = m.hp
    assert [x.kind for x in hp.mixers] == ["attention", "attention_2", "gla", "attention_2", "attention"]
    assert (hp.streams, hp.embed_scale, hp.logit_softcap, hp.norm_eps) == (3, 3.0, 0.0, 1e-6)
    a, b, c, d, e = hp.mixers
    assert (a.heads, a.kv_heads, a.dim, a.rot_dims, a.rot_base, a.rot_scaling, a.scale) == (6, 1, 10, 4, 10000.0, None, 1.0)
    assert (b.window, b.keep, d.window, d.keep, d.rot_dims, c.tau, c.vdim, e.rot_scaling["factor"]) == (33, 0, 200, 1, 0, 0.5, 12, 8.0)
    f = hp.mlps[2]
    assert hp.mlps[1] is None and (f.experts, f.top, f.groups, f.keep, f.scale, f.ff) == (8, 4, 4, 3, 0.7, 20)
    assert m.layers[1].experts is None and m.layers[2].rank == 1
    assert m.kv_bytes_per_token() == 4 * (10 + 10 + 6 + 12 + 4 * (14 + 4) + 2 * (16 + 6))
    L = config_file(cfg)["layers"]
    mix = lambda k, **kw: dict(L[k], mixer=dict(L[k]["mixer"], **kw))  # noqa: E731
    few = dict(L[2]["mlp"], router=dict(L[2]["mlp"]["router"], top=7))     # three groups of two hold six
    for bad in (dict(L[0], type="retention"), mix(0, kv_heads=4), mix(0, rot={"dims": 12, "base": 10.0}), mix(2, tau=0.0),
                dict(L[0], mlp={"kind": "dense", "ff": 8}), dict(L[2], mlp=few)):
        with pytest.raises(ValueError):
            type(hp).from_config(dict(cfg, layers=[bad]))
    with pytest.raises(ValueError):
        type(hp).from_config(dict(config_file(cfg), streams=17))
    with pytest.raises(ValueError):      # tensors that do not fit the configuration
        BugapelModel(_Reader(dict(config_file(cfg), width=48), r), torch.device("cpu"))


class _Reader:
    def __init__(self, config, r):
        self.config, self.kv, self.tensors = config, r.kv, r.tensors


def test_trace_runner_cli(ckpt, tmp_path):
    """The schedule replay program end to end on the CPU: two requests, a rest, a reused name."""
    import subprocess
    import sys
    path, cfg, W = ckpt("small")
    a, b = rand_tokens(cfg, 30, 7), rand_tokens(cfg, 9, 8)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:21], "want": [0, 20]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[21:23], "want": []}, {"id": "b", "tokens": b, "want": [8]}],
              "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[23:], "want": [6]}, {"id": "b", "tokens": a[:3], "want": [2]}],
              "end": ["a", "b"]}]
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", path, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "64", "--device", "cpu"],
                       input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    wa, wb = fwd(cfg, W, a), fwd(cfg, W, b)
    g = [torch.from_numpy(np.fromfile(out / f"{k}.f32", dtype="<f4").reshape(-1, cfg["vocab"])) for k in range(3)]
    close(g[0], wa[[0, 20]], "float32")
    close(g[1], wb[[8]], "float32")
    close(g[2], wa[[29, 2]], "float32")


def test_backend_service_loads_and_generates(ckpt, monkeypatch):
    """The gRPC backend servicer (what the gateway talks to): LoadModel on the checkpoint directory,
    Predict with a numeric prompt; greedy tokens follow the oracle."""
    import asyncio
    from localai_amd.grpc import backend_pb as pb
    from localai_amd.grpc.servicer import EngineServicer
    monkeypatch.setenv("LOCALAI_MAX_NUM_SEQS", "4")
    path, cfg, W = ckpt("small")
    prompt = [3, 17, 5, 9, 30]

    async def run():
        sv = EngineServicer(device="cpu")
        r = await sv.LoadModel(pb.ModelOptions(ModelFile=path, ContextSize=64))
        assert r.success, r.message
        return await sv.Predict(pb.PredictOptions(Prompt=" ".join(str(t) for t in prompt), Tokens=5, Temperature=0.0,
                                                  IgnoreEOS=True))
    rep = asyncio.run(run())
    gen = [int(x) for x in rep.message.decode().strip("<>").split("><")]
    assert rep.tokens == 5 and rep.prompt_tokens == len(prompt) and len(gen) == 5
    ref = fwd(cfg, W, prompt + gen[:-1])
    for j, t in enumerate(gen):
        row = ref.logits[len(prompt) - 1 + j]
        assert float(row.max() - row[t]) <= 0.3 * float(row.std()), j       # served in bf16 by default
