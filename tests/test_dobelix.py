"""Dobelix through the framework (reader, model class, K/V pools, convolution tails and recurrent state
slots, native scheduler, schedule replay, generation) against the plain oracle of
tests/dobelix_oracle.py.

Every test builds its own small random checkpoint.  The CPU runs use the operator layer's PyTorch
paths; the `gpu` runs put the same engine on the HIP kernels, in bf16 and in fp32.
"""
import json
import os

import numpy as np
import pytest
import torch

import dobelix_oracle as oracle
from localai_amd.engine.llm_engine import EngineConfig, LLMEngine
from localai_amd.engine.sampling_params import SamplingParams

DEVICES = ["cpu", pytest.param("cuda:0", marks=pytest.mark.gpu)]
MODES = [("cpu", "float32"), ("cpu", "bfloat16"),
         pytest.param("cuda:0", "float32", marks=pytest.mark.gpu), pytest.param("cuda:0", "bfloat16", marks=pytest.mark.gpu)]


def lightning(heads=3, dim=8, vdim=6, decay=None):
    decay = decay or [0.55 + 0.44 * (i + 1) / (heads + 1) for i in range(heads)]
    return {"type": "lightning", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "decay": decay}}


def attention(heads=4, kv=2, dim=12, rot=8, chunk=20, base=100.0, scale=0.4):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "rot": {"dims": rot, "base": base}}
    if chunk:
        m["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": m}


def ff(layer, n=40):
    return dict(layer, mlp={"kind": "dense", "ff": n} if n else None)


def config(layers, vocab, width, taps, eps=1e-5, es=1.5, ls=0.8):
    return {"vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps}, "embedding": {"scale": es},
            "logit_scale": ls, "layers": layers}


# layer orders and sizes unlike one another: either mixer first and last, one mixer only, 1 to 5 taps, chunks
# shorter than a page / several pages / odd / longer than the prompts / none, kv heads 1 / several / = heads,
# rotation over a part / the whole / none of a head, key width of lightning heads above and below the value
# width, one head, a head that forgets nothing, layers without a feed-forward, scales 1 and others
CONFIGS = {
    "small": config([ff(lightning()), ff(attention()), ff(lightning(heads=2, dim=10, vdim=14, decay=[1.0, 0.3]), 0),
                     ff(attention(heads=3, kv=3, dim=8, rot=8, chunk=7))], 61, 48, 4),
    "varied": config([ff(attention(heads=6, kv=1, dim=10, rot=4, chunk=33, base=10000.0, scale=1.0), 24),
                      ff(attention(heads=2, kv=1, dim=6, rot=6, chunk=0), 0),
                      ff(lightning(heads=5, dim=4, vdim=12), 36),
                      ff(attention(heads=4, kv=4, dim=14, rot=0, chunk=200), 28)], 83, 40, 1, eps=1e-6, es=3.0, ls=1.0),
    "scan": config([ff(lightning(heads=1, dim=16, vdim=4, decay=[0.9]), 20), ff(lightning(heads=4, dim=6, vdim=6), 0)], 50, 32, 2,
                   es=1.0, ls=2.5),
    # sizes no vector load likes (odd width, odd head widths and counts)
    "odd": config([ff(attention(heads=5, kv=5, dim=7, rot=2, chunk=13), 30), ff(lightning(heads=3, dim=5, vdim=7), 13),
                   ff(attention(heads=3, kv=1, dim=9, rot=6, chunk=40), 17)], 51, 35, 5, eps=1e-6),
    # widths the GPU's specialised paths take: split-KV decode and prefill kernels, matrix-core tiles, the
    # vectorised page append, GEMM depths % 256, recurrences over several registers and columns a thread
    "wide": config([ff(attention(heads=8, kv=2, dim=64, rot=32, chunk=50, scale=0.3), 512),
                    ff(lightning(heads=4, dim=64, vdim=96), 256),
                    ff(attention(heads=4, kv=4, dim=32, rot=32, chunk=24), 64),
                    ff(lightning(heads=2, dim=128, vdim=32), 0),
                    ff(attention(heads=4, kv=1, dim=128, rot=128, chunk=37, scale=0.2), 256)], 97, 256, 3),
}


def make_weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    D, taps = cfg["width"], cfg["canon"]["taps"]

    def rnd(*shape, s=1.0):
        return (torch.randn(*shape, generator=g) * s).to(torch.bfloat16)

    def lin(n, k, s=1.0):
        return rnd(n, k, s=s * k ** -0.5)

    def norm(n):
        return (1.0 + 0.2 * torch.randn(n, generator=g)).to(torch.bfloat16)

    W = {"embed": rnd(cfg["vocab"], D, s=0.7), "final.norm": norm(D), "head": lin(cfg["vocab"], D)}
    for i, L in enumerate(cfg["layers"]):
        p, m = f"l{i}.mix.", L["mixer"]
        W[f"l{i}.norm1"], W[f"l{i}.canon1"] = norm(D), rnd(D, taps, s=0.5)
        H, d, dv = m["heads"], m["dim"], m["vdim"]
        W[p + "q"], W[p + "g"], W[p + "o"] = lin(H * d, D, 1.5), lin(H * dv, D, 2.0), lin(D, H * dv)
        if L["type"] == "lightning":
            W[p + "k"], W[p + "v"], W[p + "norm"] = lin(H * d, D, 1.5), lin(H * dv, D, 1.5), norm(H * dv)
        else:
            G = m["kv_heads"]
            W[p + "k"] = lin(G * d, D, 1.5)
            W[p + "q.norm"], W[p + "k.norm"] = norm(H * d), norm(G * d)
            W[p + "temp"] = (1.0 + 0.4 * torch.randn(H, generator=g)).to(torch.bfloat16)
            W[p + "pb"] = (-2.5 + 0.5 * torch.randn(H, generator=g)).to(torch.bfloat16)
        if L["mlp"]:
            p, n = f"l{i}.mlp.", L["mlp"]["ff"]
            W[f"l{i}.norm2"] = norm(D)
            W[p + "gate"], W[p + "up"], W[p + "down"] = lin(n, D, 1.5), lin(n, D), lin(D, n)
    return W


def write_checkpoint(path, cfg, W):
    from safetensors.torch import save_file
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(dict(cfg, architecture="Dobelix"), f)
    save_file({k: v.contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))


_CKPT = {}


@pytest.fixture(scope="module")
def ckpt(tmp_path_factory):
    def get(name, seed=0):
        key = (name, seed)
        if key not in _CKPT:
            cfg = CONFIGS[name]
            W = make_weights(cfg, seed)
            path = str(tmp_path_factory.mktemp(f"dobelix_{name}_{seed}"))
            write_checkpoint(path, cfg, W)
            _CKPT[key] = (path, cfg, {k: v.double() for k, v in W.items()})
        return _CKPT[key]
    return get


def engine(path, device, dtype="float32", tokens=256, slots=4, bs=16, graphs=False):
    return LLMEngine(EngineConfig(model_path=path, device=device, context_size=tokens, max_num_seqs=slots,
                                  max_batched_tokens=tokens, block_size=bs, max_kv_tokens=tokens, kv_pool_exact=True,
                                  use_graphs=graphs, dtype=dtype, state_slots=slots, record_tokens=True))


def close(got, want, dtype):
    """Every position, its mean taken off, in units of the wanted logits' spread: fp32 to rounding, bf16 to 16-bit rounding."""
    got, want = got.detach().double().cpu(), want.double()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    err = d.pow(2).mean(-1).sqrt() / want.std(-1).clamp_min(1e-6)
    limit = 1e-4 if dtype == "float32" else 0.12
    assert float(err.max()) < limit and float(err.median()) < limit / 3, (int(err.argmax()), float(err.max()), float(err.median()))


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
        _ORACLE[key] = oracle.forward(cfg, W, toks)
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
    toks = rand_tokens(cfg, 75, 1)            # past most chunks, pages of 16
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype)
    close(replay_alone(eng, 1, toks, [len(toks)]), want, dtype)
    # the very first tokens: a one-token prompt, then two (zero state, zeros before the convolution)
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
    # cuts in the middle of pages, chunks and the convolution's reach, at their edges, and single tokens throughout
    for rid, cuts in enumerate([portions(75, [2]), portions(75, [5, 2, 17, 3, 31]), portions(75, [34, 1, 1, 7]),
                                [25] + [1] * 50, [1] * 75, portions(75, [20, 13, 7, 10])], 1):
        close(replay_alone(eng, rid, toks, cuts), want, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_long_decoding_over_chunks_and_pages(ckpt, device, dtype):
    path, cfg, W = ckpt("small")
    toks = rand_tokens(cfg, 170, 4)           # chunks of 20 and 7, pages of 16
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype)
    close(replay_alone(eng, 1, toks, [10] + [1] * 160), want, dtype)


@pytest.mark.parametrize("device,dtype", MODES)
def test_long_prompt_scanned_in_segments(ckpt, device, dtype):
    """1100 tokens in one step (long portions of lightning layers are scanned in segments on the GPU), then decoding."""
    path, cfg, W = ckpt("scan")
    toks = rand_tokens(cfg, 1110, 6)
    want = fwd(cfg, W, toks)
    eng = engine(path, device, dtype, tokens=1152)
    close(replay_alone(eng, 1, toks, [1100] + [1] * 10), want, dtype)


# --------------------------------------------------------------------------------------- batches, reuse
@pytest.mark.parametrize("device,dtype", MODES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_mixed_batches_of_unequal_requests_with_page_and_slot_reuse(ckpt, name, device, dtype):
    """Four live requests at most in a pool of 160 tokens with 4 state slots, ten requests in all:
    portions of some beside single tokens of others, every finished request's pages and slot taken
    over by the next (whose convolution tail and recurrent state must start from zero, not from the
    leftovers).  Every position must equal the request run alone (the oracle)."""
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
    """Every layer holds the stream's convolution tail in fp32, a lightning layer an fp32 state beside it, an
    attention layer K / V pages of the serving dtype."""
    path, cfg, W = ckpt("small")
    kv = engine(path, device, "bfloat16", tokens=64, slots=2, bs=16).kv
    assert len(kv.k) == len(kv.state) == 4
    for i, (shape, G, d) in enumerate([((2, 3, 6, 8), 0, 0), (None, 2, 12), ((2, 2, 14, 10), 0, 0), (None, 3, 8)]):
        tail = kv.state[i][0]
        assert tail.dtype == torch.float32 and tuple(tail.shape) == (2, 3, 48)
        if shape:
            assert kv.k[i] is None and kv.state[i][1].dtype == torch.float32 and tuple(kv.state[i][1].shape) == shape
        else:
            assert len(kv.state[i]) == 1 and kv.k[i].dtype == torch.bfloat16
            assert tuple(kv.k[i].shape[1:]) == (G, 16, d) and tuple(kv.v[i].shape[1:]) == (G, 2, d, 8)


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
            row = ref[len(p) - 1 + j]
            margin_ok = (1e-3 if dtype == "float32" else 0.15) * float(row.std())
            assert t == int(row.argmax()) or float(row.max() - row[t]) <= margin_ok, (k, j)
    assert eng.sched.num_free_state_slots == 4


def test_registry_reader_and_configuration(ckpt):
    from localai_amd.models import model_class
    from localai_amd.models.dobelix import DobelixModel
    from localai_amd.models.hf_checkpoint import open_model
    path, cfg, W = ckpt("varied")
    r = open_model(path)
    assert r.architecture == "dobelix" and model_class(r.architecture) is DobelixModel
    m = DobelixModel(r, torch.device("cpu"), dtype=torch.float32)
    hp = m.hp
    assert [x.kind for x in hp.mixers] == ["attention", "attention", "lightning", "attention"]
    assert (hp.taps, hp.embed_scale, hp.logit_scale, hp.norm_eps) == (1, 3.0, 1.0, 1e-6) and hp.ffs == [24, 0, 36, 28]
    a, b, c, d = hp.mixers
    assert (a.heads, a.kv_heads, a.dim, a.rot_dims, a.rot_base, a.chunk, a.scale) == (6, 1, 10, 4, 10000.0, 33, 1.0)
    assert (b.chunk, d.chunk, d.rot_dims, c.vdim, len(c.decay)) == (0, 200, 0, 12, 5)
    assert m.layers[1].norm2 is None and m.kv_bytes_per_token() == 4 * 2 * (10 + 6 + 4 * 14)
    L = cfg["layers"]
    for bad in (dict(L[0], type="retention"), dict(L[0], mixer=dict(L[0]["mixer"], vdim=12)),
                dict(L[0], mixer=dict(L[0]["mixer"], kv_heads=4)), dict(L[2], mixer=dict(L[2]["mixer"], decay=[0.5])),
                dict(L[0], mlp={"kind": "moe"})):
        with pytest.raises(ValueError):
            type(hp).from_config(dict(cfg, layers=[bad]))
    with pytest.raises(ValueError):      # tensors that do not fit the configuration
        DobelixModel(_Reader(dict(cfg, width=48), r), torch.device("cpu"))


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
    close(g[2], torch.stack([wa[29], wa[2]]), "float32")


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
        row = ref[len(prompt) - 1 + j]
        assert float(row.max() - row[t]) <= 0.15 * float(row.std()), j      # served in bf16 by default
