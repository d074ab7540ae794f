"""Bugapel: a decoder-only design described layer by layer in its config.json.

The residual is kept as n parallel streams (hyper-connections), all equal to the scaled embedding at first.
A sublayer reads a weighted sum of them through a layer norm with weight and bias; its result is added to every
stream while the streams are mixed by an n x n matrix (ops.hyper_streams: exchange, weighted sum and norm of
the next sublayer in one launch).  The output norm reads the plain sum; the embedding table is the head, its
logits soft-capped.  Three mixers:

  * "attention": grouped-query attention, rotate-half positions with wavelength-dependent scaling
    (ops.rot_freqs), then queries and keys over their root mean square per head (ops.head_rope_pages, which
    also appends K / V to the pages); causal softmax with a 1 added to the denominator (a sink logit of 0);
  * "attention_2": projections with biases (added in ops.head_rope_pages and, for the output, in the boundary),
    interleaved rotation, sliding window beside which the first tokens of the sequence stay visible
    (window, keep of the attention kernels);
  * "gla": gated linear attention with one decay per head and key channel from a low-rank projection
    (ops.gla), a unit norm per head and a silu gate; its Dk x Dv state per head is per-sequence fp32 state
    in the scheduler's slot pool.

Feed-forward: routed experts down(max(up h, 0)^2) without gates (layered.RoutedExperts), chosen by softmax scores
within the best groups of neighbouring experts (ops.router_softmax).

bf16 serving keeps the streams, norms, angles, scores and weights, routers, decays and the recurrence with
its state in fp32; dtype=torch.float32 serves in true fp32 end to end.
"""
from __future__ import annotations

import os
from dataclasses import dataclass, field
from typing import List, Optional

import torch

from .. import ops
from .decoder import ForwardBatch, KVCache, TPInfo
from .layered import LayeredModel, RoutedExperts

# decode rows of attention layers outside the split-KV decode kernel's widths: keys dealt to about this many
# workgroups a batch
DECODE_WGS = int(os.environ.get("LOCALAI_AMD_BUGAPEL_DECODE_WGS", "1024"))


@dataclass
class MixSpec:
    kind: str                 # "attention" | "attention_2" | "gla"
    heads: int
    dim: int                  # query / key width per head
    vdim: int
    kv_heads: int = 0         # attention mixers
    scale: float = 1.0
    rot_dims: int = 0
    rot_base: float = 10000.0
    rot_scaling: Optional[dict] = None
    window: int = 0           # keys i - window < j <= i (0: all) ..
    keep: int = 0             # .. and the first `keep`
    tau: float = 1.0          # gla


@dataclass
class MoeSpec:
    ff: int                   # an expert's hidden width
    experts: int
    top: int
    groups: int = 1
    keep: int = 1
    scale: float = 1.0


@dataclass
class BugapelHParams:
    n_vocab: int
    n_embd: int
    norm_eps: float
    streams: int = 1
    embed_scale: float = 1.0
    logit_softcap: float = 0.0
    mixers: List[MixSpec] = field(default_factory=list)
    mlps: List[Optional[MoeSpec]] = field(default_factory=list)
    arch: str = "bugapel"
    name: str = ""

    @property
    def n_layer(self) -> int:
        return len(self.mixers)

    @staticmethod
    def _mixer(kind: str, m: dict, where: str) -> MixSpec:
        H, dim = int(m["heads"]), int(m["dim"])
        vdim = int(m.get("vdim") or dim)
        if kind == "gla":
            if not float(m["tau"]) > 0 or dim > ops.GLA_MAX_KEY:
                raise ValueError(f"{where}: tau above 0, key heads up to {ops.GLA_MAX_KEY} wide")
            return MixSpec(kind, H, dim, vdim, tau=float(m["tau"]))
        if kind not in ("attention", "attention_2"):
            raise ValueError(f"{where}: unknown mixer type {kind!r}")
        r, mask = m.get("rot") or {}, m.get("mask") or {}
        s = MixSpec(kind, H, dim, vdim, kv_heads=int(m.get("kv_heads") or H), scale=float(m["scale"]),
                    rot_dims=int(r.get("dims") or 0), rot_base=float(r.get("base", 10000.0)),
                    rot_scaling=dict(r["scaling"]) if r.get("scaling") else None, window=int(mask.get("size") or 0),
                    keep=int(mask.get("keep_first") or 0))
        if H % s.kv_heads or s.rot_dims % 2 or s.rot_dims > dim or s.window < 0 or s.keep < 0:
            raise ValueError(f"{where}: heads a multiple of kv_heads, rot.dims even and at most dim, mask not negative")
        return s

    @staticmethod
    def _moe(f: dict, where: str) -> MoeSpec:
        if f.get("kind") != "moe":
            raise ValueError(f"{where}: unknown feed-forward kind {f.get('kind')!r}")
        r = f["router"]
        g = r.get("groups") or {}
        s = MoeSpec(int(f["expert"]["ff"]), int(r["experts"]), int(r["top"]), groups=int(g.get("count") or 1),
                    keep=int(g.get("keep") or g.get("count") or 1), scale=float(r.get("scale", 1.0)))
        if s.groups < 1 or s.experts % s.groups or not 1 <= s.keep <= s.groups or not 1 <= s.top <= s.keep * (s.experts // s.groups):
            raise ValueError(f"{where}: equal groups, whose kept ones hold at least `top` experts")
        return s

    @staticmethod
    def from_config(c: dict, name: str = "") -> "BugapelHParams":
        hp = BugapelHParams(n_vocab=int(c["vocab"]), n_embd=int(c["width"]), norm_eps=float(c["norm"]["eps"]),
                            streams=int(c.get("streams") or 1),
                            embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                            logit_softcap=float(c.get("logit_softcap") or 0.0), name=name)
        if not 1 <= hp.streams <= 16:
            raise ValueError("streams: 1 to 16")
        for i, L in enumerate(c["layers"]):
            hp.mixers.append(hp._mixer(L.get("type"), L["mixer"], f"layer {i}"))
            hp.mlps.append(hp._moe(L["mlp"], f"layer {i}") if L.get("mlp") else None)
        return hp


@dataclass
class _Exchange:
    """A sublayer's numbers at its two boundaries: what it reads of the streams and its norm, what it does to them."""
    in_w: torch.Tensor                           # fp32 [n]
    out_w: torch.Tensor                          # fp32 [n]
    mix: torch.Tensor                            # fp32 [n, n], [from, to]
    norm: tuple                                  # (weight, bias, eps)


@dataclass
class _Layer:
    win: ops.QWeight                             # attention: q | k | v rows; gla: q | k | v | gate | decay rank
    wo: ops.QWeight
    hc1: Optional[_Exchange] = None
    hc2: Optional[_Exchange] = None
    win_b: Optional[torch.Tensor] = None         # attention_2: fp32 biases of win and wo
    wo_b: Optional[torch.Tensor] = None
    freqs: Optional[torch.Tensor] = None
    sink: Optional[torch.Tensor] = None          # attention: zeros fp32 [H]
    a2: Optional[ops.QWeight] = None             # gla: decay logits from the rank
    a2_b: Optional[torch.Tensor] = None
    rank: int = 0
    mix_norm: Optional[torch.Tensor] = None      # fp32 [vdim]
    router: Optional[torch.Tensor] = None        # fp32 [E, D]
    experts: Optional[RoutedExperts] = None


class BugapelModel(LayeredModel):
    arch = "bugapel"
    # what this family launches from ops/csrc (ops.require_kernels: a first run compiles only these)
    kernel_sources = ("elementwise.hip", "hyper_streams.hip", "rope_pages.hip", "gla.hip", "attention_mix.hip", "attention.hip",
                      "moe_dense.hip", "moe.hip", "sampling.hip", "decode_loop.hip", "gemm_skinny.hip")

    def __init__(self, reader, device: torch.device, tp: Optional[TPInfo] = None, max_pos: Optional[int] = None,
                 rope_overrides: Optional[dict] = None, lora=None, dtype: torch.dtype = torch.bfloat16):
        self._begin(reader, device, tp, max_pos, lora, dtype)
        self.hp = hp = BugapelHParams.from_config(reader.config, str(reader.kv.get("general.name", "")))
        self.vocab_local = hp.n_vocab
        D = hp.n_embd
        emb = self._shaped("embed", (hp.n_vocab, D))
        self.tok_embd = ops.QWeight.from_float(emb.to(device))     # bf16 table, exact: stored as bf16
        self.output = self._qw(emb)                                # the table is also the head (unscaled)
        self.layers: List[_Layer] = []
        for i, (m, f) in enumerate(zip(hp.mixers, hp.mlps)):
            p = f"l{i}."
            L = self._load_gla(p + "mix.", m) if m.kind == "gla" else self._load_attention(p + "mix.", m)
            L.hc1 = self._exchange(p, 1)
            if f is not None:
                L.hc2 = self._exchange(p, 2)
                L.router = self._f32(p + "mlp.router", (f.experts, D))
                L.experts = RoutedExperts([(None, self._shaped(p + f"mlp.e{e}.up", (f.ff, D)),
                                            self._shaped(p + f"mlp.e{e}.down", (D, f.ff))) for e in range(f.experts)],
                                          device, dtype, "relu2")
            self.layers.append(L)
        self.out_norm = self._norm("final.norm")
        self.T = None

    # --------------------------------------------------------------------------- loading
    def _norm(self, name: str) -> tuple:
        D = self.hp.n_embd
        return self._f32(name, (D,)), self._f32(name + ".b", (D,)), self.hp.norm_eps

    def _exchange(self, p: str, q: int) -> _Exchange:
        n, h = self.hp.streams, f"{p}hc{q}."
        return _Exchange(self._f32(h + "in", (n,)), self._f32(h + "out", (n,)), self._f32(h + "mix", (n, n)),
                         self._norm(f"{p}norm{q}"))

    def _load_attention(self, p: str, m: MixSpec) -> _Layer:
        D, sh = self.hp.n_embd, self._shaped
        rows = (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim))
        L = _Layer(self._qw(torch.cat([sh(p + n, (N, D)) for n, N in rows], 0)), self._qw(sh(p + "o", (D, m.heads * m.vdim))))
        L.freqs, _ = ops.rot_freqs(m.rot_dims, m.rot_base, m.rot_scaling, self.device)
        if m.kind == "attention":
            L.sink = torch.zeros(m.heads, dtype=torch.float32, device=self.device)
        else:
            L.win_b = torch.cat([sh(p + n + ".b", (N,)) for n, N in rows], 0).to(self.device).contiguous()
            L.wo_b = self._f32(p + "o.b", (D,))
        return L

    def _load_gla(self, p: str, m: MixSpec) -> _Layer:
        D, sh = self.hp.n_embd, self._shaped
        Cq, Cv = m.heads * m.dim, m.heads * m.vdim
        a1 = self._raw(p + "a1")
        if a1.dim() != 2 or a1.shape[1] != D:
            raise ValueError(f"{p}a1 reads the layer's input")
        win = torch.cat([sh(p + "q", (Cq, D)), sh(p + "k", (Cq, D)), sh(p + "v", (Cv, D)), sh(p + "g", (Cv, D)), a1], 0)
        if win.shape[0] % 8:     # rows of zeros up to a multiple of 8: the projection's rows stay 16-byte aligned in bf16
            win = torch.cat([win, torch.zeros(8 - win.shape[0] % 8, D)], 0)
        L = _Layer(self._qw(win), self._qw(sh(p + "o", (D, Cv))))
        L.rank = a1.shape[0]
        L.a2, L.a2_b = self._qw(sh(p + "a2", (Cq, L.rank))), self._f32(p + "a2.b", (Cq,))
        L.mix_norm = self._f32(p + "norm", (m.vdim,))
        return L

    # --------------------------------------------------------------------------- engine interface
    def _run_specs(self):
        """KVCache.layered spec of every layer: pages for an attention layer, the recurrent state of a gla layer."""
        return [(0, 0, 0, [((m.heads, m.vdim, m.dim), torch.float32)]) if m.kind == "gla"
                else (m.kv_heads, m.dim, m.vdim, None) for m in self.hp.mixers]

    def _attention_specs(self):
        return [m for m in self.hp.mixers if m.kind != "gla"]

    # --------------------------------------------------------------------------- forward
    def _attention(self, L: _Layer, m: MixSpec, x, fb, kv, i, b, ws=None):
        kc, vc = kv.k[i], kv.v[i]
        first = m.kind == "attention"
        q = ops.head_rope_pages(ops.linear(x, L.win, L.win_b), m.heads, m.dim, m.kv_heads, m.dim, m.vdim, fb.pos, fb.slots,
                                L.freqs, m.rot_dims, not first, kc, vc, unit_eps=self.hp.norm_eps if first else None,
                                dtype=self.dtype)
        splits = 1
        if fb.decode:
            span = min(fb.max_len or 1, m.window + m.keep) if m.window else fb.max_len or 1
            splits = max(1, min(32, DECODE_WGS // max(x.shape[0], 1), -(-span // 32)))
        return self._attend(q, m, kc, vc, fb, b, splits, ws, window=m.window, keep=m.keep if m.window else 0, sink=L.sink)

    def _gla(self, L: _Layer, m: MixSpec, x, fb, kv, i, b):
        proj = self._dense(ops.linear(x, L.win))             # [T, q | k | v | gate | decay rank]
        c0 = 2 * m.heads * (m.dim + m.vdim)
        z = self._dense(ops.linear(proj[:, c0:c0 + L.rank].contiguous(), L.a2))
        return ops.gla(proj, z, L.a2_b, m.tau, m.heads, m.dim, m.vdim, fb.pos, b.cu_q, fb.sslots, kv.state[i][0], L.mix_norm,
                       self.hp.norm_eps, max_rows=b.max_rows)

    def forward(self, fb: ForwardBatch, kv: KVCache, attn_workspace=None, return_hidden: bool = False,
                local_logits: bool = False, layer_out: Optional[list] = None) -> torch.Tensor:
        """fp32 logits [R, V] of the rows fb.logits_idx selects (all rows when None).  Rows of one
        sequence are consecutive; fb.decode batches bring one row per sequence (fb.sslots per row),
        other batches fb.cu_q / fb.row_seq / fb.sslots per sequence.  layer_out: a list that
        receives the sum of the streams (fp32) after every layer (diagnostics)."""
        hp = self.hp
        if fb.sslots is None or kv.state is None:
            raise ValueError("bugapel: the batch needs state slots (engine built without a state pool?)")
        b = self._batch_rows(fb)
        x0 = self._embed(fb.tokens, hp.embed_scale)
        X = torch.empty(x0.shape[0], hp.streams, hp.n_embd, dtype=torch.float32, device=x0.device)

        def boundary(y, done: Optional[_Exchange], nxt: Optional[_Exchange]):
            """The finished sublayer's result into the streams, the next sublayer's input (or the output norm's) out of them."""
            kw = dict(mix=done.mix, out_w=done.out_w) if done is not None else dict(init=x0)
            return ops.hyper_streams(X, y, in_w=None if nxt is None else nxt.in_w,
                                     norm=self.out_norm if nxt is None else nxt.norm, out_dtype=self.dtype, **kw)

        x = boundary(None, None, self.layers[0].hc1 if self.layers else None)
        for i, (L, m, f) in enumerate(zip(self.layers, hp.mixers, hp.mlps)):
            after = self.layers[i + 1].hc1 if i + 1 < hp.n_layer else None
            if m.kind == "gla":
                a = self._gla(L, m, x, fb, kv, i, b)
            else:
                a = self._attention(L, m, x, fb, kv, i, b, attn_workspace)
            x = boundary(ops.linear(a, L.wo, L.wo_b), L.hc1, L.hc2 if f is not None else after)
            if f is not None:
                ids, wts = ops.router_softmax(x, L.router, None, f.top, f.groups, f.keep, f.scale)
                x = boundary(L.experts(x, ids, wts), L.hc2, after)
            if layer_out is not None:
                layer_out.append(X.sum(1))
        return x if return_hidden else self._logits(x, fb, hp.logit_softcap)
