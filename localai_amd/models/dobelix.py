"""Dobelix: a decoder-only design described layer by layer in its config.json.

The residual stream is normed on the sublayer's OUTPUT only, x <- x + n1(mixer(x + conv(x))), x <- x +
n2(ff(x)) (ff optional), n an RMS norm with a plain weight; the sublayers read the stream itself.  What
a mixer reads first passes a short causal convolution on the stream (ops.stream_conv: branch norm,
residual add, convolution, and in decode batches the tail, in one launch); the last taps - 1 rows of
the stream are per-sequence state of every layer.  The embedding and the logits are scaled.  Two mixers:

  * "lightning": linear attention with a fixed decay per head on silu-activated q, k, v, one RMS norm
    over all heads together and a sigmoid gate (ops.lightning); its Dk x Dv state per head is
    per-sequence fp32 state in the scheduler's slot pool;
  * "attention": grouped-query attention whose values are its raw keys.  Queries and keys are normed
    over their whole projections, then rotated, queries times a number per head
    (ops.qk_row_norm_rope_pages); a key visible within the query's chunk weighs sigmoid(score + bias
    of the head), not normalised over the keys (sigmoid_bias of the attention kernels), and the
    output gate is applied as the kernels store their result.

Feed-forward: down(gelu_tanh(gate h) * up h).

The model plugs into LLMEngine like the other layer-list families: ForwardBatch, KVCache.layered, the
native scheduler's block tables and state slots; one query row per token, so prompt portions and
decoded tokens of different sequences share a forward (`mixed_batches`).  bf16 serving keeps the
residual stream with its convolution and tails, norms, angles, scores and weights and the recurrence
with its state in fp32; dtype=torch.float32 serves in true fp32 end to end.
"""
from __future__ import annotations

import os
from dataclasses import dataclass, field
from typing import List, Optional, Tuple

import torch

from .. import ops
from .decoder import ForwardBatch, KVCache, TPInfo
from .layered import LayeredModel

# decode rows of attention layers outside the split-KV decode kernel's widths: matrix-core tiles, keys dealt to
# about this many workgroups a batch
DECODE_TILES = os.environ.get("LOCALAI_AMD_DOBELIX_DECODE_TILES", "1") == "1"
DECODE_WGS = int(os.environ.get("LOCALAI_AMD_DOBELIX_DECODE_WGS", "1024"))


@dataclass
class MixSpec:
    kind: str                 # "lightning" | "attention"
    heads: int
    dim: int                  # query / key width per head
    vdim: int
    decay: Tuple[float, ...] = ()     # lightning, per head
    kv_heads: int = 0         # attention
    scale: float = 1.0
    chunk: int = 0            # keys of the query's chunk of this many positions (0: all)
    rot_dims: int = 0
    rot_base: float = 10000.0


@dataclass
class DobelixHParams:
    n_vocab: int
    n_embd: int
    norm_eps: float
    taps: int = 1             # of the convolution on the stream
    embed_scale: float = 1.0
    logit_scale: float = 1.0
    mixers: List[MixSpec] = field(default_factory=list)
    ffs: List[int] = field(default_factory=list)      # hidden width of the dense feed-forward, 0: none
    arch: str = "dobelix"
    name: str = ""

    @property
    def n_layer(self) -> int:
        return len(self.mixers)

    @staticmethod
    def from_config(c: dict, name: str = "") -> "DobelixHParams":
        hp = DobelixHParams(n_vocab=int(c["vocab"]), n_embd=int(c["width"]), norm_eps=float(c["norm"]["eps"]),
                            taps=int((c.get("canon") or {}).get("taps") or 0),
                            embed_scale=float((c.get("embedding") or {}).get("scale", 1.0)),
                            logit_scale=float(c.get("logit_scale", 1.0)), name=name)
        if hp.taps < 1:
            raise ValueError("canon.taps must be at least 1")
        for i, L in enumerate(c["layers"]):
            m, kind = L["mixer"], L.get("type")
            H, dim = int(m["heads"]), int(m["dim"])
            vdim = int(m.get("vdim") or dim)
            if kind == "lightning":
                s = MixSpec(kind, H, dim, vdim, decay=tuple(float(d) for d in m["decay"]))
                if len(s.decay) != H:
                    raise ValueError(f"layer {i}: one decay per head")
            elif kind == "attention":
                r = m.get("rot") or {}
                s = MixSpec(kind, H, dim, vdim, kv_heads=int(m.get("kv_heads") or H), scale=float(m["scale"]),
                            chunk=int((m.get("mask") or {}).get("size") or 0), rot_dims=int(r.get("dims") or 0),
                            rot_base=float(r.get("base", 10000.0)))
                if H % s.kv_heads or vdim != dim or s.rot_dims % 2 or s.rot_dims > dim:
                    raise ValueError(f"layer {i}: heads a multiple of kv_heads, values as wide as keys, rot.dims even and at most dim")
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            hp.mixers.append(s)
            f = L.get("mlp")
            if f and f.get("kind") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {f.get('kind')!r}")
            hp.ffs.append(int(f["ff"]) if f else 0)
        return hp


@dataclass
class _Layer:
    norm1: torch.Tensor
    conv_t: torch.Tensor                         # fp32 [taps, D], tap-major
    win: ops.QWeight                             # lightning: q | k | v | gate rows; attention: q | k | gate
    wo: ops.QWeight
    decay: Optional[torch.Tensor] = None         # lightning: fp32 [H]
    mix_norm: Optional[torch.Tensor] = None      # fp32 [H vdim]
    q_norm: Optional[torch.Tensor] = None        # attention: fp32 [H dim]
    k_norm: Optional[torch.Tensor] = None        # fp32 [G dim]
    temp: Optional[torch.Tensor] = None          # fp32 [H]
    bias: Optional[torch.Tensor] = None          # fp32 [H]
    freqs: Optional[torch.Tensor] = None
    norm2: Optional[torch.Tensor] = None
    gate_up: Optional[ops.QWeight] = None
    down: Optional[ops.QWeight] = None


class DobelixModel(LayeredModel):
    arch = "dobelix"
    # what this family launches from ops/csrc (ops.require_kernels: a first run compiles only these)
    kernel_sources = ("elementwise.hip", "norm_chain.hip", "shortconv.hip", "rope_pages.hip", "retention.hip",
                      "attention_mix.hip", "attention.hip", "sampling.hip", "decode_loop.hip", "gemm_skinny.hip")

    def __init__(self, reader, device: torch.device, tp: Optional[TPInfo] = None, max_pos: Optional[int] = None,
                 rope_overrides: Optional[dict] = None, lora=None, dtype: torch.dtype = torch.bfloat16):
        self._begin(reader, device, tp, max_pos, lora, dtype)
        self.hp = hp = DobelixHParams.from_config(reader.config, str(reader.kv.get("general.name", "")))
        self.vocab_local = hp.n_vocab
        D = hp.n_embd
        sh, qw = self._shaped, self._qw
        self.tok_embd = ops.QWeight.from_float(sh("embed", (hp.n_vocab, D)).to(device))   # bf16 table, exact
        self.layers: List[_Layer] = []
        for i, (m, ff) in enumerate(zip(hp.mixers, hp.ffs)):
            p = f"l{i}."
            L = self._load_lightning(p, m) if m.kind == "lightning" else self._load_attention(p, m)
            if ff:
                L.norm2 = self._f32(p + "norm2", (D,))
                L.gate_up = qw(torch.cat([sh(p + "mlp.gate", (ff, D)), sh(p + "mlp.up", (ff, D))], 0))
                L.down = qw(sh(p + "mlp.down", (D, ff)))
            self.layers.append(L)
        self.out_norm = ("rms", self._f32("final.norm", (D,)), hp.norm_eps)
        self.output = qw(sh("head", (hp.n_vocab, D)))
        self.T = None

    # --------------------------------------------------------------------------- loading
    def _layer(self, p: str, win: torch.Tensor, wo: torch.Tensor) -> _Layer:
        D, taps = self.hp.n_embd, self.hp.taps
        conv = self._shaped(p + "canon1", (D, taps)).t().contiguous().to(self.device)
        return _Layer(self._f32(p + "norm1", (D,)), conv, self._qw(win), self._qw(wo))

    def _load_lightning(self, p: str, m: MixSpec) -> _Layer:
        D, H = self.hp.n_embd, m.heads
        sh, x = self._shaped, p + "mix."
        win = torch.cat([sh(x + "q", (H * m.dim, D)), sh(x + "k", (H * m.dim, D)), sh(x + "v", (H * m.vdim, D)),
                         sh(x + "g", (H * m.vdim, D))], 0)
        L = self._layer(p, win, sh(x + "o", (D, H * m.vdim)))
        L.decay = torch.tensor(m.decay, dtype=torch.float32, device=self.device)
        L.mix_norm = self._f32(x + "norm", (H * m.vdim,))
        return L

    def _load_attention(self, p: str, m: MixSpec) -> _Layer:
        D, H, G = self.hp.n_embd, m.heads, m.kv_heads
        sh, x = self._shaped, p + "mix."
        win = torch.cat([sh(x + "q", (H * m.dim, D)), sh(x + "k", (G * m.dim, D)), sh(x + "g", (H * m.vdim, D))], 0)
        L = self._layer(p, win, sh(x + "o", (D, H * m.vdim)))
        L.q_norm, L.k_norm = self._f32(x + "q.norm", (H * m.dim,)), self._f32(x + "k.norm", (G * m.dim,))
        L.temp, L.bias = self._f32(x + "temp", (H,)), self._f32(x + "pb", (H,))
        L.freqs = ops.linear_rot_freqs(m.rot_dims, m.rot_base, 1.0, self.device)
        return L

    # --------------------------------------------------------------------------- engine interface
    def _run_specs(self):
        """KVCache.layered spec of every layer: the stream's convolution tail (fp32), beside pages for an
        attention layer or the recurrent state of a lightning layer."""
        tail = ((self.hp.taps - 1, self.hp.n_embd), torch.float32)
        return [(m.kv_heads, m.dim, m.vdim, [tail]) if m.kind == "attention"
                else (0, 0, 0, [tail, ((m.heads, m.vdim, m.dim), torch.float32)]) for m in self.hp.mixers]

    def _attention_specs(self):
        return [m for m in self.hp.mixers if m.kind == "attention"]

    # --------------------------------------------------------------------------- forward
    def _attention(self, L: _Layer, m: MixSpec, h, fb, kv, i, row_seq, cu_q, tiles, tile_rows, splits, ws=None):
        proj = self._dense(ops.linear(h, L.win))             # [T, q | k | gate]
        kc, vc = kv.k[i], kv.v[i]
        q = ops.qk_row_norm_rope_pages(proj, m.heads, m.dim, m.kv_heads, fb.pos, fb.slots, L.q_norm, L.k_norm,
                                       self.hp.norm_eps, L.freqs, m.rot_dims, kc, vc, head_scale=L.temp)
        T, N = q.shape
        gate = proj[:, (m.heads + m.kv_heads) * m.dim:]
        kw = dict(chunk=m.chunk, sigmoid_bias=L.bias, gate=gate)
        if fb.decode and fb.seq_lens is not None and self._decode_kernel_ok(m, kv.block_size):
            return ops.attn_decode(q.view(T, m.heads, m.dim), kc, vc, fb.block_tables, fb.seq_lens, m.scale, fb.max_len,
                                   workspace=ws, **kw).view(T, N)
        if isinstance(tiles, tuple):
            tiles, pf = tiles
            if (pf is not None and not fb.decode and tile_rows == T and fb.ctx_lens is not None
                    and self._prefill_kernel_ok(m) and kv.block_size % 16 == 0):
                return ops.attn_prefill(q.view(T, m.heads, m.dim), kc, vc, cu_q, fb.ctx_lens, fb.block_tables, m.scale,
                                        tiles=pf, **kw).view(T, N)
        return ops.attn_mix(q, kc, vc, row_seq, fb.pos, fb.block_tables, m.heads, m.scale, tiles=tiles,
                            tile_rows=tile_rows, cu_q=cu_q, key_splits=splits, **kw)

    def _lightning(self, L: _Layer, m: MixSpec, h, fb, kv, i, cu_q):
        proj = self._dense(ops.linear(h, L.win))             # [T, q | k | v | gate]
        return ops.lightning(proj, m.heads, m.dim, m.vdim, fb.pos, cu_q, fb.sslots, kv.state[i][1], L.decay, L.mix_norm,
                             self.hp.norm_eps, max_rows=1 if fb.decode else fb.max_q)

    def forward(self, fb: ForwardBatch, kv: KVCache, attn_workspace=None, return_hidden: bool = False,
                local_logits: bool = False, layer_out: Optional[list] = None) -> torch.Tensor:
        """fp32 logits [R, V] of the rows fb.logits_idx selects (all rows when None).  Rows of one
        sequence are consecutive; fb.decode batches bring one row per sequence (fb.sslots per row),
        other batches fb.cu_q / fb.row_seq / fb.sslots per sequence.  layer_out: a list that
        receives the fp32 residual stream after every layer (diagnostics)."""
        hp = self.hp
        T = fb.tokens.shape[0]
        if fb.sslots is None or kv.state is None:
            raise ValueError("dobelix: the batch needs state slots (engine built without a state pool?)")
        if fb.decode:
            row_seq, cu_q, tiles = self._single_rows(T)
            tile_rows = T if (DECODE_TILES and not self.f32 and fb.tokens.is_cuda) else 0
            splits_for = lambda m: max(1, min(32, DECODE_WGS // max(T, 1), -(-(m.chunk or fb.max_len or 1) // 32)))  # noqa: E731
        else:
            row_seq, cu_q, tiles, tile_rows = fb.row_seq, fb.cu_q, fb.tiles, fb.tile_rows
            if row_seq is None:
                raise ValueError("dobelix: prompt batches need fb.row_seq")
            splits_for = lambda m: 1  # noqa: E731
        if fb.tokens.is_cuda and hp.n_embd % 8:   # the embedding kernel reads 8 columns per thread
            res = self.tok_embd.materialize_bf16().index_select(0, fb.tokens.long()).float() * hp.embed_scale
        else:
            res = ops.embed(fb.tokens, self.tok_embd, hp.embed_scale)
        if not res.is_contiguous() or res.dtype != torch.float32:
            res = res.float().contiguous()
        eps, n = hp.norm_eps, hp.n_layer

        def boundary(branch, w, i):
            """The branch's norm and the residual add, then what the next reader takes: layer i's convolved
            stream, or the model's norm after the last layer."""
            post = ("rms", w, eps) if branch is not None else None
            if i == n:
                return ops.norm_chain(res, branch, post, self.out_norm, out_dtype=self.dtype)
            return ops.stream_conv(res, branch, post, self.layers[i].conv_t, row_seq, cu_q, fb.pos, fb.sslots, kv.state[i][0],
                                   single=fb.decode, out_dtype=self.dtype)

        h = boundary(None, None, 0)
        for i, (L, m, ff) in enumerate(zip(self.layers, hp.mixers, hp.ffs)):
            if m.kind == "attention":
                ws = attn_workspace.get((m.heads, m.kv_heads, m.dim)) if isinstance(attn_workspace, dict) else None
                a = self._attention(L, m, h, fb, kv, i, row_seq, cu_q, tiles, tile_rows, splits_for(m), ws)
            else:
                a = self._lightning(L, m, h, fb, kv, i, cu_q)
            y, w = ops.linear(a, L.wo), L.norm1
            if ff:
                x = ops.norm_chain(res, y, ("rms", w, eps), ("cast",), out_dtype=self.dtype)
                y, w = ops.linear(ops.glu_act(ops.linear(x, L.gate_up), ff, ops.ACT_GEGLU, self.dtype), L.down), L.norm2
            h = boundary(y, w, i + 1)
            if layer_out is not None:
                layer_out.append(res.clone())
        if return_hidden:
            return h
        rows = h if fb.logits_idx is None else h.index_select(0, fb.logits_idx)
        lp = ops.linear(rows.contiguous(), self.output)
        logits = lp.t[0] if (lp.t.dim() == 3 and lp.t.shape[0] == 1 and lp.t.dtype == torch.float32) else self._dense(lp).float()
        return logits if hp.logit_scale == 1.0 else logits.mul_(hp.logit_scale)
