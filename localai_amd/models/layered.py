"""What the layer-list model families have in common: checks and tensor loading, the engine interface
around KVCache.layered, the choice of the attention kernel for a batch, and routed experts.

A family derives from LayeredModel, gives `arch`, `kernel_sources` and `_run_specs()` (the KVCache.layered
spec of every layer run), loads its layers through _shaped / _f32 / _qw and writes `forward`.
"""
from __future__ import annotations

import os
from dataclasses import dataclass
from typing import Dict, List, Optional, Tuple, Union

import numpy as np
import torch

from .. import ops
from ..gguf import dequantize
from .decoder import ForwardBatch, KVCache, TPInfo

ATTN_WIDTHS = (64, 80, 96, 128, 192, 256)     # head widths the decode / prefill attention kernels are instantiated for


@dataclass
class BatchRows:
    """The rows of a batch as the attention and recurrence kernels take them."""
    row_seq: torch.Tensor                     # [T] sequence of every row
    cu_q: torch.Tensor                        # [nseq + 1]
    tiles: Optional[torch.Tensor]             # 16-row work tiles of ops.attn_mix
    tile_rows: int                            # leading rows they cover
    pf: Optional[torch.Tensor]                # 64-row work tiles of ops.attn_prefill (None: no layer takes them)
    max_rows: int                             # rows of the longest portion (1: one row per sequence)


class LayeredModel:
    arch = ""
    kernel_sources: Tuple[str, ...] = ()
    stateful = True         # per-sequence state in slots: no prefix-cache reuse
    mixed_batches = True    # prompt portions and decode rows of different sequences in one forward

    def _begin(self, reader, device: torch.device, tp: Optional[TPInfo], max_pos: Optional[int], lora, dtype: torch.dtype):
        self.tp = tp or TPInfo()
        if self.tp.world > 1:
            raise ValueError(f"{self.arch}: tensor parallelism is not implemented for this design")
        if lora is not None:
            raise ValueError(f"{self.arch}: LoRA adapters are not supported")
        if dtype not in (torch.bfloat16, torch.float32):
            raise ValueError(f"{self.arch}: serving dtype is bfloat16 or float32")
        self.device, self.dtype = device, dtype
        self.f32 = dtype == torch.float32
        self.max_pos = max_pos or 1 << 20
        self.T = reader.tensors
        self._aranges: Dict[int, tuple] = {}

    # --------------------------------------------------------------------------- loading
    def _raw(self, name: str) -> torch.Tensor:
        if name not in self.T:
            raise KeyError(f"{self.arch}: missing tensor {name}")
        t = self.T[name]
        return torch.from_numpy(dequantize(t.data, t.ggml_type, t.shape).astype(np.float32).reshape(t.shape))

    def _shaped(self, name: str, shape) -> torch.Tensor:
        w = self._raw(name)
        if tuple(w.shape) != tuple(shape):
            raise ValueError(f"{self.arch}: {name} is {tuple(w.shape)}, the config asks for {tuple(shape)}")
        return w

    def _f32(self, name: str, shape) -> torch.Tensor:
        return self._shaped(name, shape).to(self.device).contiguous()

    def _qw(self, w: torch.Tensor) -> ops.QWeight:
        w = w.to(self.device)
        return ops.QWeight.from_f32(w) if self.f32 else ops.QWeight.from_float(w)

    # --------------------------------------------------------------------------- engine interface
    def _run_specs(self) -> list:
        raise NotImplementedError

    def _attention_specs(self) -> list:
        """The softmax-attention layers (heads, kv_heads, dim, vdim) that may use the decode / prefill kernels."""
        return []

    def kv_bytes_per_token(self) -> int:
        es = 4 if self.f32 else 2
        return max(es, sum(g * (dk + dv) * es for g, dk, dv, *_ in self._run_specs()))

    def new_kv_cache(self, num_blocks: int, block_size: int, state_slots: int = 0) -> KVCache:
        return KVCache.layered(self._run_specs(), num_blocks, block_size, self.device, self.dtype, state_slots)

    def _decode_kernel_ok(self, m, block_size: int) -> bool:
        """Decode batches of this attention on the framework's split-KV decode attention kernel (the llama
        families'): bf16, equal key and value widths it is instantiated for."""
        return (not self.f32 and self.device.type == "cuda" and m.dim == m.vdim and m.dim in ATTN_WIDTHS
                and m.heads // m.kv_heads <= 16 and block_size % 16 == 0
                and (128 % block_size == 0 or block_size % 128 == 0) and ops._has("la_attn_decode"))

    def _prefill_kernel_ok(self, m) -> bool:
        """Batches of prompt portions only, for this attention, on the framework's prefill attention kernel
        (64 query rows of one head per workgroup)."""
        return (not self.f32 and self.device.type == "cuda" and m.dim == m.vdim and m.dim in ATTN_WIDTHS
                and ops._has("la_attn_prefill"))

    def decode_workspace(self, Bp: int, ctx: int, block_size: int):
        """Split-KV buffers of the decode attention kernel per (heads, kv heads, width) of the layers it serves."""
        out = {}
        for m in self._attention_specs():
            key = (m.heads, m.kv_heads, m.dim)
            if key not in out and self._decode_kernel_ok(m, block_size):
                out[key] = ops.decode_workspace(Bp, m.heads, m.kv_heads, m.dim, ctx, self.device, block_size)
        return out or None

    def prefill_tiles(self, q_lens, device):
        """((16-row work tiles of the leading prompt portions for ops.attn_mix, 64-row tiles of the same
        portions for ops.attn_prefill where a layer has the widths that kernel takes), rows they cover)."""
        if device.type != "cuda" or self.f32:
            return None, 0
        mix, rows = ops.attn_mix_tiles(q_lens, device)
        pf = None
        if any(self._prefill_kernel_ok(m) for m in self._attention_specs()):
            pf = ops.prefill_tiles(q_lens, device)
        return (mix, pf), rows

    # --------------------------------------------------------------------------- batches
    def _single_rows(self, T: int):
        """(row -> sequence, row ranges, one-row work tiles) of a batch with one row per sequence."""
        a = self._aranges.get(T)
        if a is None:
            r = torch.arange(T + 1, dtype=torch.int32, device=self.device)
            tiles = torch.stack([r[:T], torch.zeros_like(r[:T])], 1).contiguous()
            a = self._aranges[T] = (r[:T].contiguous(), r, tiles)
        return a

    def _batch_rows(self, fb: ForwardBatch) -> BatchRows:
        T = fb.tokens.shape[0]
        if fb.decode:
            row_seq, cu_q, tiles = self._single_rows(T)
            return BatchRows(row_seq, cu_q, tiles, T if not self.f32 and fb.tokens.is_cuda else 0, None, 1)
        if fb.row_seq is None:
            raise ValueError(f"{self.arch}: prompt batches need fb.row_seq")
        tiles, pf = fb.tiles if isinstance(fb.tiles, tuple) else (fb.tiles, None)
        return BatchRows(fb.row_seq, fb.cu_q, tiles, fb.tile_rows, pf, fb.max_q)

    # --------------------------------------------------------------------------- forward pieces
    def _dense(self, p: ops.Partial) -> torch.Tensor:
        """A projection's rows as one contiguous [T, N] matrix of the activation dtype."""
        t = p.t
        if p.bias is None and t.dim() == 3 and t.shape[0] == 1:
            t = t[0]
        elif p.bias is not None or t.dim() == 3:
            if t.is_cuda and p.N % 4 == 0:
                return ops.reduce(p, dtype=self.dtype)
            t = p.dense()
        return t if t.dtype == self.dtype else t.to(self.dtype)

    def _embed(self, tokens: torch.Tensor, scale: float = 1.0) -> torch.Tensor:
        """fp32 [T, D] rows of the embedding table times scale."""
        if tokens.is_cuda and self.tok_embd.K % 8:   # the embedding kernel reads 8 columns per thread
            x = self.tok_embd.materialize_bf16().index_select(0, tokens.long()).float() * scale
        else:
            x = ops.embed(tokens, self.tok_embd, scale)
        return x if x.is_contiguous() and x.dtype == torch.float32 else x.float().contiguous()

    def _logits(self, x: torch.Tensor, fb: ForwardBatch, softcap: float = 0.0) -> torch.Tensor:
        """fp32 logits of the rows fb.logits_idx selects (all when None), softcap tanh(. / softcap) when given."""
        rows = x if fb.logits_idx is None else x.index_select(0, fb.logits_idx)
        lp = ops.linear(rows.contiguous(), self.output)
        if softcap <= 0 and lp.t.dim() == 3 and lp.t.shape[0] == 1:
            return lp.t[0]
        if lp.N % 4 == 0 or not lp.t.is_cuda:
            return ops.reduce(lp, softcap=softcap)       # slabs, soft cap and fp32 rows in one launch
        lg = lp.dense()
        return torch.tanh(lg / softcap) * softcap if softcap > 0 else lg

    def _attend(self, q: torch.Tensor, m, kc: torch.Tensor, vc: torch.Tensor, fb: ForwardBatch, b: BatchRows, splits: int = 1,
                workspace=None, **kw) -> torch.Tensor:
        """Softmax attention of rows q [T, heads dim] over a layer's pages: decode batches on the split-KV decode
        kernel, batches of portions only on the prefill kernel, where they take the widths; everything else on
        ops.attn_mix.  kw: what all of them take (window, keep, sink, chunk, ...).  Returns [T, heads vdim]."""
        T = q.shape[0]
        if fb.decode and fb.seq_lens is not None and self._decode_kernel_ok(m, kc.shape[2]):
            ws = workspace.get((m.heads, m.kv_heads, m.dim)) if isinstance(workspace, dict) else None
            return ops.attn_decode(q.view(T, m.heads, m.dim), kc, vc, fb.block_tables, fb.seq_lens, m.scale, fb.max_len,
                                   workspace=ws, **kw).view(T, -1)
        if (b.pf is not None and not fb.decode and b.tile_rows == T and fb.ctx_lens is not None and self._prefill_kernel_ok(m)
                and kc.shape[2] % 16 == 0):
            return ops.attn_prefill(q.view(T, m.heads, m.dim), kc, vc, b.cu_q, fb.ctx_lens, fb.block_tables, m.scale,
                                    tiles=b.pf, **kw).view(T, -1)
        return ops.attn_mix(q, kc, vc, b.row_seq, fb.pos, fb.block_tables, m.heads, m.scale, tiles=b.tiles,
                            tile_rows=b.tile_rows, cu_q=b.cu_q, key_splits=splits, **kw)


# (token, expert) pair GEMVs up to this many rows, grouped rows + library GEMMs beyond
MOE_PAIR_MAX_T = int(os.environ.get("LOCALAI_AMD_LAYERED_PAIR_MAX_T", "32"))
# from this many rows on the grouped expert kernels give way to library GEMMs per expert
MOE_DENSE_MIN_T = 6144


class RoutedExperts:
    """The experts of one layer: down(act(up x)), or down(act(gate x) * up x) for gated ones.  weights[e] = (gate or
    None, up, down); act: "silu" (gated), "relu2" (ungated, max(., 0)^2) or ("clamp", limit, slope) (gated, ops.glu_clamp).
    Rows take one of three paths by batch size: pair GEMVs, the grouped expert GEMMs (bf16 widths % 256; routed on
    the device), or rows grouped by expert through library GEMMs."""

    def __init__(self, weights: List[tuple], device: torch.device, dtype: torch.dtype, act: Union[str, tuple]):
        self.E, self.act, self.dtype = len(weights), act, dtype
        self.F, self.D = weights[0][1].shape
        self.gated = act != "relu2"
        f32 = dtype == torch.float32
        put = lambda k: torch.stack([w[k] for w in weights]).to(device=device, dtype=dtype).contiguous()  # noqa: E731
        qw = ops.QWeight.from_f32 if f32 else ops.QWeight.from_float
        self.wg, self.wu, self.wd = put(0) if self.gated else None, put(1), put(2)
        # first projection per expert: [gate; up] rows fused, or views of the stacked up rows
        self.first = [qw(torch.cat([self.wg[e], self.wu[e]], 0) if self.gated else self.wu[e]) for e in range(self.E)]
        self.down = [qw(self.wd[e]) for e in range(self.E)]
        self.moe_first = self.moe_down = None
        if not f32 and device.type == "cuda" and self.D % 256 == 0 and self.F % 256 == 0:
            self.moe_first, self.moe_down = ops.MoEWeights(self.first), ops.MoEWeights(self.down)

    def _hidden(self, p: ops.Partial) -> torch.Tensor:
        """The experts' hidden activations [rows, F] from the first projection's result."""
        if isinstance(self.act, tuple):
            return ops.glu_clamp(p, self.F, self.act[1], self.act[2], out_dtype=self.dtype)
        if self.act == "silu":
            return ops.glu_act(p, self.F, ops.ACT_SWIGLU, self.dtype)
        if self.dtype == torch.bfloat16 and (self.F % 4 == 0 or not p.t.is_cuda) and (p.t.dim() == 3 or p.t.dtype == torch.bfloat16):
            return ops.act(p, self.F, ops.ACT_RELU2)
        return torch.relu(p.dense()).square().to(self.dtype)

    def __call__(self, x: torch.Tensor, ids: torch.Tensor, wts: torch.Tensor):
        """The weighted sum of every row's chosen experts: fp32 [T, D], or a Partial of it.  ids int32 [T, top], wts fp32 [T top]."""
        T, top = ids.shape
        capturing = x.is_cuda and torch.cuda.is_current_stream_capturing()
        if self.moe_first is not None and (T < MOE_DENSE_MIN_T or capturing) and T > 2:
            order, off = ops.moe_route(ids, self.E)
            h = self._hidden(ops.moe_linear(x, self.moe_first, order, off, top, T))
            return ops.moe_linear(h, self.moe_down, order, off, top, T, down=True, wts=wts)
        if T <= MOE_PAIR_MAX_T or capturing:
            clamp = self.act[1:] if isinstance(self.act, tuple) else None
            return ops.moe_pairs(x, self.wg, self.wu, self.wd, ids, wts, clamp=clamp)
        # rows grouped by expert (device), one host read of the group offsets, then per expert both projections
        # as library GEMMs over its rows and a weighted scatter-add in fp32
        order, off = ops.moe_route(ids, self.E)
        off_h = off.cpu().tolist()
        order_l = order.long()
        tok = order_l // top
        xs = x.index_select(0, tok)
        wsel = wts.index_select(0, order_l)
        out = torch.zeros(T, self.D, dtype=torch.float32, device=x.device)
        with ops.blas_tuning_paused():
            for e in range(self.E):
                r0, r1 = off_h[e], off_h[e + 1]
                if r1 > r0:
                    y = ops.linear(self._hidden(ops.linear(xs[r0:r1].contiguous(), self.first[e])), self.down[e])
                    y = y.t[0] if y.t.dim() == 3 and y.t.shape[0] == 1 else (y.t if y.t.dim() == 2 else y.dense())
                    out.index_add_(0, tok[r0:r1], y.float() * wsel[r0:r1].unsqueeze(1))
        return out
