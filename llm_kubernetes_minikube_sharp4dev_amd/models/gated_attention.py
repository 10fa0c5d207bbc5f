"""Causal softmax attention mixers with biased projections and one output gate per element over the engine's paged
cache: differential attention (two maps per head over the same values, subtracted) and attention whose queries and
keys are RMS-normed over the whole projection before rotation.  One kernel files a step's keys and values
(``ops.qkv_file``: bias, norm, rotation, cache write); prompt rows and decode rows then attend through the cache, so
whole prompts, portions and decode rows are one code path.
"""
from __future__ import annotations

import math
from dataclasses import dataclass, field

import torch

from .. import ops
from .attention import AttnMeta
from .window_attention import RotarySpec, _cache_pair


def _pad8(n: int) -> int:
    return -(-int(n) // 8) * 8


def _row_tiles(meta: AttnMeta, rows: int, device):
    """Tile list of the staged prefill kernel (``rows`` queries each), built once per step and kept on the meta."""
    t = meta.row_tiles.get(rows)
    if t is None:
        ts, tq = ops.row_tiles(meta.q_lens_cpu, meta.ctx_lens_cpu, rows)
        t = meta.row_tiles[rows] = (torch.from_numpy(ts).to(device, non_blocking=True), torch.from_numpy(tq).to(device, non_blocking=True))
    return t


@dataclass
class DiffAttnSpec:
    """Differential attention: head h holds two query / key maps of ``dim`` columns each (``[map 1, map 2]``, queries times
    ``1 + temp_coef ln(floor((p + 1) / temp_every) + 1)`` at position p; ``temp_every`` 0: plain) and one value of ``vdim`` columns; the
    output is ``rms(a1 - lambda a2) * (1 - diff)`` of the two maps' softmax averages a1, a2 (``lambda`` a number of the
    layer).  Head sizes here are the kernels' (multiples of 8); ``true_vdim`` is the checkpoint's."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    diff: float
    temp_coef: float = 0.0
    temp_every: int = 0
    true_vdim: int = 0

    @classmethod
    def from_dict(cls, m: dict) -> "DiffAttnSpec":
        t = m.get("q_temp") or {}
        s = cls(int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m.get("vdim", m["dim"])),
                float(m.get("scale", int(m["dim"]) ** -0.5)), float(m["diff"]), float(t.get("coef", 0.0)), int(t.get("every", 0)))
        s.true_vdim = s.vdim
        if s.heads % s.kv_heads or s.temp_every < 0 or not ops.diff_attention_supported(s.heads, s.kv_heads, _pad8(s.dim), _pad8(s.vdim)):
            raise ValueError(f"unsupported differential attention sizes {m}")
        return s

    def padded(self) -> "DiffAttnSpec":
        return DiffAttnSpec(self.heads, self.kv_heads, _pad8(self.dim), _pad8(self.vdim), self.scale, self.diff, self.temp_coef,
                            self.temp_every, self.true_vdim)

    def segments(self) -> list:
        return [("q", self.heads * 2 * self.dim), ("k", self.kv_heads * 2 * self.dim), ("v", self.kv_heads * self.vdim), ("g", self.heads * self.vdim)]

    def make_caches(self, num_blocks: int, block_size: int, dtype, device) -> tuple:
        return _cache_pair(num_blocks, self.kv_heads, block_size, 2 * self.dim, self.vdim, dtype, device)

    def bytes_per_token(self, dtype) -> int:
        return self.kv_heads * (2 * self.dim + self.vdim) * torch.tensor([], dtype=dtype).element_size()


def diff_lambda(lq1, lk1, lq2, lk2, diff: float) -> float:
    """The layer's weight of the second map (float64, once at load)."""
    d = [t.double().cpu() for t in (lq1, lk1, lq2, lk2)]
    return math.exp(float((d[0] * d[1]).sum())) - math.exp(float((d[2] * d[3]).sum())) + diff


def diff_attention(u: torch.Tensor, rows, caches, meta: AttnMeta, spec: DiffAttnSpec, bias, lam, eps: float, out) -> torch.Tensor:
    """u [T, q | k | v | g ..] = the fused projections (``rows``: their layout, q | k | v adjacent; ``spec``: the padded sizes); ``bias``
    f32 over q | k | v; ``lam`` f32 [1].  ``out`` [T, >= heads * vdim]."""
    H, G, dim, vdim = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    kc, vc = caches[0], caches[1]
    ops.qkv_file(u, rows.off["q"], H, G, 2 * dim, vdim, bias, None, None, 0, 0, eps, 0, None, 1.0, meta.positions, kc, vc, meta.slots)
    q = u[:, rows.off["q"]:rows.off["q"] + H * 2 * dim]
    Tp, Bd = meta.num_prefill_tokens, meta.num_decode
    opt = dict(scale=spec.scale, temp_coef=spec.temp_coef, temp_every=spec.temp_every, lam=lam, eps=eps, norm_vdim=spec.true_vdim,
               out_scale=1.0 - spec.diff)
    gcol = rows.off["g"]
    if Tp:
        r = ops.diff_prefill_rows(H, G, dim, vdim, u.dtype) if u.is_cuda else 16
        ops.diff_attention_prefill(q[:Tp], kc, vc, meta.block_tables_p, meta.cu_q, meta.ctx_lens_p, H, G, dim, vdim, u[:Tp], gcol, out[:Tp],
                                   tiles=_row_tiles(meta, r, u.device) if u.is_cuda else None, **opt)
    if Bd:
        span = meta.block_tables_d.shape[1] * kc.shape[2]
        Z = ops.sig_decode_splits(Bd, G, H // G, span)
        ops.diff_attention_decode(q[Tp:Tp + Bd], kc, vc, meta.block_tables_d, meta.ctx_lens_d, H, G, dim, vdim, u[Tp:Tp + Bd], gcol,
                                  out[Tp:Tp + Bd], splits=Z, **opt)
    return out


@dataclass
class RowNormAttnSpec:
    """Grouped-query causal softmax attention; q and k RMS-normed over the whole projection (all heads at once) with a weight
    per row, then rotated in adjacent pairs; scores ``cap * tanh(scale q.k / cap)`` (``softcap`` 0: plain).  Head sizes here are the
    kernels' (multiples of 8); ``true_dim`` is the checkpoint's (the divisor of the means counts true columns)."""
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    softcap: float = 0.0
    rot: RotarySpec = field(default_factory=RotarySpec)
    true_dim: int = 0

    @classmethod
    def from_dict(cls, m: dict) -> "RowNormAttnSpec":
        s = cls(int(m["heads"]), int(m.get("kv_heads", m["heads"])), int(m["dim"]), int(m.get("vdim", m["dim"])),
                float(m.get("scale", int(m["dim"]) ** -0.5)), float(m.get("softcap") or 0.0), RotarySpec.from_dict(m.get("rot"), "ramp"))
        s.true_dim = s.dim
        if s.heads % s.kv_heads or s.softcap < 0 or s.rot.dims > s.dim:
            raise ValueError(f"unsupported attention sizes {m}")
        return s

    def padded(self) -> "RowNormAttnSpec":
        return RowNormAttnSpec(self.heads, self.kv_heads, _pad8(self.dim), _pad8(self.vdim), self.scale, self.softcap, self.rot, self.true_dim)

    def segments(self) -> list:
        return [("q", self.heads * self.dim), ("k", self.kv_heads * self.dim), ("v", self.kv_heads * self.vdim), ("g", self.heads * self.vdim)]

    def make_caches(self, num_blocks: int, block_size: int, dtype, device) -> tuple:
        return _cache_pair(num_blocks, self.kv_heads, block_size, self.dim, self.vdim, dtype, device)

    def bytes_per_token(self, dtype) -> int:
        return self.kv_heads * (self.dim + self.vdim) * torch.tensor([], dtype=dtype).element_size()


def row_norm_attention(u: torch.Tensor, rows, caches, meta: AttnMeta, spec: RowNormAttnSpec, bias, q_norm, k_norm, freq, hscale, eps: float,
                       out, out_scale: float = 1.0) -> torch.Tensor:
    """u [T, q | k | v | g ..] = the fused projections (q | k | v adjacent; ``spec``: the padded sizes); ``bias`` f32 over q | k | v,
    ``q_norm`` / ``k_norm`` f32 over all q / k rows.  ``out`` [T, >= heads * vdim], times ``out_scale``."""
    H, G, dim, vdim = spec.heads, spec.kv_heads, spec.dim, spec.vdim
    kc, vc = caches[0], caches[1]
    ops.qkv_file(u, rows.off["q"], H, G, dim, vdim, bias, q_norm, k_norm, H * spec.true_dim, G * spec.true_dim, eps, spec.rot.dims, freq,
                 spec.rot.magnitude, meta.positions, kc, vc, meta.slots)
    q = u[:, rows.off["q"]:rows.off["q"] + H * dim]
    Tp, Bd = meta.num_prefill_tokens, meta.num_decode
    gcol = rows.off["g"]
    if Tp:
        if u.is_cuda and ops.tile_attention_supported(H, G, dim, vdim, u.dtype):
            ops.tile_attention_prefill(q[:Tp], kc, vc, meta.block_tables_p, meta.cu_q, meta.ctx_lens_p, H, G, dim, vdim, u[:Tp], gcol, out[:Tp],
                                       _row_tiles(meta, ops.tile_attention_rows(H, G), u.device), scale=spec.scale, softcap=spec.softcap,
                                       out_scale=out_scale)
        else:
            ops.sink_attention_prefill(q[:Tp], kc, vc, meta.block_tables_p, meta.cu_q, meta.ctx_lens_p, H, G, dim, vdim, hscale, ops.MASK_CAUSAL, 0,
                                       False, u[:Tp], gcol, out[:Tp], tiles=_row_tiles(meta, ops.SIG_TILE_ROWS, u.device) if u.is_cuda else None,
                                       softcap=spec.softcap, gate_elem=True, out_scale=out_scale)
    if Bd:
        span = meta.block_tables_d.shape[1] * kc.shape[2]
        Z = ops.sig_decode_splits(Bd, G, H // G, span)
        ops.sink_attention_decode(q[Tp:Tp + Bd], kc, vc, meta.block_tables_d, meta.ctx_lens_d, H, G, dim, vdim, hscale, ops.MASK_CAUSAL, 0, False,
                                  u[Tp:Tp + Bd], gcol, out[Tp:Tp + Bd], splits=Z, softcap=spec.softcap, gate_elem=True, out_scale=out_scale)
    return out
