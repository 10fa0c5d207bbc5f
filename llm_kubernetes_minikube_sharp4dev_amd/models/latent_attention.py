"""Latent attention over a cached latent: one cache row per token (``ops.latent``) serves all heads of a layer and every later
layer that shares it, so a layer without a latent of its own owns no cache at all.  Queries are brought to the latent (through
``W_uk^T``) once per token, the averaged latents go through ``W_uv`` afterwards; whole prompts, portions and decode rows read the same
cache rows.  (``models.window_attention.latent_window_attention`` is the mixer that caches expanded keys and values.)
"""
from __future__ import annotations

from dataclasses import dataclass, field
from typing import Optional

import torch

from .. import ops
from .attention import AttnMeta
from .linear_state import FusedRows, fused_mult
from .window_attention import RotarySpec


def _pad8(n: int) -> int:
    return -(-int(n) // 8) * 8


@dataclass
class CachedLatentAttnSpec:
    """Queries ``W_uq rms(W_dq h)`` of ``heads`` heads with ``dim`` plain and ``rot_dim`` rotated columns (dimension i pairs with i +
    rot_dim / 2); cached per token: ``rms`` of the first ``kv_rank`` columns of ``W_dkv h`` and the rotated last ``rot_dim``; keys
    ``[W_uk c | common rotated part]``, values ``W_uv c``; score times ``scale``; sliding window (0: causal); one learned sink score
    per head (``sink``).  ``kv_from``: the earlier layer whose cache this one reads (None: it has its own)."""
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    window: int = 0
    rot: RotarySpec = field(default_factory=RotarySpec)
    kv_from: Optional[int] = None
    sink: bool = True

    @classmethod
    def from_dict(cls, m: dict, sink: bool = True) -> "CachedLatentAttnSpec":
        rd = int(m.get("rot_dim", 0))
        rot = dict(m.get("rot") or {})
        rot["dims"] = rd
        kv_from = m.get("kv_from")
        s = cls(int(m["heads"]), int(m["dim"]), rd, int(m.get("vdim", m["dim"])), int(m["q_rank"]), int(m["kv_rank"]),
                float(m.get("scale", (int(m["dim"]) + rd) ** -0.5)), int((m.get("mask") or {}).get("size", 0)),
                RotarySpec.from_dict(rot, "none"), None if kv_from is None else int(kv_from), sink)
        if s.window < 0 or rd % 2 or min(s.heads, s.dim, s.vdim, s.q_rank, s.kv_rank) < 1:
            raise ValueError(f"unsupported latent attention sizes {m}")
        return s

    @property
    def qdim(self) -> int:
        """Columns of a query head in the projection (plain + rotated, padded to 16-byte fragments)."""
        return _pad8(self.dim + self.rot_dim)

    @property
    def kdim(self) -> int:
        """Plain columns of a query head that meet W_uk (zero weights behind ``dim``)."""
        return _pad8(self.dim)

    @property
    def vdim_p(self) -> int:
        return _pad8(self.vdim)

    @property
    def row(self) -> tuple:
        return ops.latent_row(self.kv_rank, self.rot_dim)

    def rows(self, width: int) -> FusedRows:
        seg = [("dq", self.q_rank)]
        if self.kv_from is None:
            seg.append(("dkv", self.kv_rank + self.rot_dim))
        return FusedRows(seg, fused_mult(width))

    def make_cache(self, num_blocks: int, block_size: int, dtype, device):
        return None if self.kv_from is not None else torch.zeros(num_blocks, block_size, sum(self.row), dtype=dtype, device=device)

    def bytes_per_token(self, dtype) -> int:
        return 0 if self.kv_from is not None else sum(self.row) * torch.tensor([], dtype=dtype).element_size()


def cached_latent_attention(h, w_in, rows: FusedRows, w_uq, w_uk, w_uv, dq_norm, dkv_norm, sink, cache, meta: AttnMeta,
                            spec: CachedLatentAttnSpec, freq, eps: float) -> torch.Tensor:
    """h [T, W] -> concatenated head outputs [T, H vdim_p].  ``w_in``: fused ``W_dq | W_dkv``; ``w_uq`` [H qdim, q_rank]; ``w_uk`` [H, RP,
    kdim] (transposed per head: it acts on queries); ``w_uv`` [H, vdim_p, RP]; ``dkv_norm`` None: ``cache`` is another layer's and is
    only read."""
    H, (rp, rdp) = spec.heads, spec.row
    u = ops.linear(h, w_in)
    T = u.shape[0]
    cq = ops.latent_prep(u, rows.off["dq"], spec.q_rank, dq_norm, rows.off.get("dkv", 0), spec.kv_rank, dkv_norm, spec.rot_dim, freq,
                         meta.positions, eps, cache, meta.slots, rp)
    q = ops.linear(cq, w_uq)
    qa = torch.empty(T, H, rp + rdp, dtype=u.dtype, device=u.device)
    ops.head_linear(q, w_uk, spec.qdim, qa)
    ops.latent_query_rot(q, qa, H, spec.qdim, spec.dim, spec.rot_dim, freq, meta.positions, rp)
    lat = torch.empty(T, H, rp, dtype=u.dtype, device=u.device)
    Tp, Bd = meta.num_prefill_tokens, meta.num_decode
    if Tp:
        ops.latent_attention_prefill(qa[:Tp], cache, meta.block_tables_p, meta.cu_q, meta.ctx_lens_p, spec.window, spec.scale, sink, rp,
                                     lat[:Tp], max(meta.q_lens_cpu))
    if Bd:
        span = meta.block_tables_d.shape[1] * cache.shape[1]
        Z = ops.latent_decode_splits(Bd, H, min(span, spec.window) if spec.window else span)
        ops.latent_attention_decode(qa[Tp:Tp + Bd], cache, meta.block_tables_d, meta.ctx_lens_d, spec.window, spec.scale, sink, rp,
                                    lat[Tp:Tp + Bd], splits=Z)
    out = torch.empty(T, H, spec.vdim_p, dtype=u.dtype, device=u.device)
    ops.head_linear(lat.view(T, H * rp), w_uv, rp, out)
    return out.view(T, H * spec.vdim_p)
