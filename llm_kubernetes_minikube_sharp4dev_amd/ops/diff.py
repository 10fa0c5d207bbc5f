"""Entry points of the kernels behind causal attention with biased projections and element gates (``csrc/qkv_file.hip``,
``csrc/attn_diff.hip``, ``csrc/attn_tile.hip``), with their CPU implementations:

* ``qkv_file``               -- bias, RMS norm over a whole projection, rotation of adjacent pairs; q in place, k and v in the cache;
* ``diff_attention_*``       -- two softmax maps per head over the same values, subtracted, normed, gated;
* ``tile_attention_prefill`` -- one map with an optional score cap on the LDS-staged prompt kernel of the differential form.

Layouts are those of ``ops.mixers``: K cache ``[blocks, G, BS, dim]`` (both maps of a differential head behind one another: ``2 dim``
columns), V cache key-contiguous ``[blocks, G, vdim, BS]``.
"""
from __future__ import annotations

import math
from typing import Optional, Sequence

import numpy as np
import torch

from ._ext import lib, use_hip
from .mixers import _gather_kv

__all__ = ["qkv_file", "row_tiles", "diff_attention_supported", "diff_attention_prefill", "diff_attention_decode", "diff_prefill_rows",
           "tile_attention_supported", "tile_attention_rows", "tile_attention_prefill"]

DIFF_MAX_HEAD = 256          # largest map size and value size of the kernels
TILE_WAVE_ROWS = 32          # queries a wave of the staged prefill kernel holds


def qkv_file(u, col0: int, H: int, G: int, dim: int, vdim: int, bias, q_w, k_w, norm_q: int, norm_k: int, eps: float, rot: int, freq,
             mag: float, positions, k_cache, v_cache, slots):
    """Columns ``[col0, ..)`` of ``u`` hold ``[q: H dim | k: G dim | v: G vdim]``.  In f32: ``bias`` (f32 over all of them, or None) is
    added; with ``q_w`` / ``k_w`` (f32 [H dim] / [G dim], or None) q is divided by its root mean square over the whole projection (sum of
    squares / ``norm_q``, k likewise with ``norm_k``) and multiplied by the weight; the first ``rot`` dimensions of every q and k head are
    rotated in adjacent pairs by ``position * freq[i]``, cos and sin times ``mag``.  q in place, k and v into the paged cache at
    ``slots`` (< 0: nothing is cached)."""
    if use_hip(u):
        lib().qkv_file(u, int(col0), H, G, dim, vdim, bias, q_w, k_w, int(norm_q), int(norm_k), float(eps), int(rot), freq, float(mag),
                       positions, k_cache, v_cache, slots)
        return u
    T, nq, nk = u.shape[0], H * dim, G * dim
    x = u[:, col0:col0 + nq + nk + G * vdim].float()
    if bias is not None:
        x = x + bias.float()
    q, k, v = x[:, :nq], x[:, nq:nq + nk], x[:, nq + nk:]
    if q_w is not None:
        q = q / torch.sqrt(q.pow(2).sum(-1, keepdim=True) / norm_q + eps) * q_w
        k = k / torch.sqrt(k.pow(2).sum(-1, keepdim=True) / norm_k + eps) * k_w
    q, k, v = q.reshape(T, H, dim).clone(), k.reshape(T, G, dim).clone(), v.reshape(T, G, vdim)
    half = rot // 2
    if half:
        ang = positions[:T].float().view(T, 1, 1) * freq.float()[:half].view(1, 1, half)
        c, s = torch.cos(ang) * mag, torch.sin(ang) * mag
        for t in (q, k):
            a, b = t[..., 0:rot:2].clone(), t[..., 1:rot:2].clone()
            t[..., 0:rot:2] = a * c - b * s
            t[..., 1:rot:2] = b * c + a * s
    u[:, col0:col0 + nq] = q.reshape(T, -1).to(u.dtype)
    BS = k_cache.shape[2]
    sl = slots[:T].long()
    ok = sl >= 0
    blk, off = sl[ok] // BS, sl[ok] % BS
    k_cache[blk, :, off, :] = k[ok].to(k_cache.dtype)
    v_cache[blk, :, :, off] = v[ok].to(v_cache.dtype)
    return u


def row_tiles(q_lens: Sequence[int], ctx_lens: Optional[Sequence[int]], rows: int):
    """(tile_seq, tile_q0) int32: one entry per ``rows`` queries of each chunk, heaviest (latest end position) first."""
    tiles = []
    for b, n in enumerate(q_lens):
        past = (ctx_lens[b] - n) if ctx_lens is not None else 0
        tiles += [(past + s + rows, b, s) for s in range(0, n, rows)]
    tiles.sort(key=lambda t: -t[0])
    return (np.asarray([t[1] for t in tiles], dtype=np.int32), np.asarray([t[2] for t in tiles], dtype=np.int32))


def diff_attention_supported(H: int, G: int, dim: int, vdim: int) -> bool:
    return H >= 1 and G >= 1 and H % G == 0 and 1 <= dim <= DIFF_MAX_HEAD and 1 <= vdim <= DIFF_MAX_HEAD


def tile_attention_rows(H: int, G: int) -> int:
    """Queries per workgroup of the staged prefill kernel: its four waves hold 32 queries each, of up to 4 heads of a kv group."""
    rep = H // G
    return TILE_WAVE_ROWS * (1 if rep % 4 == 0 else 2 if rep % 2 == 0 else 4)


def tile_attention_supported(H: int, G: int, dim: int, vdim: int, dtype) -> bool:
    return dtype == torch.bfloat16 and H % G == 0 and max(dim, vdim) <= DIFF_MAX_HEAD and dim % 8 == 0 and vdim % 8 == 0


def diff_prefill_rows(H: int, G: int, dim: int, vdim: int, dtype) -> int:
    """Queries per entry of the tile list ``diff_attention_prefill`` takes."""
    return tile_attention_rows(H, G) if tile_attention_supported(H, G, dim, vdim, dtype) else 16


def _temperature(qpos, coef: float, every: int):
    if not every or coef == 0.0:
        return torch.ones_like(qpos, dtype=torch.float32)
    return 1.0 + coef * torch.log((torch.div(qpos + 1, every, rounding_mode="floor") + 1).float())


def _diff_rows(q, k, v, qpos, scale, temp_coef, temp_every, lam, eps, norm_vdim, out_scale):
    """q f32 [S, H, 2, dim] at positions qpos [S]; k f32 [n, G, 2, dim], v f32 [n, G, vdim] at positions 0..n-1."""
    rep = q.shape[1] // k.shape[1]
    kk, vv = k.repeat_interleave(rep, 1), v.repeat_interleave(rep, 1)
    s = torch.einsum("ihmd,jhmd->mhij", q, kk) * (scale * _temperature(qpos, temp_coef, temp_every)).view(1, 1, -1, 1)
    seen = torch.arange(k.shape[0], device=q.device).view(1, -1) <= qpos.view(-1, 1)
    a = torch.einsum("mhij,jhe->mihe", torch.softmax(s.masked_fill(~seen, float("-inf")), -1), vv)
    o = a[0] - float(lam) * a[1]
    return o / torch.sqrt(o.pow(2).sum(-1, keepdim=True) / norm_vdim + eps) * out_scale


def _gate(o, gate, gate_col):
    S, H, e = o.shape
    return (o * torch.sigmoid(gate[:, gate_col:gate_col + H * e].float()).view(S, H, e)).reshape(S, H * e)


def diff_attention_prefill(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, H: int, G: int, dim: int, vdim: int, gate, gate_col: int, out,
                           scale: float, temp_coef: float, temp_every: int, lam, eps: float, norm_vdim: int, out_scale: float, tiles=None):
    """Causal differential attention of query chunks over their sequences' cached keys.  q: rows whose first H * 2 dim columns are the
    queries (head by head [map 1, map 2]); a query at position p is multiplied by ``1 + temp_coef ln(floor((p + 1) / temp_every) + 1)``
    (f32, with the score scale; ``temp_every`` 0: 1).  Per head ``o = a1 - lam a2`` (lam f32 [1]) divided by its root mean square over the
    values (sum of squares / ``norm_vdim``), times ``out_scale``, times the sigmoid of the gate column ``gate_col + h vdim + d``.
    ``tiles``: ``row_tiles`` of ``diff_prefill_rows`` queries."""
    if use_hip(q):
        rows = diff_prefill_rows(H, G, dim, vdim, q.dtype)
        if tiles is None:
            ts, tq = row_tiles((cu_q[1:] - cu_q[:-1]).tolist(), ctx_lens.tolist(), rows)
            tiles = (torch.from_numpy(ts).to(q.device), torch.from_numpy(tq).to(q.device))
        if rows != 16:
            lib().tile_attention_prefill(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, tiles[0], tiles[1], 2, H, G, dim, vdim, float(scale),
                                         0.0, float(temp_coef), int(temp_every), lam, float(eps), int(norm_vdim), float(out_scale), gate,
                                         int(gate_col), out)
        else:
            lib().diff_attention_prefill(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, tiles[0], tiles[1], H, G, dim, vdim, float(scale),
                                         float(temp_coef), int(temp_every), lam, float(eps), int(norm_vdim), float(out_scale), gate,
                                         int(gate_col), out)
        return out
    cu = cu_q.tolist()
    for b in range(len(cu) - 1):
        s0, s1, n = cu[b], cu[b + 1], int(ctx_lens[b])
        k, v = _gather_kv(k_cache, v_cache, block_tables[b], n)
        qpos = torch.arange(n - (s1 - s0), n)
        o = _diff_rows(q[s0:s1, : H * 2 * dim].float().reshape(-1, H, 2, dim), k.view(n, G, 2, dim), v, qpos, scale, temp_coef, temp_every,
                       lam, eps, norm_vdim, out_scale)
        out[s0:s1, : H * vdim] = _gate(o, gate[s0:s1], gate_col).to(out.dtype)
    return out


def diff_attention_decode(q, k_cache, v_cache, block_tables, ctx_lens, H: int, G: int, dim: int, vdim: int, gate, gate_col: int, out,
                          scale: float, temp_coef: float, temp_every: int, lam, eps: float, norm_vdim: int, out_scale: float,
                          splits: int = 1, part=None):
    """One query row per sequence at its last position (ctx - 1) over its cached keys (see ``diff_attention_prefill``)."""
    B = q.shape[0]
    if use_hip(q):
        if splits > 1 and part is None:
            part = torch.empty(B * H * splits * 2 * (vdim + 2), dtype=torch.float32, device=q.device)
        lib().diff_attention_decode(q, k_cache, v_cache, block_tables, ctx_lens, int(splits), H, G, dim, vdim, float(scale), float(temp_coef),
                                    int(temp_every), lam, float(eps), int(norm_vdim), float(out_scale), gate, int(gate_col), out, part)
        return out
    for b in range(B):
        n = int(ctx_lens[b])
        k, v = _gather_kv(k_cache, v_cache, block_tables[b], n)
        o = _diff_rows(q[b:b + 1, : H * 2 * dim].float().reshape(1, H, 2, dim), k.view(n, G, 2, dim), v, torch.tensor([n - 1]), scale,
                       temp_coef, temp_every, lam, eps, norm_vdim, out_scale)
        out[b:b + 1, : H * vdim] = _gate(o, gate[b:b + 1], gate_col).to(out.dtype)
    return out


def tile_attention_prefill(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, H: int, G: int, dim: int, vdim: int, gate, gate_col: int, out,
                           tiles, scale: float, softcap: float = 0.0, out_scale: float = 1.0):
    """Causal grouped-query attention of bf16 query chunks on the staged prompt kernel: scores ``scale q.k`` (``softcap`` > 0: ``cap *
    tanh(score / cap)``), element gate, times ``out_scale`` (GPU only; elsewhere ``sink_attention_prefill`` computes the same)."""
    lib().tile_attention_prefill(q, k_cache, v_cache, block_tables, cu_q, ctx_lens, tiles[0], tiles[1], 1, H, G, dim, vdim, float(scale),
                                 float(softcap), 0.0, 0, None, 0.0, int(vdim), float(out_scale), gate, int(gate_col), out)
    return out
