"""Entry points of attention over a cached latent (``csrc/latent_attn.hip``, ``csrc/head_linear.hip``): a token's cache row is
``[latent c | zeros | rotated key part | zeros]``, common to all query heads and to every layer that reads it.  A head's key
``[W_uk c | common part]`` and value ``W_uv c`` are never formed: its query goes through ``W_uk^T`` once (so the score is a dot
product with the cache row), and the softmax average of the latents goes through ``W_uv`` afterwards.

    s(i, j) = scale * <[W_uk^T q | rotated q]_i, row_j>     for first(i) <= j <= i
    p(i, j) = exp(s(i, j)) / (exp(sink_h) + sum_j' exp(s(i, j')))          out_i = W_uv sum_j p(i, j) c_j

Cache ``[blocks, BS, KD]`` in the activation dtype, ``KD = RP + RDP`` (``latent_row``).  GPU tensors go to the HIP kernels, CPU
tensors to the torch implementations below.
"""
from __future__ import annotations

import torch

from ._ext import lib, use_hip

__all__ = ["latent_row", "latent_prep", "latent_query_rot", "head_linear", "latent_attention_prefill", "latent_attention_decode",
           "latent_decode_splits"]


def latent_row(kv_rank: int, rot_dim: int) -> tuple:
    """(RP, RDP): columns of a cache row that hold the latent and the rotated part, padded to the kernels' sizes."""
    rp = next((p for p in (128, 256, 512) if kv_rank <= p), -(-kv_rank // 64) * 64)
    rdp = next((p for p in (64, 128) if rot_dim <= p), -(-rot_dim // 64) * 64)
    return rp, rdp


def _rotate_halves(x, positions, freq, rd: int):
    """x f32 [T, ..., rd]: dimension i pairs with i + rd / 2, angle position * freq[i]."""
    half = rd // 2
    ang = positions.float().view(-1, *([1] * (x.dim() - 1))) * freq.float()[:half]
    c, s = torch.cos(ang), torch.sin(ang)
    u, v = x[..., :half], x[..., half:rd]
    return torch.cat([u * c - v * s, v * c + u * s], -1)


def latent_prep(u, dq_col: int, q_rank: int, dq_norm, dkv_col: int, kv_rank: int, dkv_norm, rot_dim: int, freq, positions, eps: float,
                cache, slots, rp: int):
    """cq [T, q_rank] = the columns ``[dq_col, dq_col + q_rank)`` of ``u`` divided by their RMS times ``dq_norm`` (f32 arithmetic).
    With ``dkv_norm`` (None: this layer reads another layer's cache) also the token's cache row at ``slots`` (< 0: none): the
    normed latent of the columns behind ``dkv_col`` and the ``rot_dim`` columns that follow, rotated by position."""
    if use_hip(u):
        return lib().latent_prep(u, int(dq_col), int(q_rank), dq_norm, int(dkv_col), int(kv_rank), dkv_norm, int(rot_dim), freq, positions,
                                 float(eps), cache, slots, int(rp))
    T = u.shape[0]

    def rms(x, w):
        return x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps) * w

    cq = rms(u[:, dq_col:dq_col + q_rank].float(), dq_norm).to(u.dtype)
    if dkv_norm is not None:
        row = torch.zeros(T, cache.shape[2], dtype=torch.float32, device=u.device)
        row[:, :kv_rank] = rms(u[:, dkv_col:dkv_col + kv_rank].float(), dkv_norm)
        kr = u[:, dkv_col + kv_rank:dkv_col + kv_rank + rot_dim].float()
        row[:, rp:rp + rot_dim] = _rotate_halves(kr, positions[:T], freq, rot_dim)
        BS = cache.shape[1]
        sl = slots[:T].long()
        ok = sl >= 0
        cache[sl[ok] // BS, sl[ok] % BS] = row[ok].to(cache.dtype)
    return cq


def latent_query_rot(q, qa, H: int, qdim: int, dim: int, rot_dim: int, freq, positions, rp: int):
    """Rotated parts of the queries: ``q`` rows hold H heads of ``qdim`` columns, ``[dim plain | rot_dim | padding]``; their rotated
    columns go to ``qa[..., rp : rp + rot_dim]`` (``qa`` [T, H, KD]), zeros behind them."""
    if use_hip(q):
        lib().latent_query_rot(q, qa, int(H), int(qdim), int(dim), int(rot_dim), freq, positions, int(rp))
        return qa
    T = q.shape[0]
    r = q[:, : H * qdim].view(T, H, qdim)[..., dim:dim + rot_dim].float()
    qa[..., rp:] = 0
    qa[..., rp:rp + rot_dim] = _rotate_halves(r, positions[:T], freq, rot_dim).to(qa.dtype)
    return qa


def head_linear(x, w, x_head: int, out):
    """Per-head products: ``out[t, h, :N] = w[h] x[t, h * x_head : h * x_head + K]`` for ``w`` [H, N, K] and ``out`` [T, H, >= N]
    (a view whose last dimension is contiguous); f32 accumulation."""
    if use_hip(x):
        lib().head_linear(x, w, int(x_head), out)
        return out
    H, N, K = w.shape
    T = x.shape[0]
    xs = torch.stack([x[:, h * x_head:h * x_head + K] for h in range(H)], 0).float()           # [H, T, K]
    out[..., :N] = torch.bmm(xs, w.float().transpose(1, 2).contiguous()).transpose(0, 1).to(out.dtype)
    return out


def latent_decode_splits(B: int, H: int, span: int) -> int:
    """Workgroups per (sequence, head block) of the decode kernel: about one workgroup per CU, never more than one per 128 keys."""
    blocks = max(1, B * -(-H // 16))
    return int(max(1, min(256 // blocks if blocks <= 256 else 1, -(-span // 128))))


def _rows(qa, kv, qpos, window: int, scale: float, sink, rp: int):
    """qa f32 [S, H, KD] at positions qpos [S]; kv f32 [n, KD] at positions 0 .. n - 1 -> [S, H, rp]."""
    s = torch.einsum("ihd,jd->hij", qa, kv) * scale
    j, i = torch.arange(kv.shape[0], device=kv.device).view(1, -1), qpos.view(-1, 1)
    seen = j <= i
    if window > 0:
        seen = seen & (i - j < window)
    s = s.masked_fill(~seen[None], float("-inf"))
    m = s.amax(-1, keepdim=True)
    if sink is not None:
        m = torch.maximum(m, sink.view(-1, 1, 1))
    e = torch.exp(s - m)
    den = e.sum(-1, keepdim=True) + (torch.exp(sink.view(-1, 1, 1) - m) if sink is not None else 0.0)
    return torch.einsum("hij,jd->ihd", e / den, kv[:, :rp])


def _gather(cache, table, n):
    BS = cache.shape[1]
    return cache[table[: (n + BS - 1) // BS].long()].reshape(-1, cache.shape[2])[:n].float()


def latent_attention_prefill(qa, cache, block_tables, cu_q, ctx_lens, window: int, scale: float, sink, rp: int, out, max_len: int):
    """Query chunks over their sequences' cached rows (their own included).  ``qa`` [T, H, KD]; ``sink`` f32 [H] or None; ``window`` 0:
    causal; ``out`` [T, H, rp] receives the averaged latents."""
    if use_hip(qa):
        lib().latent_attn_prefill(qa, cache, block_tables, cu_q, ctx_lens, int(window), float(scale), sink, int(rp), out, int(max_len))
        return out
    cu = cu_q.tolist()
    for b in range(len(cu) - 1):
        s0, s1 = cu[b], cu[b + 1]
        n = int(ctx_lens[b])
        out[s0:s1] = _rows(qa[s0:s1].float(), _gather(cache, block_tables[b], n), torch.arange(n - (s1 - s0), n, device=qa.device), window,
                           scale, sink, rp).to(out.dtype)
    return out


def latent_attention_decode(qa, cache, block_tables, ctx_lens, window: int, scale: float, sink, rp: int, out, splits: int = 1):
    """One query row per sequence at its last position (ctx - 1)."""
    if use_hip(qa):
        lib().latent_attn_decode(qa, cache, block_tables, ctx_lens, window, float(scale), sink, int(rp), out, int(splits))
        return out
    for b in range(qa.shape[0]):
        n = int(ctx_lens[b])
        if n < 1:
            continue
        out[b:b + 1] = _rows(qa[b:b + 1].float(), _gather(cache, block_tables[b], n), torch.tensor([n - 1], device=qa.device), window, scale,
                             sink, rp).to(out.dtype)
    return out
