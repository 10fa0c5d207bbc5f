"""Entry point of the matrix-memory recurrence with exponential gates (``csrc/mlstm.hip``): per head and sequence, from
log input gates i_t and log forget gates f_t,

    m_t = max(f_t + m_(t-1), i_t)                      m_0 = 0
    S_t = exp(f_t + m_(t-1) - m_t) S_(t-1) + exp(i_t - m_t) k_t v_t^T        n_t likewise with k_t alone
    o_t = S_t^T q_t / (max(|n_t . q_t|, exp(-m_t)) + 1e-6)

all of it f32.  GPU tensors go to the HIP kernels (a chunked matrix form for prompt portions, a state-streaming form for
decode rows); CPU tensors to the loop below.  Sequences of a step are rows ``[cu[s], cu[s+1])`` with state slot
``slots[s]`` (< 0: a padding row), a fresh state when ``positions[cu[s]] == 0``.  State of a layer: ``(S f32 [slots, H, dk,
dv], nm f32 [slots, H, Z, dk + 4])`` -- the normaliser n and, behind it, m, once per block of ``MLSTM_COLS`` state columns
(``Z = ceil(dv / MLSTM_COLS)``: the workgroups of a head own their copy, so none waits for another).
"""
from __future__ import annotations

import torch

from ._ext import lib, use_hip

__all__ = ["mlstm_scan", "mlstm_supported", "mlstm_state", "MLSTM_COLS"]

MLSTM_MAX_DK = 256
MLSTM_COLS = 64          # state columns of a workgroup
DENOM_EPS = 1e-6


def mlstm_supported(dk: int, dv: int) -> bool:
    return 1 <= dk <= MLSTM_MAX_DK and dv >= 1


def mlstm_state(slots: int, H: int, dk: int, dv: int, device):
    return (torch.zeros(slots, H, dk, dv, dtype=torch.float32, device=device),
            torch.zeros(slots, H, -(-dv // MLSTM_COLS), dk + 4, dtype=torch.float32, device=device))


def mlstm_scan(q, k, v, gates, state, cu, slots, positions, H: int, dk: int, dv: int, q_scale: float = 1.0, max_len: int = 1):
    """o f32 [T, H * dv].  q, k: rows of ``H * dk``, v: rows of ``H * dv`` (bf16 or f32; q is multiplied by ``q_scale`` in f32);
    ``gates`` f32 [T, 2 * H]: log input gates, then log forget gates.  ``max_len``: the most rows of a sequence."""
    if use_hip(q):
        return lib().mlstm_scan(q, k, v, gates, state[0], state[1], cu, slots, positions, H, dk, dv, float(q_scale), int(max_len))
    T = q.shape[0]
    o = torch.zeros(T, H * dv, dtype=torch.float32, device=q.device)
    cul, sl = cu.tolist(), slots.tolist()
    Sg, nm = state
    for s in range(len(cul) - 1):
        r0, r1 = cul[s], cul[s + 1]
        if sl[s] < 0 or r1 <= r0:
            continue
        fresh = int(positions[r0]) == 0
        S = torch.zeros_like(Sg[sl[s]]) if fresh else Sg[sl[s]].clone()
        n = torch.zeros_like(nm[sl[s], :, 0, :dk]) if fresh else nm[sl[s], :, 0, :dk].clone()
        m = torch.zeros_like(nm[sl[s], :, 0, dk]) if fresh else nm[sl[s], :, 0, dk].clone()
        qq = (q[r0:r1, : H * dk].float() * q_scale).view(-1, H, dk)
        kk = k[r0:r1, : H * dk].float().view(-1, H, dk)
        vv = v[r0:r1, : H * dv].float().view(-1, H, dv)
        for t in range(r1 - r0):
            i, f = gates[r0 + t, :H], gates[r0 + t, H:2 * H]
            new = torch.maximum(f + m, i)
            a, b = torch.exp(f + m - new), torch.exp(i - new)
            S = a.view(H, 1, 1) * S + (b.view(H, 1) * kk[t]).unsqueeze(-1) * vv[t].unsqueeze(1)
            n = a.view(H, 1) * n + b.view(H, 1) * kk[t]
            m = new
            den = torch.maximum((n * qq[t]).sum(-1).abs(), torch.exp(-m)) + DENOM_EPS
            o[r0 + t] = (torch.einsum("hij,hi->hj", S, qq[t]) / den.view(H, 1)).reshape(-1)
        Sg[sl[s]] = S
        nm[sl[s], :, :, :dk] = n.unsqueeze(1)
        nm[sl[s], :, :, dk] = m.unsqueeze(1)
    return o
