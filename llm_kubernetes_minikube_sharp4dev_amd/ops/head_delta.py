"""Entry points of the gated delta rule with one decay per head (``csrc/head_delta.hip``), with its CPU implementation:

    g_t = exp(-exp(A_log) softplus(a_t + dt_bias)),  beta_t = sigmoid(b_t)                 one number per head and token
    S <- g_t S;  u = beta_t (v_t - S^T k_t);  S <- S + k_t u^T;  o_t = S^T q_t              S [dk, dv] f32
    out_t = o_t / rms(o_t) * w * silu(gate_t)

with k the unit key of the head and q its unit query times dk^-1/2.  Everything behind the projections and convolutions is f32.
A step of single tokens streams the state once, with norm and gate in the same kernel; steps with prompt portions run in chunks of
16 tokens as masked products (a decay that is the same for all key channels factors out of them).
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ._ext import lib, use_hip
from .delta import _unit

__all__ = ["head_delta", "head_delta_supported"]

HEAD_DELTA_MAX_DK = 256
HEAD_DELTA_MAX_DV = 1024


def head_delta_supported(dk: int, dv: int) -> bool:
    return 1 <= dk <= HEAD_DELTA_MAX_DK and 1 <= dv <= HEAD_DELTA_MAX_DV


def head_delta(q, k, v, b, a, dt_bias, A_log, gate, norm_w, eps: float, state, cu, slots, positions, H: int, Hk: int, dk: int, dv: int, out,
               max_len: int = 1):
    """q, k rows of ``Hk * dk`` (value head h reads q / k head ``h // (H / Hk)``), v rows of ``H * dv``: the convolutions' results in bf16 or
    f32; b, a: rows of H, gate: rows of ``H * dv`` of the same type; ``norm_w`` f32 [H * dv]; ``state`` f32 [slots, H, dk, dv]; sequences of
    the step as rows ``[cu[s], cu[s + 1])`` with state slot ``slots[s]`` (< 0: a padding row, its outputs are zero), from a zero state when
    ``positions[cu[s]] == 0``.  Result in the first ``H * dv`` columns of ``out``."""
    if use_hip(q):
        lib().head_delta(q, k, v, b, a, dt_bias, A_log, gate, norm_w, float(eps), state, cu, slots, positions, H, Hk, dk, dv, out, int(max_len))
        return out
    rep = H // Hk
    cul, sl = cu.tolist(), slots.tolist()
    out[:, : H * dv] = 0
    for s in range(len(cul) - 1):
        r0, r1 = cul[s], cul[s + 1]
        if sl[s] < 0 or r1 <= r0:
            continue
        n = r1 - r0
        S = state[sl[s]].clone() if int(positions[r0]) > 0 else torch.zeros_like(state[sl[s]])
        kk = _unit(k[r0:r1, : Hk * dk].float().reshape(n, Hk, dk)).repeat_interleave(rep, 1)
        qq = (_unit(q[r0:r1, : Hk * dk].float().reshape(n, Hk, dk)) * dk ** -0.5).repeat_interleave(rep, 1)
        vv = v[r0:r1, : H * dv].float().reshape(n, H, dv)
        beta = torch.sigmoid(b[r0:r1, :H].float())
        g = torch.exp(-torch.exp(A_log.float()) * F.softplus(a[r0:r1, :H].float() + dt_bias, threshold=30.0))
        o = torch.empty(n, H, dv)
        for t in range(n):
            S = g[t].view(H, 1, 1) * S
            u = beta[t].view(H, 1) * (vv[t] - torch.einsum("hij,hi->hj", S, kk[t]))
            S = S + kk[t].unsqueeze(-1) * u.unsqueeze(1)
            o[t] = torch.einsum("hij,hi->hj", S, qq[t])
        state[sl[s]] = S
        o = (o / torch.sqrt(o.pow(2).mean(-1, keepdim=True) + eps)).reshape(n, H * dv) * norm_w
        out[r0:r1, : H * dv] = (o * F.silu(gate[r0:r1, : H * dv].float())).to(out.dtype)
    return out
