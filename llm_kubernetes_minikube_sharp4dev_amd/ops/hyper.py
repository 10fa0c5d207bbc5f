"""Entry points of the kernels around a residual stream that is kept as several mixed copies
(``csrc/hyper_stream.hip``) and of the skinny projections that stay in f32 (``csrc/row_proj.hip``), with their
CPU implementations:

* ``stream_hyper_norm`` -- one pass over a token's streams: the sublayer's result (dense rows and weighted expert
  rows) written back through the stream mixing matrix, the next sublayer's combination of the streams, its layer norm;
* ``relu_sq_``          -- the square of relu, in place;
* ``gate_proj``         -- log input / log forget gates of a gated recurrence: f32 projections with soft cap and
  log-sigmoid;
* ``router_choice``     -- f32 router logits, softmax or sigmoid scores, choice scores with a correction, group-limited
  choice, normalised weights.
"""
from __future__ import annotations

import torch
import torch.nn.functional as F

from ._ext import lib, use_hip

__all__ = ["stream_hyper_norm", "relu_sq_", "gate_proj", "router_choice", "SCORE_SIGMOID", "SCORE_SOFTMAX", "GROUP_TOP2", "GROUP_MAX"]

SCORE_SIGMOID, SCORE_SOFTMAX = 0, 1      # how router logits become scores
GROUP_TOP2, GROUP_MAX = 0, 1             # a group's score: the sum of its two largest choice scores, or the largest
WEIGHT_SUM_FLOOR = 1e-20                 # added to the sum of the chosen scores before the division
MAX_STREAMS = 8


def stream_hyper_norm(x, streams: int, a=None, b=None, y=None, y_w=None, mix=None, w_out=None, w_in=None, norm_w=None,
                      eps: float = 1e-6, out_dtype=torch.bfloat16, idx=None, out_scale: float = 1.0):
    """One sublayer boundary of a stream kept as ``streams`` copies X_s (f32): with a sublayer result ``r = a + b +
    sum_k y_w[t, k] y[t * top + k]`` (any of the terms may be None; all None: no update)

        X_t <- sum_s mix[s, t] X_s + w_out[t] r          all t at once from the old copies
        u = sum_s w_in[s] X_s                            (w_in None: ones)
        h = (u - mean) / sqrt(var + eps) * norm_w * out_scale

    ``x``: f32 [T, streams, W], updated in place, or f32 [T, W] while all copies are still equal (an update then
    returns a new [T, streams, W]).  ``a``, ``b`` [T, W], ``y`` [T * top, W] activations; ``y_w`` f32 [T, top].
    ``norm_w`` None: no ``h``.  ``idx`` (int64 rows, no update): only those rows are normed.  Returns (x, h)."""
    if use_hip(x):
        return tuple(lib().stream_hyper_norm(x, int(streams), a, b, y, y_w, mix, w_out, w_in, norm_w, float(eps), out_dtype, idx,
                                             float(out_scale)))
    T, W = x.shape[0], x.shape[-1]
    r = None
    for t in (a, b):
        if t is not None:
            r = t.float() if r is None else r + t.float()
    if y is not None:
        e = (y.float().view(T, -1, W) * y_w.view(T, -1, 1)).sum(1)
        r = e if r is None else r + e
    X = x if x.dim() == 3 else x.view(T, 1, W).expand(T, streams, W)
    if r is not None:
        new = torch.einsum("tsw,so->tow", X, mix) + w_out.view(1, streams, 1) * r.unsqueeze(1)
        if x.dim() == 3:
            x.copy_(new)
        else:
            x = new.contiguous()
        X = x
    if norm_w is None:
        return x, None
    if idx is not None:
        X = X.index_select(0, idx)
    u = X.sum(1) if w_in is None else torch.einsum("tsw,s->tw", X, w_in)
    d = u - u.mean(-1, keepdim=True)
    h = d / torch.sqrt(d.pow(2).mean(-1, keepdim=True) + eps) * (norm_w * out_scale)
    return x, h.to(out_dtype)


def relu_sq_(x):
    """``max(x, 0)^2`` in place on a (possibly strided) block of columns."""
    if use_hip(x):
        lib().relu_sq_(x)
        return x
    return x.copy_(F.relu(x.float()).square().to(x.dtype))


def gate_proj(h, w, bias, heads: int, cap: float):
    """f32 [T, 2 * heads]: for ``z = h w^T + bias`` (``w`` [2 * heads, W] in h's dtype, products summed in f32) soft-capped to
    ``c = cap * tanh(z / cap)``, the first ``heads`` columns are ``c`` (log input gates), the others
    ``log sigmoid(c)`` (log forget gates)."""
    if use_hip(h):
        return lib().gate_proj(h, w, bias, int(heads), float(cap))
    c = cap * torch.tanh((h.float() @ w.float().T + bias) / cap)
    return torch.cat([c[:, :heads], F.logsigmoid(c[:, heads:])], 1)


def router_choice(h, w_router, top: int, groups: int = 1, keep: int = 1, scale: float = 1.0, score: int = SCORE_SOFTMAX,
                  correction=None, group_score: int = GROUP_MAX):
    """(experts int32 [T, top], weights f32 [T, top]) for rows ``h`` [T, W] and ``w_router`` [E, W] in h's dtype (logits are f32
    sums).  Scores s = softmax or sigmoid of the logits (evaluated in f64); choice scores are ``s + correction`` (f32 [E] or None);
    the experts form ``groups`` equal groups of neighbours of which only the ``keep`` with the best group score (from
    choice scores) can be chosen; the ``top`` largest choice scores among those (ties: the lower index); weights
    ``s / (sum of the chosen s + 1e-20) * scale``."""
    E = w_router.shape[0]
    if E % groups or not 1 <= keep <= groups or not 1 <= top <= (E // groups) * keep:
        raise ValueError(f"router: {top} of {E} experts in {keep} of {groups} groups")
    if use_hip(h):
        ex, wt = lib().router_choice(h, w_router, int(top), int(groups), int(keep), float(scale), int(score), correction, int(group_score))
        return ex, wt
    z = (h.float() @ w_router.float().T).double()
    s = torch.softmax(z, -1) if score == SCORE_SOFTMAX else torch.sigmoid(z)
    c = s if correction is None else s + correction.double()
    T = c.shape[0]
    if groups > 1:
        per = E // groups
        cg = c.view(T, groups, per)
        gs = cg.amax(-1) if group_score == GROUP_MAX else cg.topk(min(2, per), dim=-1).values.sum(-1)
        best = gs.sort(dim=-1, descending=True, stable=True).indices[:, :keep]
        ok = torch.zeros(T, groups, dtype=torch.bool, device=c.device).scatter_(1, best, True)
        c = c.masked_fill(~ok.repeat_interleave(per, dim=1), float("-inf"))
    ex = c.sort(dim=-1, descending=True, stable=True).indices[:, :top]
    sc = s.gather(1, ex)
    return ex.to(torch.int32), (sc / (sc.sum(-1, keepdim=True) + WEIGHT_SUM_FLOOR) * scale).float()
