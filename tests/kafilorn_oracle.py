"""Plain float64 implementation of the Kafilorn decoder, written from its equations: whole sequences only, one
function per mechanism, loops over tokens and heads where a recurrence, a router or a mask is involved.  It shares no
code with the package (not even its config reader): ``cfg`` is the checkpoint's ``config.json`` as a dict and
``sd`` a dict of tensors under the checkpoint names.

    X_s = embed[token] * scale                                       s = 1 .. streams
    per layer and sublayer q:  u = sum_s in_q[s] X_s;  y = sublayer(ln(u) w);
                               X_t <- sum_s mix_q[s, t] X_s + out_q[t] y          (the feed-forward may be absent)
    logits = logit_scale * head . (ln(sum_s X_s) w_f)                ln(v) = (v - mean) / sqrt(var + eps)
"""
from __future__ import annotations

import math

import torch

F64 = torch.float64


def ln(v, w, eps):
    mu = v.mean(-1, keepdim=True)
    d = v - mu
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms(v, w, eps):
    return v / torch.sqrt((v * v).mean(-1, keepdim=True) + eps) * w


def sigmoid(z):
    return 1.0 / (1.0 + torch.exp(-z))


def silu(z):
    return z * sigmoid(z)


def log_sigmoid(z):
    return -torch.log1p(torch.exp(-z)) if z >= 0 else z - torch.log1p(torch.exp(z))


def rotate_halves(x, pos, dims, base):
    """x [T, n]: dimensions (i, i + dims / 2), i < dims / 2, turned by pos * base^(-2 i / dims); the rest unchanged."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        a = pos.to(F64) * base ** (-2.0 * i / dims)
        u, v = x[:, i], x[:, i + half]
        out[:, i] = u * torch.cos(a) - v * torch.sin(a)
        out[:, i + half] = v * torch.cos(a) + u * torch.sin(a)
    return out


def stream_read(X, w_in):
    """X [T, S, W] -> u [T, W]."""
    return sum(w_in[s] * X[:, s] for s in range(X.shape[1]))


def stream_write(X, mix, w_out, y):
    """All streams at once from the old ones; ``mix`` is indexed [from, to]."""
    S = X.shape[1]
    new = torch.zeros_like(X)
    for t in range(S):
        for s in range(S):
            new[:, t] += mix[s, t] * X[:, s]
        new[:, t] += w_out[t] * y
    return new


def mlstm(h, m, w, eps):
    """Matrix memory with exponential gates and a running maximum that starts at 0."""
    T = h.shape[0]
    H, d, dv, cap = m["heads"], m["dim"], m["vdim"], float(m["gate_cap"])
    q = (h @ w["q"].T).view(T, H, d) * d ** -0.5
    k = (h @ w["k"].T).view(T, H, d)
    v = (h @ w["v"].T).view(T, H, dv)
    ig = cap * torch.tanh((h @ w["i"].T + w["i.b"]) / cap)
    fr = cap * torch.tanh((h @ w["f"].T + w["f.b"]) / cap)
    o = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        S, n, mx = torch.zeros(d, dv, dtype=F64), torch.zeros(d, dtype=F64), torch.zeros((), dtype=F64)
        for t in range(T):
            f = log_sigmoid(fr[t, hd])
            i = ig[t, hd]
            new = torch.maximum(f + mx, i)
            a, b = torch.exp(f + mx - new), torch.exp(i - new)
            S = a * S + b * torch.outer(k[t, hd], v[t, hd])
            n = a * n + b * k[t, hd]
            mx = new
            o[t, hd] = (S.T @ q[t, hd]) / (torch.maximum((n @ q[t, hd]).abs(), torch.exp(-mx)) + 1e-6)
    y = o / torch.sqrt((o * o).mean(-1, keepdim=True) + eps)
    return (y.reshape(T, H * dv) * w["norm"] * sigmoid(h @ w["g"].T)) @ w["o"].T


def latents(h, m, w, eps):
    """The layer's cached pair: normed latent [T, kv_rank] and rotated key part [T, rot_dim]."""
    kvr, r = m["kv_rank"], m["rot_dim"]
    ckv = h @ w["dkv"].T
    return rms(ckv[:, :kvr], w["dkv.norm"], eps), rotate_halves(ckv[:, kvr:], torch.arange(h.shape[0]), r, m["rot"]["base"])


def latent_attention(h, m, w, eps, c, kr):
    """Windowed softmax attention with a sink over keys and values expanded from the latent ``c`` and the common rotated
    key part ``kr`` (this layer's or an earlier layer's)."""
    T = h.shape[0]
    H, d, r, dv = m["heads"], m["dim"], m["rot_dim"], m["vdim"]
    pos = torch.arange(T)
    cq = rms(h @ w["dq"].T, w["dq.norm"], eps)
    q = (cq @ w["uq"].T).view(T, H, d + r)
    ku = (c @ w["uk"].T).view(T, H, d)
    vv = (c @ w["uv"].T).view(T, H, dv)
    dist = torch.arange(T).view(-1, 1) - torch.arange(T).view(1, -1)
    seen = dist >= 0
    if m.get("mask"):
        seen = seen & (dist < m["mask"]["size"])
    out = torch.zeros(T, H, dv, dtype=F64)
    for hd in range(H):
        qr = rotate_halves(q[:, hd, d:], pos, r, m["rot"]["base"])
        s = ((q[:, hd, :d] @ ku[:, hd].T + qr @ kr.T) * m["scale"]).masked_fill(~seen, -math.inf)
        top = torch.maximum(s.max(-1, keepdim=True).values, w["sink"][hd])
        e = torch.exp(s - top)
        out[:, hd] = e / (e.sum(-1, keepdim=True) + torch.exp(w["sink"][hd] - top)) @ vv[:, hd]
    return out.reshape(T, H * dv) @ w["o"].T


def dense_ff(h, w):
    return torch.clamp(h @ w["up"].T, min=0.0) ** 2 @ w["down"].T


def expert(h, w, p):
    return (silu(h @ w[p + "gate"].T) * (h @ w[p + "up"].T)) @ w[p + "down"].T


def route(z, r, correction):
    """z [E] router logits -> (chosen experts, weights)."""
    E, top = r["experts"], r["top"]
    e = torch.exp(z - z.max())
    s = e / e.sum()
    choice = s + correction
    gr = r.get("groups")
    if gr:
        n = E // gr["count"]
        gs = torch.stack([choice[a * n:(a + 1) * n].max() for a in range(gr["count"])])
        best = set(gs.sort(descending=True, stable=True).indices[:gr["keep"]].tolist())
        for a in range(gr["count"]):
            if a not in best:
                choice = choice.clone()
                choice[a * n:(a + 1) * n] = -math.inf
    chosen = choice.sort(descending=True, stable=True).indices[:top]
    return chosen.tolist(), s[chosen] / (s[chosen].sum() + 1e-20)


def moe_ff(h, mlp, w):
    T = h.shape[0]
    z = h @ w["router"].T
    corr = w["correction"] if "correction" in w else torch.zeros(z.shape[1], dtype=F64)
    out = torch.zeros(T, w["e0.down"].shape[0], dtype=F64)
    for t in range(T):
        chosen, wgt = route(z[t], mlp["router"], corr)
        for e, a in zip(chosen, wgt):
            out[t] += a * expert(h[t:t + 1], w, f"e{e}.")[0]
    if mlp.get("shared"):
        out = out + expert(h, w, "shared.")
    return out


def forward(cfg: dict, sd: dict, tokens, return_streams: bool = False):
    """-> logits [T, vocab] float64 (and the sum of the streams after every layer)."""
    sd = {k: v.to(F64) for k, v in sd.items()}
    eps, S = cfg["norm"]["eps"], cfg["streams"]
    x0 = sd["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    X = torch.stack([x0] * S, dim=1)
    streams, lat = [], {}
    for i, L in enumerate(cfg["layers"]):
        p = f"l{i}."
        wm = {k[len(p) + 4:]: v for k, v in sd.items() if k.startswith(p + "mix.")}
        m = L["mixer"]
        h = ln(stream_read(X, sd[p + "hc1.in"]), sd[p + "norm1"], eps)
        if L["type"] == "mlstm":
            y = mlstm(h, m, wm, eps)
        elif L["type"] == "latent_attention":
            src = m.get("kv_from")
            if src is None:
                src = i
                lat[i] = latents(h, m, wm, eps)
            y = latent_attention(h, m, wm, eps, *lat[src])
        else:
            raise ValueError(L["type"])
        X = stream_write(X, sd[p + "hc1.mix"], sd[p + "hc1.out"], y)
        if L.get("mlp"):
            wf = {k[len(p) + 4:]: v for k, v in sd.items() if k.startswith(p + "mlp.")}
            h = ln(stream_read(X, sd[p + "hc2.in"]), sd[p + "norm2"], eps)
            y = dense_ff(h, wf) if L["mlp"]["kind"] == "dense" else moe_ff(h, L["mlp"], wf)
            X = stream_write(X, sd[p + "hc2.mix"], sd[p + "hc2.out"], y)
        streams.append(X.sum(1))
    logits = ln(X.sum(1), sd["final.norm"], eps) @ sd["head"].T * cfg["logit_scale"]
    return (logits, streams) if return_streams else logits
