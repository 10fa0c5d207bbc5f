"""Plain, slow float64 implementations of the Kebepel decoder's mechanisms, written from their
equations, one function per mechanism, over whole sequences (no cache, no chunks, no batching,
token-by-token recurrences).  The tests compare the framework against these; nothing here imports
the package.

Notation: T tokens, W model width; linear weights are [out, in] and applied as W x; ``sd`` maps the
checkpoint's tensor names to float64 tensors; ``p`` is a name prefix such as ``l3.mix.``; ``m`` is a
mixer's dict from config.json.
"""
import math

import torch

F64 = torch.float64


def rms_unit(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, sd, name, eps):
    mu = x.mean(-1, keepdim=True)
    d = x - mu
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * sd[name] + sd[name + ".b"]


def silu(x):
    return x * torch.sigmoid(x)


def softplus(x):
    return torch.where(x > 30.0, x, torch.log1p(torch.exp(torch.clamp(x, max=30.0))))


def l2_unit(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def causal_conv(x, w):
    """x [T, C], w [C, taps]; the last column multiplies the current token; zeros before the start."""
    T, C = x.shape
    taps = w.shape[1]
    y = torch.zeros(T, C, dtype=F64)
    for t in range(T):
        for k in range(taps):
            src = t - (taps - 1) + k
            if src >= 0:
                y[t] += w[:, k] * x[src]
    return y


def biased(h, sd, name):
    return h @ sd[name].T + sd[name + ".b"]


# ------------------------------------------------------------------ attention
def causal_softmax(q, k, v, scale, cap=0.0):
    """q [T, d], k [T, d], v [T, e] of one head: [T, e].  cap > 0: scores become cap * tanh(score / cap)."""
    T = q.shape[0]
    s = (q @ k.T) * scale
    if cap:
        s = cap * torch.tanh(s / cap)
    s = s.masked_fill(torch.ones(T, T, dtype=torch.bool).triu(1), float("-inf"))
    return torch.softmax(s, -1) @ v


def temperature(T, spec):
    """Multiplier of the query at every position."""
    if not spec:
        return torch.ones(T, dtype=F64)
    return torch.tensor([1.0 + spec["coef"] * math.log(math.floor((p + 1) / spec["every"]) + 1.0) for p in range(T)], dtype=F64)


def diff_lambda(sd, p, m):
    return float(torch.exp((sd[p + "lq1"] * sd[p + "lk1"]).sum()) - torch.exp((sd[p + "lq2"] * sd[p + "lk2"]).sum()) + m["diff"])


def diff_attention_core(q, k, v, m, lam, eps):
    """q [T, H, 2, dim] (temperature applied), k [T, G, 2, dim], v [T, G, vdim] -> heads [T, H, vdim], without
    the output gate."""
    T, H = q.shape[0], q.shape[1]
    rep = H // k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    for h in range(H):
        g = h // rep
        a1 = causal_softmax(q[:, h, 0], k[:, g, 0], v[:, g], m["scale"])
        a2 = causal_softmax(q[:, h, 1], k[:, g, 1], v[:, g], m["scale"])
        out[:, h] = rms_unit(a1 - lam * a2, eps) * (1.0 - m["diff"])
    return out


def diff_attention(h, sd, p, m, eps):
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = biased(h, sd, p + "q").view(T, H, 2, d) * temperature(T, m.get("q_temp")).view(T, 1, 1, 1)
    k = biased(h, sd, p + "k").view(T, G, 2, d)
    v = biased(h, sd, p + "v").view(T, G, e)
    o = diff_attention_core(q, k, v, m, diff_lambda(sd, p, m), eps).reshape(T, H * e)
    return (o * torch.sigmoid(h @ sd[p + "g"].T)) @ sd[p + "o"].T


def rotary_table(rot):
    """(frequencies, magnitude of cos and sin)."""
    d, base = rot["dims"], rot["base"]
    f = [base ** (-2.0 * i / d) for i in range(d // 2)]
    s = rot.get("scaling")
    if not s:
        return f, 1.0

    def turns(t):
        return d * math.log(s["original"] / (2.0 * math.pi * t)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(turns(s["fast"])), 0), min(math.ceil(turns(s["slow"])), d - 1)
    out = []
    for i, x in enumerate(f):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(x / s["factor"] * r + x * (1.0 - r))
    return out, 0.1 * math.log(s["factor"]) + 1.0


def rotate_pairs(x, rot):
    """x [T, heads, dim]: dimensions (2 i, 2 i + 1) of the first rot.dims turned by position * frequency."""
    if not rot or not rot.get("dims"):
        return x
    f, mag = rotary_table(rot)
    y = x.clone()
    for t in range(x.shape[0]):
        for i, fi in enumerate(f):
            c, s = math.cos(t * fi) * mag, math.sin(t * fi) * mag
            u, v = x[t, :, 2 * i], x[t, :, 2 * i + 1]
            y[t, :, 2 * i] = u * c - v * s
            y[t, :, 2 * i + 1] = v * c + u * s
    return y


def normed_attention(h, sd, p, m, eps):
    """Softmax attention whose q and k are RMS-normed over the whole projection, then rotated; capped scores,
    element gate."""
    T = h.shape[0]
    H, G, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (rms_unit(biased(h, sd, p + "q"), eps) * sd[p + "q.norm"]).view(T, H, d)
    k = (rms_unit(biased(h, sd, p + "k"), eps) * sd[p + "k.norm"]).view(T, G, d)
    v = biased(h, sd, p + "v").view(T, G, e)
    q, k = rotate_pairs(q, m.get("rot")), rotate_pairs(k, m.get("rot"))
    o = torch.stack([causal_softmax(q[:, i], k[:, i // (H // G)], v[:, i // (H // G)], m["scale"], m.get("softcap") or 0.0) for i in range(H)], 1)
    return (o.reshape(T, H * e) * torch.sigmoid(h @ sd[p + "g"].T)) @ sd[p + "o"].T


# ------------------------------------------------------------------ recurrence
def delta_rule(q, k, v, g, beta, S=None):
    """q, k [T, H, dk], v [T, H, dv], g, beta [T, H] -> (o [T, H, dv], S [H, dk, dv]), token by token."""
    T, H, dk = q.shape
    S = torch.zeros(H, dk, v.shape[2], dtype=F64) if S is None else S.clone()
    o = torch.zeros_like(v)
    for t in range(T):
        for h in range(H):
            S[h] = g[t, h] * S[h]
            u = beta[t, h] * (v[t, h] - S[h].T @ k[t, h])
            S[h] = S[h] + torch.outer(k[t, h], u)
            o[t, h] = S[h].T @ q[t, h]
    return o, S


def gated_delta(h, sd, p, m, eps):
    T = h.shape[0]
    H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (silu(causal_conv(h @ sd[p + n].T, sd[p + n + ".conv"])) for n in ("q", "k", "v"))
    q = (l2_unit(q.view(T, G, dk)) * dk ** -0.5).repeat_interleave(H // G, 1)
    k = l2_unit(k.view(T, G, dk)).repeat_interleave(H // G, 1)
    beta = torch.sigmoid(h @ sd[p + "b"].T)
    g = torch.exp(-torch.exp(sd[p + "A_log"]) * softplus(h @ sd[p + "a"].T + sd[p + "dt_bias"]))
    o, _ = delta_rule(q, k, v.view(T, H, dv), g, beta)
    o = (rms_unit(o, eps) * sd[p + "norm"]).reshape(T, H * dv) * silu(h @ sd[p + "g"].T)
    return o @ sd[p + "o"].T


def parallel(h, sd, p, m, eps):
    return (m["left_scale"] * normed_attention(h, sd, p + "left.", m["left"], eps)
            + m["right_scale"] * gated_delta(h, sd, p + "right.", m["right"], eps))


MIXERS = {"attention": diff_attention, "parallel": parallel}


def dense_ff(h, sd, p):
    return (silu(h @ sd[p + "gate"].T) * (h @ sd[p + "up"].T)) @ sd[p + "down"].T


# ------------------------------------------------------------------ model
def layer_runs(cfg):
    """(layer, pass number where a pass starts, else None) in the order in which they run."""
    n, loop = len(cfg["layers"]), cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    out = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        out += [(i, t if i == a else None) for i in range(a, b)]
    return out + [(i, None) for i in range(b, n)]


def forward(cfg, sd, tokens, streams=False):
    """(logits [T, vocab], the stream after every layer run)."""
    sd = {k: (v.to(F64) if v.is_floating_point() else v) for k, v in sd.items()}
    eps = cfg["norm"]["eps"]
    x = sd["embed"][torch.as_tensor(tokens)]
    taps = []
    for i, t in layer_runs(cfg):
        l, b = cfg["layers"][i], f"l{i}."
        if t is not None:
            x = x + sd["loop.step"][t]
        y = MIXERS[l["type"]](layer_norm(x, sd, b + "norm1", eps), sd, b + "mix.", l["mixer"], eps)
        x = x + layer_norm(y, sd, b + "norm1b", eps)
        if l.get("mlp"):
            y = dense_ff(layer_norm(x, sd, b + "norm2", eps), sd, b + "mlp.")
            x = x + layer_norm(y, sd, b + "norm2b", eps)
        taps.append(x)
    lg = layer_norm(x, sd, "final.norm", eps) @ sd["head"].T
    return (lg, taps) if streams else lg
