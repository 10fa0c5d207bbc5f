"""The Kafilorn decoder's mechanisms, each alone, against the plain float64 implementations of
``kafilorn_oracle``: the framework's mixers over a paged cache / state slots, whole sequences, cut into
portions and decoded token by token, on the CPU path and (``gpu`` marker) on the HIP kernels in f32 and
bf16.  Where random weights would hide a fault (a window's edge, a far key, a sink, a group that shuts a high score
out) the weights and inputs are made so that it shows."""
import math

import pytest
import torch

import kafilorn_oracle as O
from llm_kubernetes_minikube_sharp4dev_amd import ops
from llm_kubernetes_minikube_sharp4dev_amd.models import KafilornConfig, build_decoder
from test_fusasun_mixers import q16, rel_err, rnd, step_meta, tol

CPU32 = pytest.param("cpu", torch.float32, id="cpu-f32")
GPU32 = pytest.param("cuda", torch.float32, id="gpu-f32", marks=pytest.mark.gpu)
GPU16 = pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)
ALL = [CPU32, GPU32, GPU16]
BS = 16
EPS = 1e-5


def model_of(layers, W, device, dtype, seed=5, sd=None):
    """A model of bare layers [(type, mixer)] (random weights through the checkpoint names, or ``sd``); its mixers' tensors."""
    cfg = KafilornConfig.from_json({"architecture": "Kafilorn", "vocab": 11, "width": W, "norm": {"eps": EPS}, "streams": 2,
                                    "embedding": {"scale": 1.0}, "logit_scale": 1.0,
                                    "layers": [{"type": t, "mixer": m, "mlp": None} for t, m in layers]})
    m = build_decoder(cfg, device=device, dtype=dtype, seed=seed)
    if sd is not None:
        full = {k: v.cpu() for k, v in m.native_state_dict().items()}
        full.update(sd)
        m.load_state_dict_native(full)
    w = [{} for _ in layers]
    for k, v in m.native_state_dict().items():
        if ".mix." in k and ".hc" not in k:
            i, name = k.split(".mix.", 1)
            w[int(i[1:])][name] = v.cpu().double()
    return m, w


def run_mixers(m, h, cuts, device, dtype, slot=1, nblocks=40, caches=None):
    """Every layer's mixer over the same ``h`` [T, W] fed in portions of the sizes ``cuts`` (the rest as decode rows)."""
    T = h.shape[0]
    blocks = list(range(nblocks - 1, nblocks - 1 - (T + BS - 1) // BS, -1))   # pages in descending order
    caches = caches or m.make_caches(nblocks, BS, 3)
    out, at, sizes = [[] for _ in m.layers], 0, list(cuts)
    while at < T:
        dec = not sizes
        n = 1 if dec else min(sizes.pop(0), T - at)
        meta = step_meta([(at, n, blocks, slot, dec)], device)
        with torch.inference_mode():
            for i, L in enumerate(m.layers):
                y = m._mixer(L, h[at:at + n].to(dtype).to(device).contiguous(), meta, caches[i])
                out[i].append(y.float().cpu())
        at += n
    return [torch.cat(o) for o in out]


def leftovers(m, g, nblocks=40):
    """Caches and states that hold another sequence's finite leftovers."""
    caches = m.make_caches(nblocks, BS, 3)
    for c in caches:
        for t in (c if isinstance(c, tuple) else (c,)):
            t.copy_(torch.randn(t.shape, generator=g).to(t.dtype))
    return caches


def mostly(got, want, dtype):
    """Largest error of a row relative to the largest value; in bf16 one row in ten may differ more: the matrix memory's first
    outputs are a near-zero dot product times a value, which the unit norm that follows blows up to order one, so a
    rounding of q or k may turn them."""
    err = (got.double() - want).abs().amax(-1) / want.abs().max()
    if dtype == torch.float32:
        return float(err.max()) < tol(dtype), float(err.max())
    over = int((err > tol(dtype)).sum())
    return over <= max(1, err.numel() // 10), (over, float(err.max()))


MLS = {"heads": 3, "dim": 10, "vdim": 14, "gate_cap": 6.0}
LAT = {"heads": 3, "dim": 12, "rot_dim": 6, "vdim": 20, "q_rank": 14, "kv_rank": 18, "scale": 0.4, "rot": {"dims": 6, "base": 30.0},
       "mask": {"size": 13}}
SHARED = {"heads": 5, "dim": 8, "rot_dim": 6, "vdim": 10, "q_rank": 9, "kv_rank": 18, "scale": 0.25, "rot": {"dims": 6, "base": 30.0},
          "mask": {"size": 21}, "kv_from": 0}


@pytest.mark.parametrize("device,dtype", ALL)
def test_matrix_memory_mixer_whole_tokenwise_and_portions(device, dtype):
    W = 40
    m, w = model_of([("mlstm", MLS)], W, device, dtype)
    g = torch.Generator().manual_seed(1)
    h = q16(rnd(g, 53, W))
    want = O.mlstm(h, MLS, w[0], EPS)
    for cuts in ([53], [], [2, 3, 16, 2, 11, 5], [31, 2]):
        got = run_mixers(m, h, cuts, device, dtype, caches=leftovers(m, g))[0]
        ok, err = mostly(got, want, dtype)
        assert ok, (cuts, err)


@pytest.mark.parametrize("device,dtype", ALL)
def test_latent_mixers_whole_tokenwise_and_portions(device, dtype):
    """A layer with its own latent and a second one -- other heads, sizes, window and scale -- that reads the first one's cache:
    whole, one token per step, portions down to two tokens, over pages in descending order that hold leftovers."""
    W = 40
    m, w = model_of([("latent_attention", LAT), ("latent_attention", SHARED)], W, device, dtype)
    assert "dkv" not in w[1] and m.layers[1].mix.spec.bytes_per_token(dtype) == 0
    caches = m.make_caches(40, BS, 3)
    assert caches[1] is caches[0]
    g = torch.Generator().manual_seed(1)
    h = q16(rnd(g, 53, W))
    pair = O.latents(h, LAT, w[0], EPS)
    want = [O.latent_attention(h, LAT, w[0], EPS, *pair), O.latent_attention(h, SHARED, w[1], EPS, *pair)]
    for cuts in ([53], [], [2, 3, 16, 2, 11, 5], [31, 2]):
        got = run_mixers(m, h, cuts, device, dtype, caches=leftovers(m, g))
        for i in range(2):
            assert rel_err(got[i], want[i]) < tol(dtype), (cuts, i, rel_err(got[i], want[i]))


def copy_latent(size, by_latent, H=2, R=12, rd=4, sinks=(-3.0, 1.0)):
    """A latent attention layer whose projections copy input columns, so that a test writes latents and the common key part
    directly.  Input: [1 | R latent columns | rd key columns].  A latent that is one unit vector leaves its norm as sqrt(R) times
    it; values are the latent / sqrt(R).  Queries are constant: they meet latent dimension 1 (``by_latent``) or the last pair of
    the rotated part, whose frequency is 1e-6 (no turn within a test)."""
    W = 1 + R + rd
    dim, qr, vd = 8, 4, R
    m = {"heads": H, "dim": dim, "rot_dim": rd, "vdim": vd, "q_rank": qr, "kv_rank": R, "scale": 1.0, "rot": {"dims": rd, "base": 1e12}}
    if size:
        m["mask"] = {"size": size}
    dq = torch.zeros(qr, W)
    dq[0, 0] = 1.0                                      # rms norm: sqrt(qr) e_0
    uq = torch.zeros(H, dim + rd, qr)
    uk, uv = torch.zeros(H, dim, R), torch.zeros(H, vd, R)
    if by_latent:
        uq[:, 2, 0] = 1.0 / math.sqrt(qr)
        uk[:, 2, 1] = 12.0 / math.sqrt(R)
    else:
        uq[:, dim + 1, 0] = 1.0 / math.sqrt(qr)         # pair (1, 3) of 4
    for j in range(R):
        uv[:, j, j] = 1.0 / math.sqrt(R)
    dkv = torch.zeros(R + rd, W)
    dkv[:, 1:] = torch.eye(R + rd)
    o = torch.zeros(W, H * vd)
    o[:R, :R] = torch.eye(R)                            # head 0's values, head 1's marker column behind them
    o[R, vd + 1] = 1.0
    sd = {"dq": dq, "dq.norm": torch.ones(qr), "uq": uq.view(-1, qr), "dkv": dkv, "dkv.norm": torch.ones(R), "uk": uk.view(-1, R),
          "uv": uv.view(-1, R), "sink": torch.tensor(sinks), "o": o}
    return W, m, {"l0.mix." + k: v for k, v in sd.items()}


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("size,star,by_latent", [(13, 3, True), (13, 20, False), (16, 0, True), (16, 15, False), (1, 9, True), (32, 1, False),
                                                (33, 16, True), (64, 0, False)])
def test_window_edge(size, star, by_latent, device, dtype):
    """One key made to stand out at position ``star``: every query sees its marker while the key is inside its window and loses
    it on the very next position -- in a whole prompt, token by token, and with portions cut at the window's edge."""
    T, R = 90, 12
    W, mixer, sd = copy_latent(size, by_latent)
    m, w = model_of([("latent_attention", mixer)], W, device, dtype, sd=sd)
    h = torch.zeros(T, W, dtype=torch.float64)
    h[:, 0] = 1.0
    h[:, 1] = 1.0                                       # ordinary latents: e_0
    h[star, 1], h[star, 2] = 0.0, 1.0                   # the star's: e_1, the marker
    if not by_latent:
        h[star, 1 + R + 1] = 12.0                       # and a common key part that scores 12
    want = O.latent_attention(h, mixer, w[0], EPS, *O.latents(h, mixer, w[0], EPS))
    seen = torch.tensor([star <= i and i - star < size for i in range(T)])
    assert bool((want[seen, 1] > 0.5).all()) and bool((want[~seen, 1].abs() < 1e-9).all()) and 0 < int(seen.sum()) < T
    for cuts in ([T], [], [star + size - 1, 2, 2], [star + 1, size - 1, 3], [star + size, 40]):
        got = run_mixers(m, h, [c for c in cuts if c > 0], device, dtype)[0]
        assert rel_err(got, want) < tol(dtype), (cuts, rel_err(got, want))
        assert bool((got[seen, 1] > 0.5).all()) and bool((got[~seen, 1].abs() < 1e-3).all()), cuts


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("size", [None, 450, 64])
def test_far_key_among_hundreds(size, device, dtype):
    """A key 400 positions back among random ones, reachable or not: prompt in two portions, then decode rows over many pages."""
    T, R, star = 420, 12, 2
    W, mixer, sd = copy_latent(size, False)
    m, w = model_of([("latent_attention", mixer)], W, device, dtype, sd=sd)
    g = torch.Generator().manual_seed(3)
    h = q16(rnd(g, T, W, scale=0.3))
    h[:, 0] = 1.0
    h[:, 2] = 0.0
    h[:, 1 + R:] *= 0.3
    h[star, 1:1 + R] = 0.0
    h[star, 2] = 1.0
    h[star, 1 + R + 1] = 14.0
    want = O.latent_attention(h, mixer, w[0], EPS, *O.latents(h, mixer, w[0], EPS))
    far = want[400:, 1]
    assert bool((far > 0.9).all()) if size is None or size > 400 else bool((far.abs() < 0.1).all())
    got = run_mixers(m, h, [200, 190], device, dtype)[0]
    assert rel_err(got, want) < tol(dtype), rel_err(got, want)


@pytest.mark.parametrize("device,dtype", ALL)
def test_sink_weighs_the_average(device, dtype):
    """Uniform scores of 0 over n visible keys with equal values: the output is n / (n + e^sink) of the value, per head its own
    sink -- far below the scores, equal to them, far above; it counts once however the keys are cut."""
    W, mixer, sd = copy_latent(16, False, sinks=(math.log(3.0), 6.0))
    mixer = dict(mixer, heads=2)
    m, w = model_of([("latent_attention", mixer)], W, device, dtype, sd=sd)
    T, R = 40, 12
    h = torch.zeros(T, W, dtype=torch.float64)
    h[:, 0] = 1.0
    h[:, 2] = 16.0                                      # (large against eps: the normed latent is sqrt(R) e_1)
    n = torch.arange(1, T + 1).clamp(max=16).double()
    sk = w[0]["sink"]
    for cuts in ([T], [], [2, 2, 30]):
        got = run_mixers(m, h, cuts, device, dtype)[0].double()
        assert rel_err(got[:, 1], n / (n + torch.exp(sk[0]))) < tol(dtype), cuts
        assert rel_err(got[:, R], n / (n + torch.exp(sk[1]))) < tol(dtype), cuts


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("H,R,rd,window,bs", [(8, 96, 32, 50, 16), (3, 40, 8, 20, 16), (16, 300, 64, 0, 16), (20, 200, 72, 65, 32), (1, 128, 64, 7, 16),
                                             (40, 256, 64, 33, 16), (2, 600, 16, 50, 16)])
def test_latent_attention_of_many_shapes(H, R, rd, window, bs, device, dtype):
    """The attention over cached rows alone: head counts that fill and do not fill a tile, latents of every kernel instance and
    beyond, pages of 16 and 32, three sequences of a step, decode with 1 to 3 key splits, with and without sinks."""
    g = torch.Generator().manual_seed(H)
    rp, rdp = ops.latent_row(R, rd)
    KD, NB = rp + rdp, 32
    cache = torch.zeros(NB, bs, KD, dtype=torch.float64)
    cache[..., :R], cache[..., rp:rp + rd] = q16(rnd(g, NB, bs, R)), q16(rnd(g, NB, bs, rd))
    ctx, lens = [70, 50, 130], [70, 2, 33]
    nb = -(-max(ctx) // bs)
    bt = torch.stack([torch.randperm(NB, generator=g)[:nb] for _ in ctx]).to(torch.int32)
    qa = torch.zeros(105, H, KD, dtype=torch.float64)
    qa[..., :R], qa[..., rp:rp + rd] = q16(rnd(g, 105, H, R, scale=0.4)), q16(rnd(g, 105, H, rd, scale=0.4))
    sink = rnd(g, H, scale=2.0).float()
    scale = 0.15
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)   # noqa: E731
    dev = lambda t: t.to(dtype).to(device)   # noqa: E731

    def want_row(q, b, pos, sk):
        keys = cache[bt[b].long()].reshape(-1, KD)[:pos + 1]
        s = (q @ keys.T) * scale
        if window:
            s[:, :max(0, pos - window + 1)] = -math.inf
        e = torch.exp(s - s.max())
        den = e.sum(-1) + (torch.exp(sk.double() - s.max()) if sk is not None else 0.0)
        return (e / den[:, None]) @ keys[:, :rp]

    for sk in (sink, None):
        skd = sk.to(device) if sk is not None else None
        out = torch.empty(105, H, rp, dtype=dtype, device=device)
        ops.latent_attention_prefill(dev(qa), dev(cache), bt.to(device), i32([0, 70, 72, 105]), i32(ctx), window, scale, skd, rp, out, 70)
        want = torch.stack([want_row(qa[r], b, ctx[b] - lens[b] + i, sk) for b, r0 in ((0, 0), (1, 70), (2, 72)) for i, r in
                            enumerate(range(r0, r0 + lens[b]))])
        assert rel_err(out, want) < tol(dtype), rel_err(out, want)
        want = torch.stack([want_row(qa[b], b, ctx[b] - 1, sk) for b in range(3)])
        for Z in (1, 2, 3):
            out = torch.empty(3, H, rp, dtype=dtype, device=device)
            ops.latent_attention_decode(dev(qa[:3]).contiguous(), dev(cache), bt.to(device), i32(ctx), window, scale, skd, rp, out, splits=Z)
            assert rel_err(out, want) < tol(dtype), (Z, rel_err(out, want))


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("H,R,window", [(4, 96, 0), (16, 128, 45), (5, 200, 61), (16, 500, 0), (3, 512, 70), (2, 600, 50)])
def test_latent_attention_with_scores_that_climb_and_fall_far(H, R, window, device, dtype):
    """Scores that pass those of the first keys by 50 and then by 90 or 160 nats (head by head also falling, and level): the
    weights stay those of a softmax over all keys, whichever tile the largest score lies in, for prompts cut anywhere
    and for decoded rows with 1 to 3 key splits."""
    g = torch.Generator().manual_seed(R)
    rp, rdp = ops.latent_row(R, 16)
    KD, n, scale = rp + rdp, 130, 0.25
    level = torch.zeros(n, dtype=torch.float64)
    level[40:77], level[77:], level[101], level[118:] = 50.0, 90.0, 160.0, 158.0
    rows = torch.zeros(n, KD, dtype=torch.float64)
    rows[:, :R], rows[:, rp] = q16(rnd(g, n, R)), q16(level / scale)
    bt = torch.randperm(12, generator=g)[:9].to(torch.int32)[None]
    cache = torch.zeros(12, BS, KD, dtype=torch.float64)
    for i in range(n):
        cache[int(bt[0, i // BS]), i % BS] = rows[i]
    qa = torch.zeros(n, H, KD, dtype=torch.float64)
    qa[..., :R] = q16(rnd(g, n, H, R, scale=1.0 / math.sqrt(R)))
    qa[..., rp] = torch.tensor([1.0, -1.0, 0.0])[torch.arange(H) % 3]
    sink = (2.0 * torch.arange(H) - 3.0).float()
    sink[0] = 60.0
    s = torch.einsum("qhk,jk->qhj", qa, rows) * scale
    d = torch.arange(n)[:, None] - torch.arange(n)[None]
    s = s.masked_fill(((d < 0) | ((d >= window) if window else (d < 0)))[:, None], -math.inf)
    full = torch.cat([s, sink.double()[None, :, None].expand(n, H, 1)], -1)
    want = torch.einsum("qhj,jr->qhr", torch.softmax(full, -1)[..., :-1], rows[:, :rp])
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)   # noqa: E731
    dev = lambda t: t.to(dtype).to(device)   # noqa: E731
    for lo, hi in ((0, n), (0, 41), (41, 78), (78, 103), (103, n)):
        out = torch.empty(hi - lo, H, rp, dtype=dtype, device=device)
        ops.latent_attention_prefill(dev(qa[lo:hi]), dev(cache), bt.to(device), i32([0, hi - lo]), i32([hi]), window, scale, sink.to(device), rp, out,
                                     hi - lo)
        assert rel_err(out, want[lo:hi]) < tol(dtype), (lo, hi, rel_err(out, want[lo:hi]))
    at = [1, 41, 78, 102, 103, 119, n]
    for Z in (1, 2, 3):
        out = torch.empty(len(at), H, rp, dtype=dtype, device=device)
        ops.latent_attention_decode(dev(qa[[a - 1 for a in at]]), dev(cache), bt.expand(len(at), -1).contiguous().to(device), i32(at), window, scale,
                                    sink.to(device), rp, out, splits=Z)
        assert rel_err(out, want[[a - 1 for a in at]]) < tol(dtype), (Z, rel_err(out, want[[a - 1 for a in at]]))


def scan_reference(q, k, v, ig, f, scale):
    """q, k [T, H, dk], v [T, H, dv], gates [T, H] (log domain), one sequence from zero."""
    T, H, dk = q.shape
    o = torch.zeros(T, H, v.shape[2], dtype=torch.float64)
    for h in range(H):
        S, n, m = torch.zeros(dk, v.shape[2], dtype=torch.float64), torch.zeros(dk, dtype=torch.float64), torch.zeros((), dtype=torch.float64)
        for t in range(T):
            new = torch.maximum(f[t, h] + m, ig[t, h])
            a, b = torch.exp(f[t, h] + m - new), torch.exp(ig[t, h] - new)
            S, n, m = a * S + b * torch.outer(k[t, h], v[t, h]), a * n + b * k[t, h], new
            qq = q[t, h] * scale
            o[t, h] = (S.T @ qq) / (torch.maximum((n @ qq).abs(), torch.exp(-m)) + 1e-6)
    return o


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("H,dk,dv,lens", [(2, 48, 40, [37, 1, 20]), (3, 10, 70, [3, 7, 2]), (1, 128, 128, [200]), (2, 16, 24, [64, 5]),
                                         (1, 200, 130, [50, 33]), (3, 12, 18, [30, 9, 1])])
def test_matrix_memory_scan_and_slot_reuse(H, dk, dv, lens, device, dtype):
    """The recurrence alone on exact operands: several sequences of a step (both kernel forms), each then continued in a second
    and a third step of other lengths; slots that held another sequence's state; a padding row."""
    g = torch.Generator().manual_seed(dk)
    state = ops.mlstm_state(len(lens) + 2, H, dk, dv, device)
    for t in state:
        t.copy_(torch.randn(t.shape, generator=g))
    slots = list(range(len(lens), 0, -1))
    more = [[1] * len(lens), [9 + i for i in range(len(lens))]]
    total = [n + sum(m[i] for m in more) for i, n in enumerate(lens)]
    Q, K, V = ([q16(rnd(g, n, H, d)) for n in total] for d in (dk, dk, dv))
    I = [rnd(g, n, H, scale=3.0).float().double() for n in total]
    F = [torch.nn.functional.logsigmoid(rnd(g, n, H, scale=3.0) + 1.0).float().double() for n in total]
    want = [scan_reference(q, k, v, i, f, 0.3) for q, k, v, i, f in zip(Q, K, V, I, F)]
    got, at = [[] for _ in lens], [0] * len(lens)
    for step in [lens] + more:
        rows = lambda X: torch.cat([x[a:a + n].reshape(n, -1) for x, a, n in zip(X, at, step)] + [torch.zeros(1, X[0][0].numel(), dtype=torch.float64)])   # noqa: E731,B023
        cu = [0]
        for n in step:
            cu.append(cu[-1] + n)
        cu.append(cu[-1] + 1)                              # one padding row behind the sequences
        pos = [p for a, n in zip(at, step) for p in range(a, a + n)] + [0]
        i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)   # noqa: E731
        dev = lambda t: t.to(dtype).to(device).contiguous()   # noqa: E731
        o = ops.mlstm_scan(dev(rows(Q)), dev(rows(K)), dev(rows(V)), torch.cat([rows(I), rows(F)], 1).float().to(device), state, i32(cu),
                           i32(slots + [-1]), i32(pos), H, dk, dv, 0.3, max(step)).cpu()
        assert float(o[-1].abs().max()) == 0.0
        for s, n in enumerate(step):
            got[s].append(o[cu[s]:cu[s + 1]].view(n, H, dv))
            at[s] += n
    for a, b in zip(got, want):
        a = torch.cat(a).double()
        err = (a - b).abs().amax(-1) / b.abs().amax(-1).clamp(min=1e-3)
        assert float(err.max()) < 1e-3 and float(err.median()) < 1e-5, (float(err.max()), float(err.median()))


@pytest.mark.parametrize("device,dtype", ALL)
def test_matrix_memory_keeps_a_value_for_hundreds_of_tokens(device, dtype):
    """Open forget gates and one strong write at position 4: the value answers its key 300 tokens later; closed forget gates: it
    is gone after a few."""
    H, dk, dv, T = 1, 16, 16, 330
    g = torch.Generator().manual_seed(7)
    k, v = q16(rnd(g, T, H, dk, scale=0.05)), q16(rnd(g, T, H, dv, scale=0.05))
    k[4, 0] = 0.0
    k[4, 0, 3] = 4.0
    v[4, 0] = 0.0
    v[4, 0, 7] = 8.0
    q = torch.zeros(T, H, dk, dtype=torch.float64)
    q[:, 0, 3] = 1.0
    ig = torch.full((T, H), -2.0, dtype=torch.float64)
    ig[4] = 3.0
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=device)   # noqa: E731
    for fg, kept in ((-1e-4, True), (-2.0, False)):
        f = torch.full((T, H), fg, dtype=torch.float64)
        want = scan_reference(q, k, v, ig, f, 1.0)
        assert (float(want[-1, 0, 7]) > 1.0) == kept
        for cuts in ([T], [100, 100, 2] + [1] * 128):
            state = ops.mlstm_state(2, H, dk, dv, device)
            got, at = [], 0
            for n in cuts:
                sl = slice(at, at + n)
                dev = lambda t: t[sl].reshape(n, -1).to(dtype).to(device)   # noqa: E731,B023
                got.append(ops.mlstm_scan(dev(q), dev(k), dev(v), torch.cat([ig[sl], f[sl]], 1).float().to(device), state, i32([0, n]), i32([1]),
                                          i32(list(range(at, at + n))), H, dk, dv, 1.0, n).cpu())
                at += n
            got = torch.cat(got).view(T, H, dv).double()
            assert rel_err(got, want) < 1e-4, (fg, cuts[:3], rel_err(got, want))


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("T,H,W", [(5, 2, 36), (40, 3, 37), (33, 40, 256)])
def test_gates_cap_and_log_sigmoid(T, H, W, device, dtype):
    g = torch.Generator().manual_seed(W)
    h, w = q16(rnd(g, T, W)), q16(rnd(g, 2 * H, W, scale=2.0))           # sums far beyond the cap
    b = rnd(g, 2 * H).float()
    cap = 3.5
    got = ops.gate_proj(h.to(dtype).to(device), w.to(dtype).to(device), b.to(device), H, cap)
    assert got.dtype == torch.float32
    z = h @ w.T + b.double()
    c = cap * torch.tanh(z / cap)
    want = torch.cat([c[:, :H], torch.tensor([[float(O.log_sigmoid(x)) for x in r] for r in c[:, H:]])], 1)
    assert rel_err(got, want) < 1e-5
    assert float(z.abs().max()) > 2 * cap and float(got[:, :H].max()) <= cap + 1e-5 and float(got[:, H:].max()) < 0


def route_both(h, wr, r, corr, device, dtype):
    gr = r.get("groups") or {"count": 1, "keep": 1}
    return ops.router_choice(h.to(dtype).to(device), wr.to(dtype).to(device), r["top"], gr["count"], gr["keep"],
                             correction=None if corr is None else corr.float().to(device))


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("E,groups,keep,top", [(16, 4, 2, 3), (6, 3, 2, 2), (4, 4, 2, 2), (8, 1, 1, 3), (5, 1, 1, 5), (64, 8, 4, 8), (1, 1, 1, 1),
                                              (12, 2, 1, 6), (200, 10, 3, 4), (320, 1, 1, 2)])
def test_router_against_the_oracle(E, groups, keep, top, device, dtype):
    g = torch.Generator().manual_seed(E)
    W, T = 24, 37
    h = q16(rnd(g, T, W))
    wr, corr = q16(rnd(g, E, W, scale=0.5)), rnd(g, E, scale=0.3).float().double()
    r = {"experts": E, "top": top}
    if groups > 1:
        r["groups"] = {"count": groups, "keep": keep}
    ex, wt = route_both(h, wr, r, corr, device, dtype)
    assert ex.dtype == torch.int32 and wt.dtype == torch.float32
    z = h @ wr.T
    for t in range(T):
        chosen, wgt = O.route(z[t], r, corr)
        got = dict(zip(ex[t].tolist(), wt[t].tolist()))
        assert sorted(got) == sorted(chosen), t
        for e, a in zip(chosen, wgt.tolist()):
            assert abs(got[e] - a) < 1e-5, (t, e)


@pytest.mark.parametrize("device,dtype", ALL)
def test_router_correction_moves_the_choice_not_the_weights(device, dtype):
    """Scores 0.4 / 0.3 / 0.2 / 0.1 in groups of two.  The correction lifts the weakest expert over the others; its weight stays its own
    small score.  With every choice score of the kept group negative, its experts are still chosen before those of a group that is
    not kept; the group with the largest score but a low correction is left out."""
    s = torch.tensor([0.4, 0.3, 0.2, 0.1], dtype=torch.float64)
    wr = torch.zeros(4, 8, dtype=torch.float64)
    wr[:, 0] = torch.log(s)
    h = torch.zeros(2, 8, dtype=torch.float64)
    h[:, 0] = 1.0
    if dtype == torch.bfloat16:
        s = torch.softmax(q16(wr)[:, 0], 0)
    r1, r2 = {"experts": 4, "top": 2}, {"experts": 4, "top": 2, "groups": {"count": 2, "keep": 1}}
    for r, corr, pick in ((r1, [0.0, 0.0, 0.0, 0.5], [0, 3]), (r2, [0.0, 0.0, 0.0, 0.5], [2, 3]), (r2, [-0.9, -0.9, -0.5, -0.5], [2, 3]),
                          (r2, [-0.5, -0.6, -0.9, -0.9], [0, 1]), (r1, [-1.0] * 4, [0, 1])):
        c = torch.tensor(corr, dtype=torch.float64)
        ex, wt = route_both(h, q16(wr), r, c, device, dtype)
        assert sorted(ex[0].tolist()) == pick == sorted(O.route(q16(wr)[:, 0], r, c)[0]), (corr, ex)
        want = {e: float(s[e] / s[pick].sum()) for e in pick}
        for e, a in zip(ex[1].tolist(), wt[1].tolist()):
            assert abs(a - want[e]) < 5e-3


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("S,W,top", [(1, 36, 1), (2, 256, 2), (3, 1000, 3), (4, 1028, 2), (5, 90, 1), (8, 2050, 2), (4, 4096, 1)])
def test_streams_update_combination_and_norm(S, W, top, device, dtype):
    """One sublayer boundary: all copies at once from the old ones through an unsymmetric matrix indexed [from, to], every subset of
    the sublayer's terms, the next combination and its layer norm (rows with a mean); the first update from equal copies; the
    final norm of picked rows with a scale."""
    g = torch.Generator().manual_seed(W)
    T = 7
    X0 = rnd(g, T, S, W, scale=3.0).float() + 1.0
    a, b = q16(rnd(g, T, W)), q16(rnd(g, T, W))
    y, yw = q16(rnd(g, T * top, W)), rnd(g, T, top).abs().float()
    mix, wo, wi, nw = rnd(g, S, S).float(), rnd(g, S).float(), rnd(g, S).float(), rnd(g, W).float() + 1.0
    dev = lambda t: t.to(device) if t.dtype == torch.float32 else t.to(dtype).to(device)   # noqa: E731
    kw = dict(eps=EPS, out_dtype=dtype)
    for use in ((1, 0, 0), (0, 1, 1), (1, 1, 1), (0, 0, 1)):
        r = use[0] * a + use[1] * b + use[2] * (y.view(T, top, W) * yw.double().view(T, top, 1)).sum(1)
        terms = (dev(a) if use[0] else None, dev(b) if use[1] else None, dev(y) if use[2] else None, dev(yw) if use[2] else None)
        for first in (False, True):
            X = X0[:, :1].expand(T, S, W) if first else X0
            want = O.stream_write(X.double(), mix.double(), wo.double(), r)
            x = X0[:, 0].clone().contiguous().to(device) if first else X0.clone().to(device)
            new, h = ops.stream_hyper_norm(x, S, *terms, dev(mix), dev(wo), dev(wi), dev(nw), **kw)
            assert new.shape == (T, S, W) and (first or new.data_ptr() == x.data_ptr())
            assert rel_err(new, want) < 2e-6
            assert rel_err(h, O.ln(O.stream_read(want, wi.double()), nw.double(), EPS)) < max(tol(dtype), 1e-5)
    x = X0.clone().to(device)
    new, h = ops.stream_hyper_norm(x, S, dev(a), None, None, None, dev(mix), dev(wo), None, None, **kw)
    assert h is None and rel_err(new, O.stream_write(X0.double(), mix.double(), wo.double(), a)) < 2e-6
    x = X0.clone().to(device)
    _, h = ops.stream_hyper_norm(x, S, norm_w=dev(nw), idx=torch.tensor([6, 0], device=device), out_scale=0.3, **kw)
    assert torch.equal(x.cpu(), X0)
    assert rel_err(h, 0.3 * O.ln(X0.double().sum(1), nw.double(), EPS)[[6, 0]]) < max(tol(dtype), 1e-5)


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("T,H,K,N,xh", [(5, 3, 16, 128, 24), (200, 2, 128, 256, 192), (33, 8, 64, 128, 96), (7, 1, 12, 40, 16), (130, 4, 136, 24, 136)])
def test_per_head_products(T, H, K, N, xh, device, dtype):
    g = torch.Generator().manual_seed(T)
    x, w = q16(rnd(g, T, H * xh)), q16(rnd(g, H, N, K, scale=K ** -0.5))
    out = torch.full((T, H, N + 8), 5.0, dtype=dtype, device=device)
    ops.head_linear(x.to(dtype).to(device), w.to(dtype).to(device), xh, out)
    for h in range(H):
        assert rel_err(out[:, h, :N], x[:, h * xh:h * xh + K] @ w[h].T) < tol(dtype)
    assert bool((out[..., N:] == 5.0).all())               # columns behind N are not touched


@pytest.mark.parametrize("device,dtype", ALL)
def test_squared_relu_in_place(device, dtype):
    g = torch.Generator().manual_seed(4)
    x = q16(rnd(g, 5, 52))
    buf = x.to(dtype).to(device).clone()
    ops.relu_sq_(buf[:, 8:44])
    assert rel_err(buf[:, 8:44], x[:, 8:44].clamp(min=0) ** 2) < tol(dtype)
    assert torch.equal(buf[:, :8].cpu().double(), x[:, :8]) and torch.equal(buf[:, 44:].cpu().double(), x[:, 44:])


@pytest.mark.parametrize("device,dtype", ALL)
def test_cache_rows_hold_normed_latent_and_rotated_part(device, dtype):
    """What a step files: the latent over its root mean square times the weight, the common part rotated in halves by the absolute
    position, zeros in the padding columns; rows without a slot file nothing."""
    g = torch.Generator().manual_seed(2)
    T, qr, R, rd = 6, 10, 18, 6
    rp, rdp = ops.latent_row(R, rd)
    u = q16(rnd(g, T, 16 + R + rd, scale=2.0))
    wq, wkv = rnd(g, qr).float(), rnd(g, R).float()
    pos = torch.tensor([0, 1, 7, 500, 2, 31], dtype=torch.int32)
    slots = torch.tensor([17, 3, 31, -1, 0, 40], dtype=torch.int32)
    freq = torch.tensor([30.0 ** (-2.0 * i / rd) for i in range(rd // 2)], dtype=torch.float32)
    cache = torch.full((3, BS, rp + rdp), 9.0, dtype=dtype, device=device)
    cq = ops.latent_prep(u.to(dtype).to(device), 0, qr, wq.to(device), 16, R, wkv.to(device), rd, freq.to(device), pos.to(device), EPS, cache,
                         slots.to(device), rp)
    assert rel_err(cq, O.rms(u[:, :qr], wq.double(), EPS)) < tol(dtype)
    rows = torch.zeros(T, rp + rdp, dtype=torch.float64)
    rows[:, :R] = O.rms(u[:, 16:16 + R], wkv.double(), EPS)
    rows[:, rp:rp + rd] = O.rotate_halves(u[:, 16 + R:], pos, rd, 30.0)
    flat = cache.view(-1, rp + rdp)
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            assert rel_err(flat[s], rows[t]) < tol(dtype)
    assert int((flat[:, 0] == 9.0).sum()) == 3 * BS - 5
    q = q16(rnd(g, T, 3 * 24))
    qa = torch.full((T, 3, rp + rdp), 4.0, dtype=dtype, device=device)
    ops.latent_query_rot(q.to(dtype).to(device), qa, 3, 24, 12, rd, freq.to(device), pos.to(device), rp)
    for h in range(3):
        assert rel_err(qa[:, h, rp:rp + rd], O.rotate_halves(q[:, h * 24 + 12:h * 24 + 18], pos, rd, 30.0)) < tol(dtype)
    assert bool((qa[..., rp + rd:] == 0).all()) and bool((qa[..., :rp] == 4.0).all())
