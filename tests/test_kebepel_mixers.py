"""The Kebepel decoder's mechanisms, each alone, against the plain float64 implementations of ``kebepel_oracle``: the framework's
mixers over a paged cache / state slots, whole sequences, cut into portions and decoded token by token, on the CPU path and
(``gpu`` marker) on the HIP kernels in f32 and bf16.  Where random weights would hide a fault (a far key, one map's key, a step of the
query temperature, a value written long ago) the inputs are made so that it shows."""
import math

import pytest
import torch

import kebepel_oracle as O
from llm_kubernetes_minikube_sharp4dev_amd import ops
from llm_kubernetes_minikube_sharp4dev_amd.models import KebepelConfig, build_decoder
from llm_kubernetes_minikube_sharp4dev_amd.models.attention import AttnMeta

CPU32 = pytest.param("cpu", torch.float32, id="cpu-f32")
GPU32 = pytest.param("cuda", torch.float32, id="gpu-f32", marks=pytest.mark.gpu)
GPU16 = pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)
ALL = [CPU32, GPU32, GPU16]
BS = 16
EPS = 1e-5


def tol(dtype):
    return 3e-5 if dtype == torch.float32 else 4e-2


def rel_err(got, want):
    want = want.double()
    return float((got.double().cpu() - want).abs().max() / want.abs().max().clamp_min(1e-9))


def rnd(g, *shape, scale=1.0):
    return torch.randn(*shape, generator=g, dtype=torch.float64) * scale


def q16(t):
    """Values a bf16 tensor holds exactly, so both sides of a comparison start from the same numbers."""
    return t.to(torch.bfloat16).to(torch.float64)


def step_meta(seqs, device, bs=BS):
    """AttnMeta of one step, as the model runner lays it out: ``seqs`` = [(start, n, block table, state slot, decode row?)], prompt
    portions first, then decode rows (n == 1)."""
    pre, dec = [s for s in seqs if not s[4]], [s for s in seqs if s[4]]
    pos, slots, cu, ctx_p, st = [], [], [0], [], []
    for start, n, table, slot, _ in pre + dec:
        for p in range(start, start + n):
            pos.append(p)
            slots.append(table[p // bs] * bs + p % bs)
        st.append(slot)
    for start, n, *_ in pre:
        cu.append(cu[-1] + n)
        ctx_p.append(start + n)
    i32 = dict(dtype=torch.int32, device=device)

    def tables(group):
        w = max(len(s[2]) for s in group)
        return torch.tensor([list(s[2]) + [0] * (w - len(s[2])) for s in group], **i32)

    m = AttnMeta(positions=torch.tensor(pos, **i32), slots=torch.tensor(slots, **i32), num_prefill_tokens=cu[-1],
                 num_prefill_seqs=len(pre), num_decode=len(dec))
    if pre:
        m.cu_q, m.ctx_lens_p, m.block_tables_p = torch.tensor(cu, **i32), torch.tensor(ctx_p, **i32), tables(pre)
        m.q_lens_cpu, m.ctx_lens_cpu = [s[1] for s in pre], ctx_p
    if dec:
        m.block_tables_d, m.ctx_lens_d = tables(dec), torch.tensor([s[0] + 1 for s in dec], **i32)
    lens = [s[1] for s in pre] + [1] * len(dec)
    m.seq_cu = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), **i32)
    m.state_slots = torch.tensor(st, **i32)
    m.max_seq_len = max(lens)
    return m


def one_layer(kind, mixer, W, device, dtype, seed=5, change=None):
    """A one-layer model of the mechanism (random weights through the checkpoint names, ``change`` edits them) and its tensors."""
    cfg = KebepelConfig.from_json({"architecture": "Kebepel", "vocab": 11, "width": W, "norm": {"eps": EPS},
                                   "layers": [{"type": kind, "mixer": mixer, "mlp": None}]})
    m = build_decoder(cfg, device=device, dtype=dtype, seed=seed)
    if change is not None:
        sd = {k: v.cpu().float() for k, v in m.native_state_dict().items()}
        change(sd)
        m.load_state_dict_native(sd)
    return m, {k: v.cpu().double() for k, v in m.native_state_dict().items()}


def run_mixer(m, h, cuts, device, dtype, slot=1, nblocks=64, caches=None):
    """The layer's mixer over ``h`` [T, W] fed in portions of the sizes ``cuts`` (the rest as decode rows), pages in descending order."""
    T = h.shape[0]
    blocks = list(range(nblocks - 1, nblocks - 1 - (T + BS - 1) // BS, -1))
    caches = caches or m.make_caches(nblocks, BS, 3)
    out, at, sizes = [], 0, list(cuts)
    while at < T:
        dec = not sizes
        n = 1 if dec else min(sizes.pop(0), T - at)
        meta = step_meta([(at, n, blocks, slot, dec)], device)
        with torch.inference_mode():
            y = m._mixer(m.layers[0], h[at:at + n].to(dtype).to(device).contiguous(), meta, caches[0])
        out.append(y.float().cpu())
        at += n
    return torch.cat(out)


def att(heads, kv, dim, vdim, scale, diff, temp=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    return dict(m, q_temp={"coef": temp[0], "every": temp[1]}) if temp else m


def par(heads, kv, dim, vdim, scale, rot, cap, rh, rkv, rdim, rvdim, conv, ls=0.7, rs=1.3):
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if cap:
        left["softcap"] = cap
    return {"left": left, "right": {"heads": rh, "kv_heads": rkv, "dim": rdim, "vdim": rvdim, "conv": conv}, "left_scale": ls, "right_scale": rs}


YARN = {"dims": 16, "base": 100.0, "scaling": {"factor": 4.0, "original": 40, "fast": 8.0, "slow": 1.0}}
KINDS = {
    "diff": ("attention", att(4, 2, 12, 20, 0.3, 0.35, (0.6, 7)), O.diff_attention),
    "diff-plain": ("attention", att(3, 3, 8, 10, 0.4, 0.8), O.diff_attention),
    "diff-group": ("attention", att(6, 1, 10, 24, 0.5, 0.1, (1.0, 1)), O.diff_attention),
    "parallel": ("parallel", par(4, 2, 24, 16, 0.3, YARN, 4.0, 4, 2, 12, 20, 3), O.parallel),
    "parallel-plain": ("parallel", par(3, 1, 10, 14, 0.4, {"dims": 6, "base": 1000.0}, 0.0, 3, 3, 9, 11, 2, 1.0, 1.0), O.parallel),
    "parallel-wide": ("parallel", par(2, 2, 40, 8, 0.2, {"dims": 40, "base": 50.0}, 30.0, 2, 1, 72, 100, 7, 1.5, 0.4), O.parallel),
}


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("kind", list(KINDS))
def test_mixer_whole_portions_and_token_by_token(kind, device, dtype):
    """A whole prompt in one step, token by token from the first token on, and portions of 1, 2, 2, 3, 16, 17, 5 tokens followed by decode
    rows give the oracle's result at every position."""
    typ, mixer, fn = KINDS[kind]
    W, T = 40, 61
    m, sd = one_layer(typ, mixer, W, device, dtype)
    h = q16(rnd(torch.Generator().manual_seed(3), T, W))
    want = fn(h, sd, "l0.mix.", mixer, EPS)
    for cuts in ([T], [1], [1, 2, 2, 3, 16, 17, 5], [30, 2, 29]):
        got = run_mixer(m, h, cuts, device, dtype)
        err = (got.double() - want).abs().amax(1) / want.abs().max()
        # (bf16: the first tokens of a delta rule are a near-zero dot product times a value that its unit norm blows up)
        assert float(err[4:].max()) < 2 * tol(dtype) and float(err.max()) < (tol(dtype) if dtype == torch.float32 else 0.5), (cuts, err)


# ---------------------------------------------------------------------------- attention: far keys, maps, temperature, caps
def set_identity_heads(sd, p, heads, kv, dim, maps, W):
    """q and k of every head read the first ``dim * maps`` inputs; v of every kv head reads inputs behind them; no biases."""
    for n, h in (("q", heads), ("k", kv)):
        sd[p + n].zero_()
        sd[p + n + ".b"].zero_()
        for i in range(h * maps * dim):
            sd[p + n][i, i % (maps * dim)] = 1.0
    sd[p + "v.b"].zero_()


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("far_map", [0, 1])
def test_differential_attention_finds_a_far_key_in_either_map(far_map, device, dtype):
    """300 positions; ONE key of one map lines up with the last query, the other map is flat: the average of that map is the far
    key's value, in a prompt step, in a portion and in decoding, far back, at page borders and in the last places."""
    W, T, dim = 24, 300, 4
    mixer = att(4, 2, dim, 8, 1.0, 0.4)
    m, sd = one_layer("attention", mixer, W, device, dtype, change=lambda s: set_identity_heads(s, "l0.mix.", 4, 2, dim, 2, W))
    g = torch.Generator().manual_seed(1)
    for far in (0, 15, 16, 31, 130, 287, 288, 298, 299):
        h = q16(rnd(g, T, W, scale=0.05))
        h[:, 8:] = q16(rnd(g, T, W - 8))
        spike = torch.tensor([3.0, -3.0, 3.0, 3.0])
        h[far, 4 * far_map:4 * far_map + 4] = spike
        h[-1, 4 * far_map:4 * far_map + 4] = spike
        want = O.diff_attention(h, sd, "l0.mix.", mixer, EPS)
        for cuts in ([T], [T - 1], [200, 98, 2]):
            got = run_mixer(m, h, cuts, device, dtype)
            assert rel_err(got[-1], want[-1]) < tol(dtype), (far, cuts, rel_err(got[-1], want[-1]))
        # the far key matters: without it the result is another one
        h2 = h.clone()
        h2[far, 8:] = -h2[far, 8:]
        if far != T - 1:
            other = O.diff_attention(h2, sd, "l0.mix.", mixer, EPS)
            assert rel_err(other[-1], want[-1]) > 4 * tol(dtype)


@pytest.mark.parametrize("device,dtype", ALL)
def test_normed_attention_finds_a_far_key(device, dtype):
    """The same for one map with rotation and score cap, without the recurrence beside it (right_scale 0)."""
    W, T, dim = 24, 260, 8
    mixer = par(4, 2, dim, 8, 1.0, {"dims": 4, "base": 1e6, "scaling": {"factor": 2.0, "original": 64, "fast": 4.0, "slow": 1.0}}, 20.0, 2, 2, 4, 4, 2, rs=0.0)

    def change(s):
        set_identity_heads(s, "l0.mix.left.", 4, 2, dim, 1, W)
        s["l0.mix.left.q.norm"].fill_(1.5)
        s["l0.mix.left.k.norm"].fill_(1.5)

    m, sd = one_layer("parallel", mixer, W, device, dtype, change=change)
    g = torch.Generator().manual_seed(2)
    for far in (0, 16, 47, 129, 255, 258):
        h = q16(rnd(g, T, W))
        h[:, 4:8] *= 0.1
        h[far, :8] = torch.tensor([0.0, 0.0, 0.0, 0.0, 2.0, -2.0, 2.0, 2.0])
        h[-1, :8] = h[far, :8]
        want = O.parallel(h, sd, "l0.mix.", mixer, EPS)
        for cuts in ([T], [T - 1], [100, 158, 2]):
            got = run_mixer(m, h, cuts, device, dtype)
            assert rel_err(got[-1], want[-1]) < tol(dtype), (far, cuts)


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("every", [1, 5, 16])
def test_query_temperature_steps_at_its_places(every, device, dtype):
    """Two keys whose scores differ: the temperature of a position is read off the weights.  Every position around every step, in
    prompts and in decoding; a step one position late shows."""
    W, T, dim = 24, 50, 4
    mixer = att(2, 1, dim, 8, 1.0, 0.3, (1.3, every))
    m, sd = one_layer("attention", mixer, W, device, dtype, change=lambda s: set_identity_heads(s, "l0.mix.", 2, 1, dim, 2, W))
    h = torch.zeros(T, W, dtype=torch.float64)
    h[:, 8:] = q16(rnd(torch.Generator().manual_seed(9), T, W - 8))
    h[:, 0], h[:, 4] = 1.0, 0.5
    h[0, 0], h[1, 4] = 2.0, 2.0
    want = O.diff_attention(h, sd, "l0.mix.", mixer, EPS)
    late = dict(mixer, q_temp={"coef": 1.3, "every": every + 1})
    assert rel_err(O.diff_attention(h, sd, "l0.mix.", late, EPS), want) > 2 * tol(dtype)
    for cuts in ([T], [1], [7, 2, 20]):
        assert rel_err(run_mixer(m, h, cuts, device, dtype), want) < tol(dtype), cuts


SHAPES = [  # H, G, dim, vdim, page
    (4, 2, 32, 64, 16), (3, 1, 24, 40, 16), (8, 2, 64, 128, 32), (2, 2, 8, 8, 48), (5, 5, 128, 256, 16), (4, 1, 200, 136, 16), (20, 1, 16, 16, 32)]


def attention_case(shape, dtype, seed=0, climb=0.0):
    """Queries, a paged cache and gates of four sequences: a whole prompt, two portions behind cached keys, one of a page's size.  ``climb``:
    scores that rise (or fall) by that many nats over the keys."""
    H, G, dim, vdim, page = shape
    g = torch.Generator().manual_seed(seed)
    lens, ctxs, nb = [37, 2, 90, 16], [37, 70, 170, 16], -(-170 // page)
    T = sum(lens)
    q, k, v = (q16(rnd(g, *s)) for s in ((T, H, 2, dim), (4, 176, G, 2, dim), (4, 176, G, vdim)))
    gate = q16(rnd(g, T, H * vdim))
    if climb:
        q[..., 0], k[..., 0] = 1.0, q16(torch.linspace(0, climb * dim ** 0.5, 176, dtype=torch.float64)).view(1, -1, 1, 1)
    table = torch.randperm(4 * nb + 3, generator=g)[:4 * nb].view(4, nb)
    kc = torch.full((4 * nb + 3, G, page, 2 * dim), 7.0)
    vc = torch.full((4 * nb + 3, G, vdim, page), -9.0)
    for b in range(4):
        for j in range(ctxs[b]):
            kc[table[b, j // page], :, j % page] = k[b, j].reshape(G, 2 * dim).float()
            vc[table[b, j // page], :, :, j % page] = v[b, j].float()
    cu = torch.tensor([0] + lens).cumsum(0)
    return lens, ctxs, q, k, v, gate, table.int(), kc.to(dtype), vc.to(dtype), cu.int()


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("shape", SHAPES)
@pytest.mark.parametrize("climb", [0.0, 160.0, -160.0])
def test_attention_kernels_of_all_instances(shape, climb, device, dtype):
    """The attention ops alone (prompt rows, decode rows with 1 and 3 key splits) for every kernel instance, unequal head sizes, group
    sizes from 1 to 20, several page sizes, scores that climb or fall by 160 nats over the keys: two maps with temperature, one map
    with and without a cap.  Keys behind a sequence's end and other sequences' pages hold values that would show."""
    H, G, dim, vdim, page = shape
    lens, ctxs, q, k, v, gate, table, kc, vc, cu = attention_case(shape, dtype, 3, climb)
    T, scale, rep = sum(lens), dim ** -0.5, H // G
    lam, temp = 0.45, {"coef": 0.3, "every": 19}
    sig = torch.sigmoid(gate).view(T, H, vdim)
    want2 = torch.zeros(T, H, vdim, dtype=torch.float64)
    want1 = {cap: torch.zeros(T, H, vdim, dtype=torch.float64) for cap in (0.0, 3.0)}
    last = []
    for b, (n, ctx) in enumerate(zip(lens, ctxs)):
        last.append(int(cu[b + 1]) - 1)
        t = O.temperature(ctx, temp)
        for h in range(H):
            full = torch.zeros(ctx, 2, dim, dtype=torch.float64)
            full[ctx - n:] = q[cu[b]:cu[b + 1], h]
            a = [O.causal_softmax(full[:, i] * t.view(-1, 1), k[b, :ctx, h // rep, i], v[b, :ctx, h // rep], scale)[ctx - n:] for i in (0, 1)]
            want2[cu[b]:cu[b + 1], h] = O.rms_unit(a[0] - lam * a[1], EPS) * 0.7
            for cap, w in want1.items():
                w[cu[b]:cu[b + 1], h] = O.causal_softmax(full[:, 0], k[b, :ctx, h // rep, 0], v[b, :ctx, h // rep], scale, cap)[ctx - n:] * 0.6
    d = lambda x: x.to(device)      # noqa: E731
    qd, gd = d(q.reshape(T, -1).to(dtype)), d(gate.to(dtype))
    kd, vd, td, cud, ctx = d(kc), d(vc), d(table), d(cu), d(torch.tensor(ctxs, dtype=torch.int32))
    rows = d(torch.tensor(last))
    bound = (1e-3 if climb else 3e-5) if dtype == torch.float32 else 3e-2      # (an f32 score of 160 is off by 1e-5 and more itself)
    opt = dict(scale=scale, temp_coef=0.3, temp_every=19, lam=d(torch.tensor([lam])), eps=EPS, norm_vdim=vdim, out_scale=0.7)
    out = torch.zeros(T, H * vdim, dtype=dtype, device=device)
    ops.diff_attention_prefill(qd, kd, vd, td, cud, ctx, H, G, dim, vdim, gd, 0, out, **opt)
    assert rel_err(out, (want2 * sig).reshape(T, -1)) < bound
    for Z in (1, 3):
        od = torch.zeros(4, H * vdim, dtype=dtype, device=device)
        ops.diff_attention_decode(qd[rows], kd, vd, td, ctx, H, G, dim, vdim, gd[rows], 0, od, splits=Z, **opt)
        assert rel_err(od, (want2 * sig).reshape(T, -1)[last]) < bound, Z
    q1, k1 = d(q[:, :, 0].reshape(T, -1).to(dtype)), kd[..., :dim].contiguous()
    hs = torch.full((H,), scale, device=device)
    for cap, w in want1.items():
        w = (w * sig).reshape(T, -1)
        forms = ["sink"] + (["tile"] if device == "cuda" and ops.tile_attention_supported(H, G, dim, vdim, dtype) else [])
        for form in forms:
            out.zero_()
            if form == "tile":
                ts, tq = ops.row_tiles(lens, ctxs, ops.tile_attention_rows(H, G))
                ops.tile_attention_prefill(q1, k1, vd, td, cud, ctx, H, G, dim, vdim, gd, 0, out, (d(torch.from_numpy(ts)), d(torch.from_numpy(tq))),
                                           scale=scale, softcap=cap, out_scale=0.6)
            else:
                ops.sink_attention_prefill(q1, k1, vd, td, cud, ctx, H, G, dim, vdim, hs, ops.MASK_CAUSAL, 0, False, gd, 0, out, softcap=cap,
                                           gate_elem=True, out_scale=0.6)
            assert rel_err(out, w) < bound, (cap, form, rel_err(out, w))
        od = torch.zeros(4, H * vdim, dtype=dtype, device=device)
        ops.sink_attention_decode(q1[rows], k1, vd, td, ctx, H, G, dim, vdim, hs, ops.MASK_CAUSAL, 0, False, gd[rows], 0, od, splits=2, softcap=cap,
                                  gate_elem=True, out_scale=0.6)
        assert rel_err(od, w[last]) < bound, cap


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("H,G,dim,vdim,rot,page", [(4, 2, 48, 32, 48, 16), (3, 1, 24, 40, 16, 48), (16, 4, 128, 128, 64, 16), (6, 6, 16, 8, 0, 32)])
def test_queries_keys_values_filed(H, G, dim, vdim, rot, page, device, dtype):
    """Bias, norm over the whole projection (one loud head sets the root of all), pair rotation at positions up to 3,000 and the paged
    write at scattered slots, with and without norm; a padding row's slot files nothing.  Few rows, and many (whose values take
    their own way): runs of slots that start on and off 16-byte borders, cut by pages, and single scattered ones."""
    g = torch.Generator().manual_seed(H)
    for T in (21, 300):
        filed(H, G, dim, vdim, rot, page, device, dtype, g, T)


def filed(H, G, dim, vdim, rot, page, device, dtype, g, T):
    n, NB = (H + G) * dim + G * vdim, 500 // page
    u = q16(rnd(g, T, n))
    u[:, :dim] *= 8                                          # a norm per head would not see it in the others
    bias, qw, kw = (rnd(g, s).float().double() for s in (n, H * dim, G * dim))
    freq = (torch.rand(max(rot // 2, 1), generator=g, dtype=torch.float64) * 0.5).float().double()
    pos = torch.randint(0, 3000, (T,), generator=g, dtype=torch.int32)
    slots = torch.randperm(NB * page, generator=g)[:T].int()
    if T > 100:     # tokens in order in pages out of order, from an odd offset on, some scattered
        order = torch.randperm(NB, generator=g)
        lin = (order.view(-1, 1) * page + torch.arange(page)).reshape(-1).int()
        slots[:200], slots[200:] = lin[:200], lin[205:205 + T - 200]
        slots[17:23] = lin[400:406].flip(0)
    slots[4] = -1
    for norm in (True, False):
        x = u + bias
        q, k, v = x[:, :H * dim], x[:, H * dim:(H + G) * dim], x[:, (H + G) * dim:].view(T, G, vdim)
        if norm:
            q, k = q / torch.sqrt((q * q).sum(1, keepdim=True) / (H * dim - 3) + EPS) * qw, k / torch.sqrt((k * k).sum(1, keepdim=True) / (G * dim - 1) + EPS) * kw
        q, k = q.reshape(T, H, dim).clone(), k.reshape(T, G, dim).clone()
        ang = (pos.double().view(T, 1, 1).float() * freq.float()).double()[..., :rot // 2]
        for t in (q, k):
            if rot:
                a, b = t[..., 0:rot:2].clone(), t[..., 1:rot:2].clone()
                t[..., 0:rot:2], t[..., 1:rot:2] = 1.2 * (a * ang.cos() - b * ang.sin()), 1.2 * (b * ang.cos() + a * ang.sin())
        ud = torch.zeros(T, n + 8, dtype=dtype, device=device)
        ud[:, 8:] = u.to(dtype).to(device)
        kc, vc = torch.zeros(NB, G, page, dim, dtype=dtype, device=device), torch.zeros(NB, G, vdim, page, dtype=dtype, device=device)
        f = lambda t: t.float().to(device)      # noqa: E731
        ops.qkv_file(ud, 8, H, G, dim, vdim, f(bias), f(qw) if norm else None, f(kw) if norm else None, H * dim - 3, G * dim - 1, EPS, rot, f(freq), 1.2,
                     pos.to(device), kc, vc, slots.to(device))
        bound = 2e-5 if dtype == torch.float32 else 8e-3
        assert rel_err(ud[:, 8:8 + H * dim], q.reshape(T, -1)) < bound
        wk, wv = torch.zeros(NB, G, page, dim, dtype=torch.float64), torch.zeros(NB, G, vdim, page, dtype=torch.float64)
        for t in range(T):
            if int(slots[t]) >= 0:
                wk[slots[t] // page, :, slots[t] % page], wv[slots[t] // page, :, :, slots[t] % page] = k[t], v[t]
        assert rel_err(kc, wk) < bound and rel_err(vc, wv) < bound
        assert torch.equal(kc.cpu() == 0, (wk == 0)) and torch.equal(vc.cpu() == 0, (wv == 0))


# ---------------------------------------------------------------------------- delta rule
def run_delta(x, device, dtype, H, Hk, dk, dv, state, lens, starts, slots):
    T = sum(lens)
    i32 = dict(dtype=torch.int32, device=device)
    cu = torch.tensor([0] + list(torch.tensor(lens).cumsum(0)), **i32)
    pos = torch.cat([torch.arange(n) + s for n, s in zip(lens, starts)]).to(**i32)
    d = lambda t: t.to(dtype).to(device)      # noqa: E731
    out = torch.zeros(T, H * dv + 8, dtype=dtype, device=device)
    ops.head_delta(d(x["q"]), d(x["k"]), d(x["v"]), d(x["b"]), d(x["a"]), x["dt"].float().to(device), x["A"].float().to(device), d(x["gate"]),
                   x["w"].float().to(device).repeat(H), EPS, state, cu, torch.tensor(slots, **i32), pos, H, Hk, dk, dv, out, max(lens))
    assert not out[:, H * dv:].any()
    return out[:, :H * dv].float().cpu()


def delta_want(x, H, Hk, dk, dv, r0, n, S):
    rep = H // Hk
    q = (O.l2_unit(x["q"][r0:r0 + n].view(n, Hk, dk)) * dk ** -0.5).repeat_interleave(rep, 1)
    k = O.l2_unit(x["k"][r0:r0 + n].view(n, Hk, dk)).repeat_interleave(rep, 1)
    g = torch.exp(-torch.exp(x["A"]) * O.softplus(x["a"][r0:r0 + n] + x["dt"]))
    o, S = O.delta_rule(q, k, x["v"][r0:r0 + n].view(n, H, dv), g, torch.sigmoid(x["b"][r0:r0 + n]), S)
    return (O.rms_unit(o, EPS) * x["w"]).reshape(n, -1) * O.silu(x["gate"][r0:r0 + n]), S


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("H,Hk,dk,dv", [(6, 3, 24, 40), (4, 2, 128, 128), (2, 2, 130, 200), (2, 1, 7, 5), (1, 1, 250, 300), (3, 3, 64, 50), (5, 1, 16, 64)])
def test_delta_rule_forms_agree_with_the_recurrence(H, Hk, dk, dv, device, dtype):
    """The op alone: steps of single tokens and steps with portions of 1 to 40 tokens (chunks cut by sequence ends), sequences that
    continue an earlier state and ones that start fresh in a slot that holds leftovers, a padding row; outputs and states against
    the recurrence written out in float64; a slot that no sequence holds is not touched."""
    g = torch.Generator().manual_seed(dk)
    for lens in ([40, 1, 17, 3, 16], [1, 1, 1, 1, 1], [33]):
        T, n = sum(lens), len(lens)
        x = {"q": q16(rnd(g, T, Hk * dk)), "k": q16(rnd(g, T, Hk * dk)), "v": q16(rnd(g, T, H * dv)), "b": q16(rnd(g, T, H, scale=2.0)),
             "a": q16(rnd(g, T, H, scale=3.0)), "gate": q16(rnd(g, T, H * dv)), "dt": rnd(g, H).float().double() - 2, "A": rnd(g, H).float().double(),
             "w": (rnd(g, dv, scale=0.2) + 1).float().double()}
        S0 = rnd(g, 7, H, dk, dv, scale=0.3).float()
        slots, starts = [4, 0, -1, 6, 2][:n], [0, 5, 3, 9, 0][:n]
        state = S0.to(device).clone()
        got = run_delta(x, device, dtype, H, Hk, dk, dv, state, lens, starts, slots)
        r0 = 0
        for i, m in enumerate(lens):
            if slots[i] < 0:
                assert not got[r0:r0 + m].any()
            else:
                want, S = delta_want(x, H, Hk, dk, dv, r0, m, S0[slots[i]].double() if starts[i] else None)
                err = (got[r0:r0 + m].double() - want).abs().amax(1) / want.abs().max()
                assert float(err.max()) < (1e-4 if dtype == torch.float32 else 2e-2), (lens, i, err)
                assert rel_err(state[slots[i]], S) < 2e-5
            r0 += m
        for s in {0, 1, 2, 3, 4, 5, 6} - set(slots):
            assert torch.equal(state[s].cpu(), S0[s])


@pytest.mark.parametrize("device,dtype", ALL)
def test_delta_rule_keeps_a_value_and_forgets_at_a_large_decay(device, dtype):
    """A decay of 1 (A far below) keeps the first token's write for 400 tokens whose keys are orthogonal to it; a single token with a huge
    decay in the middle of a chunk wipes the state without costing the tokens behind it their accuracy."""
    H = Hk = 2
    dk, dv, T = 16, 8, 400
    g = torch.Generator().manual_seed(8)
    k = rnd(g, T, H, dk)
    k[..., 0] = 0.0
    k[0, :, :] = 0.0
    k[0, :, 0] = 1.0
    q = rnd(g, T, H, dk, scale=0.1)
    q[-1] = k[0]
    x = {"q": q16(q.reshape(T, -1)), "k": q16(k.reshape(T, -1)), "v": q16(rnd(g, T, H * dv)), "b": torch.full((T, H), 3.0, dtype=torch.float64),
         "a": torch.zeros(T, H, dtype=torch.float64), "gate": q16(rnd(g, T, H * dv)), "dt": torch.zeros(H, dtype=torch.float64),
         "A": torch.tensor([-30.0, -9.0], dtype=torch.float64), "w": torch.ones(dv, dtype=torch.float64)}
    for wipe in (None, 389):
        if wipe is not None:
            x["a"][wipe], x["A"] = 400.0, torch.tensor([2.0, 1.0], dtype=torch.float64)
            x["a"][:wipe] = x["a"][wipe + 1:] = -12.0
        want, S = delta_want(x, H, Hk, dk, dv, 0, T, None)
        for cuts in ([T], [390, 2, 8], [385] + [1] * 15):
            state = torch.full((2, H, dk, dv), 1e3, device=device)
            got, at = [], 0
            for n in cuts:
                part = {n_: (t[at:at + n] if t.dim() == 2 else t) for n_, t in x.items()}
                got.append(run_delta(part, device, dtype, H, Hk, dk, dv, state, [n], [at], [1]))
                at += n
            got = torch.cat(got)
            assert rel_err(got[-10:], want[-10:]) < (1e-4 if dtype == torch.float32 else 2e-2), (wipe, cuts)
            assert rel_err(state[1], S) < 3e-5


@pytest.mark.parametrize("device,dtype", ALL)
def test_state_slots_start_from_zero_and_are_independent(device, dtype):
    """Two sequences in one step with different slots, then a new sequence in a slot that holds an old state (and a poisoned
    convolution state): each equals its run alone."""
    typ, mixer, fn = KINDS["parallel"]
    W = 40
    m, sd = one_layer(typ, mixer, W, device, dtype)
    g = torch.Generator().manual_seed(7)
    ha, hb, hc = q16(rnd(g, 22, W)), q16(rnd(g, 9, W)), q16(rnd(g, 15, W))
    caches = m.make_caches(12, BS, 3)
    caches[0][2].fill_(float("nan") if dtype != torch.float32 else 1e30)      # whatever an earlier owner left
    caches[0][3].fill_(1e30)
    ta, tb = [3, 7], [5]
    run = lambda h, seqs: m._mixer(m.layers[0], h.to(dtype).to(device), step_meta(seqs, device), caches[0]).float().cpu()      # noqa: E731
    with torch.inference_mode():
        y1 = run(torch.cat([ha[:20], hb[:8]]), [(0, 20, ta, 2, False), (0, 8, tb, 0, False)])
        y2 = run(torch.cat([ha[20:], hb[8:]]), [(20, 2, ta, 2, False), (8, 1, tb, 0, True)])
        y3 = run(hc, [(0, 15, tb, 0, False)])          # c takes b's slot and pages
    for got, hh in ((torch.cat([y1[:20], y2[:2]]), ha), (torch.cat([y1[20:], y2[2:]]), hb), (y3, hc)):
        want = fn(hh, sd, "l0.mix.", mixer, EPS)
        err = (got.double() - want).abs().amax(1) / want.abs().max()
        assert float(err.max()) < (tol(dtype) if dtype == torch.float32 else 0.5) and float(err.median()) < tol(dtype), err


# ---------------------------------------------------------------------------- stream
@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("W", [36, 250, 1024, 2050, 4100])
def test_sandwiched_layer_norms(W, device, dtype):
    """Norm of the result, sum, step vector and next norm in one pass, each part present or absent; rows chosen by an index leave the
    stream alone; a large common offset of a row (mean far above the deviation) does not cost accuracy."""
    g = torch.Generator().manual_seed(W)
    for T in (5, 1030) if W <= 1024 else (5,):
        sandwich(W, T, device, dtype, g)


def sandwich(W, T, device, dtype, g):
    x, y = rnd(g, T, W).float(), q16(rnd(g, T, W) + 20)
    wp, bp, add, w, b = (rnd(g, W).float() for _ in range(5))
    D = lambda t: None if t is None else t.to(device)      # noqa: E731
    sd = {"p": wp.double(), "p.b": bp.double(), "n": w.double(), "n.b": b.double()}
    for with_y, with_add in ((True, False), (False, True), (True, True), (False, False)):
        v = x.double()
        if with_y:
            v = v + O.layer_norm(y, sd, "p", EPS)
        if with_add:
            v = v + add.double()
        want = O.layer_norm(v, sd, "n", EPS)
        xd = x.to(device).clone()
        got = ops.stream_sandwich_layernorm(xd, y.to(dtype).to(device) if with_y else None, D(wp), D(bp), D(add) if with_add else None, D(w), D(b), EPS, dtype)
        bound = 2e-5 if dtype == torch.float32 else 6e-3
        assert got.dtype == dtype and rel_err(got, want) < bound and rel_err(xd, v) < 2e-5
        idx = torch.tensor([4, 0, 2], device=device)
        xd = x.to(device).clone()
        got = ops.stream_sandwich_layernorm(xd, y.to(dtype).to(device) if with_y else None, D(wp), D(bp), D(add) if with_add else None, D(w), D(b), EPS, dtype,
                                            idx=idx)
        assert rel_err(got, want[[4, 0, 2]]) < bound and torch.equal(xd.cpu(), x)


def test_rotary_ramp_matches_the_equations():
    from llm_kubernetes_minikube_sharp4dev_amd.models.window_attention import RotarySpec

    for rot in (YARN, {"dims": 64, "base": 500000.0, "scaling": {"factor": 16.0, "original": 2048, "fast": 32.0, "slow": 1.0}}, {"dims": 6, "base": 30.0},
                {"dims": 8, "base": 10000.0, "scaling": {"factor": 1.0, "original": 100, "fast": 2.0, "slow": 2.0}}):
        s = RotarySpec.from_dict(rot, "ramp")
        f, mag = O.rotary_table(rot)
        assert torch.allclose(s.freq_tensor("cpu").double(), torch.tensor(f, dtype=torch.float64), rtol=1e-6)
        assert math.isclose(s.magnitude, mag, rel_tol=1e-12)
