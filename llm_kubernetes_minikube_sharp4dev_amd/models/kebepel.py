"""Kebepel: a decoder whose sublayers are layer-normed in front and behind, over differential attention layers and layers of
row-normed attention beside a gated delta rule, with a span of layers that runs several times.

    x = embed[token]                                                                     (f32 stream)
    per layer run:  x += step[t]                                                         only where pass t of the looped span starts
                    x += ln1b(mixer(ln1(x)));  x += ln2b(ff(ln2(x)))                     (ff may be absent)
    logits = head . ln_f(x)                   ln(v) = (v - mean) / sqrt(var + eps) * w + b

Mixers (``cfg.layers``, any order): ``attention`` -- ``models.gated_attention.diff_attention``; ``parallel`` -- ``left_scale *``
``models.gated_attention.row_norm_attention`` ``+ right_scale *`` ``models.linear_state.head_delta_mixer``, both reading the same
input.  Feed-forward: ``W_down (silu(W_gate h) * W_up h)``.

MI355X layout decisions:
  * the stream is f32 and a sublayer boundary is one pass over it (``ops.stream_sandwich_layernorm``): norm of the sublayer's result,
    sum, a looped pass's step vector, the next sublayer's norm and the activation-dtype copy for the projections; the final norm runs
    only on the rows that feed the LM head;
  * a layer has one input projection: both mixers of a parallel layer read one product ``[q k v g | q k v b a g]``, and one output
    projection: their results lie side by side, already scaled (the left one in the attention kernels, the right one in its norm
    weight), and ``[W_o left | W_o right]`` sums them in the product's f32 accumulators;
  * projection biases, the norms over whole projections, rotation and the paged write are one kernel; the query temperature multiplies
    the f32 scores; maps, lambda, head norm and gates live inside the attention kernels;
  * every layer run has its own caches: paged K / V, convolution state and f32 recurrent state over the engine's state slots.

Checkpoint format: ``config.json`` (``KebepelConfig.from_json``) and ``model.safetensors`` with ``embed``, ``head``, ``loop.step``,
``final.norm`` (+ ``.b``), ``l<i>.norm1 | norm1b | norm2 | norm2b`` (+ ``.b``), ``l<i>.mix.*`` (``left.`` / ``right.`` in a parallel layer),
``l<i>.mlp.gate | up | down``; linear weights [out, in].
"""
from __future__ import annotations

import math

import torch
import torch.nn as nn

from .. import ops
from ..parallel.tp import SINGLE, TPGroup
from .attention import AttnMeta
from .configs import KebepelConfig, pad_vocab
from .gated_attention import DiffAttnSpec, RowNormAttnSpec, diff_attention, diff_lambda, row_norm_attention
from .linear_state import FusedRows, HeadDeltaSpec, fused_mult, head_delta_mixer


def _p(*shape, **kw):
    return nn.Parameter(torch.zeros(*shape, **kw), requires_grad=False)


def _pad8(n: int) -> int:
    return -(-int(n) // 8) * 8


class _DiffAttention(nn.Module):
    """Weights of an ``attention`` mixer under checkpoint prefix ``mix.``."""

    def __init__(self, m: dict, W: int, e: dict, f: dict):
        super().__init__()
        t = self.true = DiffAttnSpec.from_dict(m)               # the checkpoint's sizes
        s = self.spec = t.padded()                              # head sizes of the kernels (zero rows / columns)
        self.rows = FusedRows(s.segments(), fused_mult(W))
        self.w_in = _p(self.rows.total, W, **e)
        self.bias = _p(self.rows.off["g"], **f)                 # over q | k | v
        self.lq1, self.lk1, self.lq2, self.lk2 = (_p(t.dim, **f) for _ in range(4))
        self.lam = _p(1, **f)
        self.o = _p(W, s.heads * s.vdim, **e)

    def init_constants(self):
        self.lam.fill_(diff_lambda(self.lq1, self.lk1, self.lq2, self.lk2, self.spec.diff))


class _Parallel(nn.Module):
    """Weights of a ``parallel`` mixer: row-normed attention under ``mix.left.``, the gated delta rule under ``mix.right.``."""

    def __init__(self, m: dict, W: int, e: dict, f: dict):
        super().__init__()
        t = self.true = RowNormAttnSpec.from_dict(m["left"])
        s = self.spec = t.padded()
        r = self.delta = HeadDeltaSpec.from_dict(m["right"])
        self.left_scale, self.right_scale = float(m.get("left_scale", 1.0)), float(m.get("right_scale", 1.0))
        self.rows = FusedRows(s.segments() + r.segments(), fused_mult(W))
        self.conv_rows = r.conv_rows()
        self.w_in = _p(self.rows.total, W, **e)
        self.bias = _p(self.rows.off["g"], **f)
        self.q_norm, self.k_norm = _p(s.heads * s.dim, **f), _p(s.kv_heads * s.dim, **f)
        self.freq = _p(max(s.rot.dims // 2, 1), **f)
        self.hscale = _p(s.heads, **f)
        self.conv_w = _p(self.conv_rows.total, r.conv, **f)     # zero rows at the alignment padding
        self.A_log, self.dt_bias = _p(r.heads, **f), _p(r.heads, **f)
        self.norm = _p(r.vdim, **f)
        self.norm_w = _p(r.heads * r.vdim, **f)                 # right_scale * norm for every head, what the kernels read
        self.out_rows = FusedRows([("left", s.heads * s.vdim), ("right", r.heads * r.vdim)], fused_mult(W))
        self.o = _p(W, self.out_rows.total, **e)

    def init_constants(self):
        self.freq.copy_(self.spec.rot.freq_tensor(self.freq.device))
        self.hscale.fill_(self.spec.scale)
        self.norm_w.copy_((self.norm * self.right_scale).repeat(self.delta.heads))


class KebepelLayer(nn.Module):
    def __init__(self, cfg: KebepelConfig, spec, dtype, device):
        super().__init__()
        W = cfg.hidden
        e = dict(dtype=dtype, device=device)
        f = dict(dtype=torch.float32, device=device)   # norms, biases and per-head constants stay f32
        self.type = spec.type
        self.ff = int(spec.mlp["ff"]) if spec.mlp else 0
        self.norms = ("norm1", "norm1b") + (("norm2", "norm2b") if self.ff else ())
        for n in self.norms:
            setattr(self, n, _p(W, **f))
            setattr(self, n + "_b", _p(W, **f))
        self.mix = {"attention": _DiffAttention, "parallel": _Parallel}[spec.type](spec.mixer, W, e, f)
        self.ffp = _pad8(self.ff)                      # zero gate / up rows and down columns behind ff (16-byte rows)
        if self.ff:
            self.gate_up, self.down = _p(2 * self.ffp, W, **e), _p(W, self.ffp, **e)

    def ln(self, n: str):
        return getattr(self, n), getattr(self, n + "_b")


class KebepelModel(nn.Module):
    stateful = True            # recurrent state per sequence: no prefix reuse, chunks run as prompt portions

    def __init__(self, cfg: KebepelConfig, tp: TPGroup = SINGLE, dtype=torch.bfloat16, device="cpu"):
        super().__init__()
        if tp.enabled:
            raise NotImplementedError("the Kebepel decoder runs on one GPU (no tensor-parallel sharding)")
        self.cfg, self.tp, self.dtype, self.device = cfg, tp, dtype, torch.device(device)
        e = dict(dtype=dtype, device=device)
        f = dict(dtype=torch.float32, device=device)
        self.vocab_lo, self.vocab_local = 0, cfg.vocab_size
        self.embed = _p(cfg.vocab_size, cfg.hidden, **e)
        self.lm_head = _p(pad_vocab(cfg.vocab_size, 64), cfg.hidden, **e)     # zero rows: logits rows start 32-byte aligned
        self.layers = nn.ModuleList([KebepelLayer(cfg, l, dtype, device) for l in cfg.layers])
        self.steps = _p(max(cfg.loop_times, 1), cfg.hidden, **f)
        self.final_norm, self.final_norm_b = _p(cfg.hidden, **f), _p(cfg.hidden, **f)
        self.runs = cfg.layer_runs()
        att = [L.mix.spec for L in self.layers]
        self.hq = max((s.heads for s in att), default=1)
        self.hkv = max((s.kv_heads for s in att), default=1)
        self.D = max((max(s.dim, s.vdim) for s in att), default=16)

    # ------------------------------------------------------------------ weights
    def _finish(self):
        for L in self.layers:
            L.mix.init_constants()
        return self

    @torch.no_grad()
    def random_init(self, seed: int = 0):
        """Random weights of a scale that keeps every mechanism active, written through the checkpoint names
        so that padding stays zero."""
        return self.load_state_dict_native(random_state_dict(self.cfg, seed))

    def _head_blocks(self, M, prefix: str):
        """(checkpoint name, first fused row, heads, true rows per head, padded rows per head) of an attention mixer's projections
        (a differential head is two maps)."""
        t, s = M.true, M.spec
        maps = 2 if isinstance(s, DiffAttnSpec) else 1
        return [(prefix + n, M.rows.off[n], h, d, dp) for n, h, d, dp in (
            ("q", s.heads * maps, t.dim, s.dim), ("k", s.kv_heads * maps, t.dim, s.dim), ("v", s.kv_heads, t.vdim, s.vdim),
            ("g", s.heads, t.vdim, s.vdim))]

    @torch.no_grad()
    def load_state_dict_native(self, sd: dict):
        """Tensors named as in the checkpoint format (module docstring)."""
        cfg, W = self.cfg, self.cfg.hidden

        def get(name, *shape):
            t = sd[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name}: checkpoint shape {tuple(t.shape)} != {tuple(shape)}")
            return t

        def put(p, name):
            p.copy_(get(name, *p.shape).to(p.dtype))

        def heads_in(dst, name, h, d, dp, *tail):
            """h heads of d checkpoint rows -> h heads of dp >= d rows (zero rows behind d)."""
            dst.view(h, dp, *tail)[:, :d].copy_(get(name, h * d, *tail).view(h, d, *tail).to(dst.dtype))

        put(self.embed, "embed")
        self.lm_head.zero_()
        self.lm_head[:cfg.vocab_size].copy_(get("head", cfg.vocab_size, W).to(self.lm_head.dtype))
        put(self.final_norm, "final.norm")
        put(self.final_norm_b, "final.norm.b")
        if cfg.loop_times:
            put(self.steps, "loop.step")
        for i, L in enumerate(self.layers):
            b, m, M = f"l{i}.", f"l{i}.mix.", L.mix
            for n in L.norms:
                put(getattr(L, n), b + n)
                put(getattr(L, n + "_b"), b + n + ".b")
            par = L.type == "parallel"
            pre, s, t = m + ("left." if par else ""), M.spec, M.true
            for p in (M.w_in, M.bias, M.o):
                p.zero_()
            for name, o, h, d, dp in self._head_blocks(M, pre):
                heads_in(M.w_in[o:o + h * dp], name, h, d, dp, W)
                if o < M.bias.numel():
                    heads_in(M.bias[o:o + h * dp], name + ".b", h, d, dp)
            M.o[:, :s.heads * s.vdim].view(W, s.heads, s.vdim)[:, :, :t.vdim].copy_(
                get(pre + "o", W, s.heads * t.vdim).view(W, s.heads, t.vdim).to(M.o.dtype))
            if not par:
                for n in ("lq1", "lk1", "lq2", "lk2"):
                    put(getattr(M, n), m + n)
            else:
                for p, n, h in ((M.q_norm, "q.norm", s.heads), (M.k_norm, "k.norm", s.kv_heads)):
                    p.zero_()
                    heads_in(p, pre + n, h, t.dim, s.dim)
                r, pre = M.delta, m + "right."
                for seg, n in r.segments():
                    M.w_in[M.rows.off[seg]:M.rows.off[seg] + n].copy_(get(pre + seg[1:], n, W).to(M.w_in.dtype))
                M.conv_w.zero_()
                for seg, n in r.segments()[:3]:
                    o = M.conv_rows.off[seg]
                    M.conv_w[o:o + n].copy_(get(f"{pre}{seg[1:]}.conv", n, r.conv).to(M.conv_w.dtype))
                put(M.A_log, pre + "A_log")
                put(M.dt_bias, pre + "dt_bias")
                put(M.norm, pre + "norm")
                o, n = M.out_rows.off["right"], r.heads * r.vdim
                M.o[:, o:o + n].copy_(get(pre + "o", W, n).to(M.o.dtype))
            if L.ff:
                L.gate_up.zero_()
                L.down.zero_()
                L.gate_up[:L.ff].copy_(get(b + "mlp.gate", L.ff, W).to(self.dtype))
                L.gate_up[L.ffp:L.ffp + L.ff].copy_(get(b + "mlp.up", L.ff, W).to(self.dtype))
                L.down[:, :L.ff].copy_(get(b + "mlp.down", W, L.ff).to(self.dtype))
        return self._finish()

    def native_state_dict(self) -> dict:
        """The inverse of :meth:`load_state_dict_native` (tests, export)."""
        cfg, W = self.cfg, self.cfg.hidden
        sd = {"embed": self.embed, "head": self.lm_head[:cfg.vocab_size], "final.norm": self.final_norm, "final.norm.b": self.final_norm_b}
        if cfg.loop_times:
            sd["loop.step"] = self.steps
        for i, L in enumerate(self.layers):
            b, m, M = f"l{i}.", f"l{i}.mix.", L.mix
            for n in L.norms:
                sd.update({b + n: getattr(L, n), b + n + ".b": getattr(L, n + "_b")})
            par = L.type == "parallel"
            pre, s, t = m + ("left." if par else ""), M.spec, M.true
            for name, o, h, d, dp in self._head_blocks(M, pre):
                sd[name] = M.w_in[o:o + h * dp].view(h, dp, W)[:, :d].reshape(h * d, W)
                if o < M.bias.numel():
                    sd[name + ".b"] = M.bias[o:o + h * dp].view(h, dp)[:, :d].reshape(h * d)
            sd[pre + "o"] = M.o[:, :s.heads * s.vdim].reshape(W, s.heads, s.vdim)[:, :, :t.vdim].reshape(W, -1)
            if not par:
                sd.update({m + n: getattr(M, n) for n in ("lq1", "lk1", "lq2", "lk2")})
            else:
                sd[pre + "q.norm"] = M.q_norm.view(s.heads, s.dim)[:, :t.dim].reshape(-1)
                sd[pre + "k.norm"] = M.k_norm.view(s.kv_heads, s.dim)[:, :t.dim].reshape(-1)
                r, pre = M.delta, m + "right."
                for seg, n in r.segments():
                    sd[pre + seg[1:]] = M.w_in[M.rows.off[seg]:M.rows.off[seg] + n]
                for seg, n in r.segments()[:3]:
                    sd[f"{pre}{seg[1:]}.conv"] = M.conv_w[M.conv_rows.off[seg]:M.conv_rows.off[seg] + n]
                o = M.out_rows.off["right"]
                sd.update({pre + "A_log": M.A_log, pre + "dt_bias": M.dt_bias, pre + "norm": M.norm, pre + "o": M.o[:, o:o + r.heads * r.vdim]})
            if L.ff:
                sd.update({b + "mlp.gate": L.gate_up[:L.ff], b + "mlp.up": L.gate_up[L.ffp:L.ffp + L.ff], b + "mlp.down": L.down[:, :L.ff]})
        return {k: v.detach().clone().contiguous() for k, v in sd.items()}

    def decode_gemm_shapes(self):
        """(weight, swiglu) of the projections a decode step runs, one per distinct shape, for the engine's
        decode GEMM routing (ops.tune_decode)."""
        if self.dtype != torch.bfloat16:
            return []   # f32 activations run on the vendor library: nothing to route
        seen, out = set(), []
        for L in self.layers:
            for w, sw in [(L.mix.w_in, False), (L.mix.o, False)] + ([(L.gate_up, True), (L.down, False)] if L.ff else []):
                if (tuple(w.shape), sw) not in seen:
                    seen.add((tuple(w.shape), sw))
                    out.append((w, sw))
        return [(w, sw) for w, sw in out + [(self.lm_head, False)] if w.numel() >= 1 << 20]

    # ------------------------------------------------------------------ caches
    def make_caches(self, num_blocks: int, block_size: int, num_slots: int) -> list:
        """One entry per layer RUN: paged (K, V) and, for a parallel layer, (convolution state, f32 state) over the slots.
        Zero-filled: a masked key or a padding column may be read (and multiplied by zero), never a NaN pattern left by the
        allocator."""
        caches = []
        for li, _ in self.runs:
            M = self.layers[li].mix
            s = M.spec
            if not ops.sigattn_supported(s.heads, s.kv_heads, s.dim, s.vdim, block_size, self.dtype):
                raise ValueError(f"attention kernels do not cover {s} with block size {block_size}")
            kv = s.make_caches(num_blocks, block_size, self.dtype, self.device)
            caches.append(kv + M.delta.make_state(num_slots, self.dtype, self.device) if isinstance(M, _Parallel) else kv)
        return caches

    def cache_block_bytes(self, block_size: int) -> int:
        return sum(self.layers[li].mix.spec.bytes_per_token(self.dtype) for li, _ in self.runs) * block_size

    def state_slot_bytes(self) -> int:
        return sum(self.layers[li].mix.delta.state_bytes(self.dtype) for li, _ in self.runs if self.layers[li].type == "parallel")

    def kv_bytes_per_token(self) -> int:
        return self.cache_block_bytes(1)

    # ------------------------------------------------------------------ forward
    def _mixer(self, L: KebepelLayer, h, meta: AttnMeta, cache):
        M, eps = L.mix, self.cfg.norm_eps
        u = ops.linear(h, M.w_in)
        T, s = u.shape[0], M.spec
        if L.type == "attention":
            y = torch.empty(T, s.heads * s.vdim, dtype=u.dtype, device=u.device)
            diff_attention(u, M.rows, cache, meta, s, M.bias, M.lam, eps, y)
        else:
            r, n = M.out_rows, M.delta.heads * M.delta.vdim
            full = r.off["right"] + n == r.total            # else: columns that nothing writes, against zero weights
            y = (torch.empty if full else torch.zeros)(T, r.total, dtype=u.dtype, device=u.device)
            row_norm_attention(u, M.rows, cache, meta, s, M.bias, M.q_norm, M.k_norm, M.freq, M.hscale, eps, y, M.left_scale)
            head_delta_mixer(u, M.rows, M.conv_rows, M.conv_w, M.dt_bias, M.A_log, M.norm_w, M.delta, eps, cache[2:], meta, y[:, r.off["right"]:])
        return ops.linear(y, M.o)

    def forward(self, ids: torch.Tensor, meta: AttnMeta, caches, taps: list = None) -> torch.Tensor:
        """-> normed hidden rows [R, W] that feed the LM head (``meta.logits_idx``, or every row).
        ``taps``: a list that receives a copy of the f32 stream after every layer run (debugging and tests)."""
        eps, dt, n = self.cfg.norm_eps, self.dtype, len(self.runs)
        x, _ = ops.embed_stream(ids, self.embed, dt)
        step = lambda t: None if t is None else self.steps[t]
        h = ops.stream_sandwich_layernorm(x, None, None, None, step(self.runs[0][1]), *self.layers[self.runs[0][0]].ln("norm1"), eps, dt)
        for i, (li, _) in enumerate(self.runs):
            L = self.layers[li]
            y, post = self._mixer(L, h, meta, caches[i]), "norm1b"
            if L.ff:
                h = ops.stream_sandwich_layernorm(x, y, *L.ln(post), None, *L.ln("norm2"), eps, dt)
                y, post = ops.linear(ops.linear_swiglu_any(h, L.gate_up), L.down), "norm2b"
            if taps is not None:     # the stream before the next pass's step vector
                t = x.clone()
                ops.stream_sandwich_layernorm(t, y, *L.ln(post), None, self.final_norm, self.final_norm_b, eps, dt)
                taps.append(t)
            if i + 1 == n:
                return ops.stream_sandwich_layernorm(x, y, *L.ln(post), None, self.final_norm, self.final_norm_b, eps, dt,
                                                     idx=meta.logits_idx)
            h = ops.stream_sandwich_layernorm(x, y, *L.ln(post), step(self.runs[i + 1][1]), *self.layers[self.runs[i + 1][0]].ln("norm1"), eps, dt)

    def head(self, hidden):
        return ops.linear(hidden, self.lm_head)[:, : self.cfg.vocab_size]

    def logits(self, hidden, gather: bool = True, dtype=torch.float32):
        lg = self.head(hidden)
        return lg if dtype is None else lg.to(dtype)

    def greedy(self, hidden):
        return self.tp.greedy_ids(self.head(hidden), self.vocab_lo)


def random_state_dict(cfg: KebepelConfig, seed: int = 0) -> dict:
    """Random f32 tensors under the checkpoint names for ``cfg`` (presets, benchmarks, tests)."""
    g = torch.Generator().manual_seed(seed)
    W = cfg.hidden

    def rn(*shape, scale=1.0, shift=0.0):
        return torch.randn(*shape, generator=g) * scale + shift

    def lin(out, inp, gain=1.0):
        return rn(out, inp, scale=gain / math.sqrt(inp))

    def ln(name, w=1.0):
        return {name: rn(W, scale=0.1, shift=w), name + ".b": rn(W, scale=0.1)}

    sd = {"embed": rn(cfg.vocab_size, W), "head": lin(cfg.vocab_size, W), **ln("final.norm")}
    if cfg.loop_times:
        sd["loop.step"] = rn(cfg.loop_times, W, scale=0.5)
    for i, l in enumerate(cfg.layers):
        b, m = f"l{i}.", f"l{i}.mix."
        sd.update({**ln(b + "norm1"), **ln(b + "norm1b", 0.7)})
        if l.type == "attention":
            s = DiffAttnSpec.from_dict(l.mixer)
            nq, nk, nv, no = 2 * s.heads * s.dim, 2 * s.kv_heads * s.dim, s.kv_heads * s.vdim, s.heads * s.vdim
            p = m
            sd.update({p + n: rn(s.dim, scale=0.3 * s.dim ** -0.25) for n in ("lq1", "lk1", "lq2", "lk2")})
        else:
            s = RowNormAttnSpec.from_dict(l.mixer["left"])
            nq, nk, nv, no = s.heads * s.dim, s.kv_heads * s.dim, s.kv_heads * s.vdim, s.heads * s.vdim
            p = m + "left."
            sd.update({p + "q.norm": rn(nq, scale=0.2, shift=1.5), p + "k.norm": rn(nk, scale=0.2, shift=1.5)})
            r, rp = HeadDeltaSpec.from_dict(l.mixer["right"]), m + "right."
            nrk, nrv = r.kv_heads * r.dim, r.heads * r.vdim
            sd.update({rp + "q": lin(nrk, W), rp + "k": lin(nrk, W), rp + "v": lin(nrv, W), rp + "b": lin(r.heads, W), rp + "a": lin(r.heads, W),
                       rp + "g": lin(nrv, W), rp + "q.conv": rn(nrk, r.conv, scale=0.5), rp + "k.conv": rn(nrk, r.conv, scale=0.5),
                       rp + "v.conv": rn(nrv, r.conv, scale=0.5), rp + "A_log": rn(r.heads, scale=0.5, shift=-1.0),
                       rp + "dt_bias": rn(r.heads, scale=0.5, shift=-1.0), rp + "norm": rn(r.vdim, scale=0.1, shift=1.0), rp + "o": lin(W, nrv)})
        sd.update({p + "q": lin(nq, W, 1.5), p + "k": lin(nk, W, 1.5), p + "v": lin(nv, W), p + "q.b": rn(nq, scale=0.3), p + "k.b": rn(nk, scale=0.3),
                   p + "v.b": rn(nv, scale=0.3), p + "g": lin(no, W), p + "o": lin(W, no)})
        if l.mlp:
            ff = int(l.mlp["ff"])
            sd.update({**ln(b + "norm2"), **ln(b + "norm2b", 0.7), b + "mlp.gate": lin(ff, W), b + "mlp.up": lin(ff, W), b + "mlp.down": lin(W, ff)})
    return sd
