"""Kafilorn: a residual stream kept as several mixed copies, over matrix-memory (mLSTM) and shared-latent attention mixers,
with squared-relu or routed-expert feed-forwards.

    X_s = embed[token] * scale                                                   s = 1 .. S    (f32 streams)
    per layer and sublayer q:  u = sum_s in_q[s] X_s;  r = sublayer(ln(u) w);
                               X_t <- sum_s mix_q[s, t] X_s + out_q[t] r          (the feed-forward may be absent)
    logits = head . (ln(sum_s X_s) w_f) * logit_scale                             ln(v) = (v - mean) / sqrt(var + eps)

Mixers (``cfg.layers``, any order): ``mlstm`` -- ``models.linear_state.mlstm_mixer``; ``latent_attention`` --
``models.latent_attention.cached_latent_attention`` (sliding window, learned sink per head; ``kv_from``: reads an earlier layer's
cache).  Feed-forward: ``dense`` -- ``W_down relu(W_up h)^2``; ``moe`` -- ``ops.router_choice`` + ``ops.routed_experts`` (+ a shared
expert of the same form for every token).

MI355X layout decisions:
  * a sublayer boundary is one pass over the token's streams (``ops.stream_hyper_norm``): the sum of the sublayer's results (mixer or
    dense rows, shared expert, weighted expert rows) through the mixing matrix, the next sublayer's combination of the streams and
    its layer norm; before the first update the copies are equal and are not materialised;
  * the latent is cached once per token (not per head, not per reading layer); scores and averages run on it directly;
  * gates and router logits are f32 results of skinny MFMA products over the normed rows, with soft cap, log-sigmoid, score and choice
    in the same kernel;
  * the matrix memory is one f32 tensor per layer over the engine's state slots.

Checkpoint format: ``config.json`` (``KafilornConfig.from_json``) and ``model.safetensors`` with ``embed``, ``head``, ``final.norm``,
``l<i>.norm1 | norm2``, ``l<i>.hc1 | hc2 .in | .out | .mix``, ``l<i>.mix.*``, ``l<i>.mlp.up | down`` (dense) or ``l<i>.mlp.router |
correction``, ``l<i>.mlp.e<j>.gate | up | down``, ``l<i>.mlp.shared.gate | up | down`` (moe); linear weights [out, in].
"""
from __future__ import annotations

import math

import torch
import torch.nn as nn

from .. import ops
from ..parallel.tp import SINGLE, TPGroup
from .attention import AttnMeta
from .configs import KafilornConfig, pad_vocab
from .latent_attention import CachedLatentAttnSpec, cached_latent_attention
from .linear_state import MLSTMSpec, mlstm_mixer


def _p(*shape, **kw):
    return nn.Parameter(torch.zeros(*shape, **kw), requires_grad=False)


def _pad8(n: int) -> int:
    return -(-int(n) // 8) * 8


class _MLSTM(nn.Module):
    """Weights of an ``mlstm`` mixer under checkpoint prefix ``mix.``."""

    def __init__(self, m: dict, W: int, e: dict, f: dict):
        super().__init__()
        s = self.spec = MLSTMSpec.from_dict(m)
        self.rows = s.rows(W)
        self.w_in = _p(self.rows.total, W, **e)
        self.w_gates = _p(2 * s.heads, W, **e)                  # input gate rows, then forget gate rows
        self.gate_bias = _p(2 * s.heads, **f)
        self.norm = _p(s.heads * s.vdim, **f)
        self.o = _p(W, s.heads * s.vdim, **e)

    def init_constants(self):
        pass


class _Latent(nn.Module):
    """Weights of a ``latent_attention`` mixer under checkpoint prefix ``mix.``."""

    def __init__(self, m: dict, W: int, e: dict, f: dict):
        super().__init__()
        s = self.spec = CachedLatentAttnSpec.from_dict(m)
        H, rp = s.heads, s.row[0]
        self.rows = s.rows(W)
        self.w_in = _p(self.rows.total, W, **e)
        self.w_uq = _p(H * s.qdim, s.q_rank, **e)
        self.w_uk = _p(H, rp, s.kdim, **e)                      # W_uk transposed per head: it acts on the queries
        self.w_uv = _p(H, s.vdim_p, rp, **e)
        self.dq_norm = _p(s.q_rank, **f)
        self.dkv_norm = _p(s.kv_rank, **f) if s.kv_from is None else None
        self.sink = _p(H, **f)
        self.o = _p(W, H * s.vdim_p, **e)
        self.freq = _p(max(s.rot_dim // 2, 1), **f)

    def init_constants(self):
        self.freq.copy_(self.spec.rot.freq_tensor(self.freq.device))


class _DenseFF(nn.Module):
    """Weights of a dense feed-forward under checkpoint prefix ``mlp.``."""

    def __init__(self, mlp: dict, W: int, e: dict):
        super().__init__()
        self.ff = int(mlp["ff"])
        self.ffp = _pad8(self.ff)                               # zero up rows and down columns behind ff
        self.up = _p(self.ffp, W, **e)
        self.down = _p(W, self.ffp, **e)


class _RoutedFF(nn.Module):
    """Weights of a mixture-of-experts feed-forward under checkpoint prefix ``mlp.``."""

    def __init__(self, mlp: dict, W: int, e: dict, f: dict):
        super().__init__()
        r = mlp["router"]
        gr = r.get("groups") or {}
        self.experts, self.top = int(r["experts"]), int(r["top"])
        self.groups, self.keep = int(gr.get("count", 1)), int(gr.get("keep", gr.get("count", 1)))
        self.ff = int(mlp["expert"]["ff"])
        self.ffp = _pad8(self.ff)
        if self.experts % self.groups or not 1 <= self.keep <= self.groups or not 1 <= self.top <= self.experts // self.groups * self.keep:
            raise ValueError(f"router: {self.top} of {self.experts} experts in {self.keep} of {self.groups} groups")
        self.router = _p(self.experts, W, **e)
        self.correction = _p(self.experts, **f)
        self.gate_up = _p(self.experts, 2 * self.ffp, W, **e)
        self.down = _p(self.experts, W, self.ffp, **e)
        sh = mlp.get("shared")
        self.sff = int(sh["ff"]) if sh else 0
        self.sffp = _pad8(self.sff)
        if self.sff:
            self.shared_gate_up = _p(2 * self.sffp, W, **e)
            self.shared_down = _p(W, self.sffp, **e)


class _Streams(nn.Module):
    """One sublayer's stream constants under checkpoint prefix ``hc1.`` / ``hc2.``."""

    def __init__(self, S: int, f: dict):
        super().__init__()
        self.w_in, self.w_out, self.mix = _p(S, **f), _p(S, **f), _p(S, S, **f)


class KafilornLayer(nn.Module):
    def __init__(self, cfg: KafilornConfig, spec, dtype, device):
        super().__init__()
        W = cfg.hidden
        e = dict(dtype=dtype, device=device)
        f = dict(dtype=torch.float32, device=device)   # norms, stream constants and per-head constants stay f32
        self.type = spec.type
        self.norm1, self.hc1 = _p(W, **f), _Streams(cfg.streams, f)
        self.mix = {"mlstm": _MLSTM, "latent_attention": _Latent}[spec.type](spec.mixer, W, e, f)
        self.kind = spec.mlp["kind"] if spec.mlp else None
        if self.kind is not None:
            self.norm2, self.hc2 = _p(W, **f), _Streams(cfg.streams, f)
            self.mlp = _DenseFF(spec.mlp, W, e) if self.kind == "dense" else _RoutedFF(spec.mlp, W, e, f)


class KafilornModel(nn.Module):
    stateful = True            # recurrent state per sequence: no prefix reuse, chunks run as prompt portions

    def __init__(self, cfg: KafilornConfig, tp: TPGroup = SINGLE, dtype=torch.bfloat16, device="cpu"):
        super().__init__()
        if tp.enabled:
            raise NotImplementedError("the Kafilorn decoder runs on one GPU (no tensor-parallel sharding)")
        if cfg.streams > ops.MAX_STREAMS:
            raise ValueError(f"{cfg.streams} streams (the stream kernel holds {ops.MAX_STREAMS})")
        self.cfg, self.tp, self.dtype, self.device = cfg, tp, dtype, torch.device(device)
        e = dict(dtype=dtype, device=device)
        f = dict(dtype=torch.float32, device=device)
        self.vocab_lo, self.vocab_local = 0, cfg.vocab_size
        self.embed = _p(cfg.vocab_size, cfg.hidden, **e)
        self.lm_head = _p(pad_vocab(cfg.vocab_size, 64), cfg.hidden, **e)     # zero rows: logits rows start 32-byte aligned
        self.layers = nn.ModuleList([KafilornLayer(cfg, l, dtype, device) for l in cfg.layers])
        self.final_norm = _p(cfg.hidden, **f)
        att = [L.mix.spec for L in self.layers if L.type == "latent_attention"]
        self.hq = max((s.heads for s in att), default=1)
        self.hkv = 1
        self.D = max((sum(s.row) for s in att), default=16)

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

    @torch.no_grad()
    def load_state_dict_native(self, sd: dict):
        """Tensors named as in the checkpoint format (module docstring)."""
        cfg, W, S = self.cfg, self.cfg.hidden, self.cfg.streams

        def get(name, *shape):
            t = sd[name]
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"{name}: checkpoint shape {tuple(t.shape)} != {tuple(shape)}")
            return t

        def put(p, name):
            p.copy_(get(name, *p.shape).to(p.dtype))

        def rows_in(dst, name, n):
            """``n`` checkpoint rows at the head of a zeroed block of rows."""
            dst[:n].copy_(get(name, n, dst.shape[1]).to(dst.dtype))

        def glu_in(gate_up, down, prefix, ff, ffp):
            gate_up.zero_()
            down.zero_()
            rows_in(gate_up[:ffp], prefix + "gate", ff)
            rows_in(gate_up[ffp:], prefix + "up", ff)
            down[:, :ff].copy_(get(prefix + "down", W, ff).to(down.dtype))

        put(self.embed, "embed")
        self.lm_head.zero_()
        rows_in(self.lm_head, "head", cfg.vocab_size)
        put(self.final_norm, "final.norm")
        for i, L in enumerate(self.layers):
            b, m = f"l{i}.", f"l{i}.mix."
            for q in (1, 2) if L.kind is not None else (1,):
                hc = getattr(L, f"hc{q}")
                put(getattr(L, f"norm{q}"), f"{b}norm{q}")
                put(hc.w_in, f"{b}hc{q}.in")
                put(hc.w_out, f"{b}hc{q}.out")
                put(hc.mix, f"{b}hc{q}.mix")
            M, s = L.mix, L.mix.spec
            H = s.heads
            M.w_in.zero_()
            if L.type == "mlstm":
                for seg, n in (("q", H * s.dim), ("k", H * s.dim), ("v", H * s.vdim), ("g", H * s.vdim)):
                    rows_in(M.w_in[M.rows.off[seg]:], m + seg, n)
                rows_in(M.w_gates[:H], m + "i", H)
                rows_in(M.w_gates[H:], m + "f", H)
                M.gate_bias[:H].copy_(get(m + "i.b", H).float())
                M.gate_bias[H:].copy_(get(m + "f.b", H).float())
                put(M.norm, m + "norm")
                put(M.o, m + "o")
            else:
                rows_in(M.w_in[M.rows.off["dq"]:], m + "dq", s.q_rank)
                put(M.dq_norm, m + "dq.norm")
                if s.kv_from is None:
                    rows_in(M.w_in[M.rows.off["dkv"]:], m + "dkv", s.kv_rank + s.rot_dim)
                    put(M.dkv_norm, m + "dkv.norm")
                for p in (M.w_uq, M.w_uk, M.w_uv, M.o):
                    p.zero_()
                qd = s.dim + s.rot_dim
                M.w_uq.view(H, s.qdim, s.q_rank)[:, :qd].copy_(get(m + "uq", H * qd, s.q_rank).view(H, qd, s.q_rank).to(self.dtype))
                M.w_uk[:, :s.kv_rank, :s.dim].copy_(get(m + "uk", H * s.dim, s.kv_rank).view(H, s.dim, s.kv_rank).transpose(1, 2).to(self.dtype))
                M.w_uv[:, :s.vdim, :s.kv_rank].copy_(get(m + "uv", H * s.vdim, s.kv_rank).view(H, s.vdim, s.kv_rank).to(self.dtype))
                put(M.sink, m + "sink")
                M.o.view(W, H, s.vdim_p)[:, :, :s.vdim].copy_(get(m + "o", W, H * s.vdim).view(W, H, s.vdim).to(self.dtype))
            if L.kind is None:
                continue
            X = L.mlp
            if L.kind == "dense":
                X.up.zero_()
                X.down.zero_()
                rows_in(X.up, b + "mlp.up", X.ff)
                X.down[:, :X.ff].copy_(get(b + "mlp.down", W, X.ff).to(self.dtype))
            else:
                put(X.router, b + "mlp.router")
                put(X.correction, b + "mlp.correction")
                for j in range(X.experts):
                    glu_in(X.gate_up[j], X.down[j], f"{b}mlp.e{j}.", X.ff, X.ffp)
                if X.sff:
                    glu_in(X.shared_gate_up, X.shared_down, b + "mlp.shared.", X.sff, X.sffp)
        return self._finish()

    def native_state_dict(self) -> dict:
        """The inverse of :meth:`load_state_dict_native` (tests, export)."""
        cfg, W = self.cfg, self.cfg.hidden
        sd = {"embed": self.embed, "head": self.lm_head[:cfg.vocab_size], "final.norm": self.final_norm}

        def glu_out(gate_up, down, prefix, ff, ffp):
            sd.update({prefix + "gate": gate_up[:ff], prefix + "up": gate_up[ffp:ffp + ff], prefix + "down": down[:, :ff]})

        for i, L in enumerate(self.layers):
            b, m = f"l{i}.", f"l{i}.mix."
            for q in (1, 2) if L.kind is not None else (1,):
                hc = getattr(L, f"hc{q}")
                sd.update({f"{b}norm{q}": getattr(L, f"norm{q}"), f"{b}hc{q}.in": hc.w_in, f"{b}hc{q}.out": hc.w_out, f"{b}hc{q}.mix": hc.mix})
            M, s = L.mix, L.mix.spec
            H = s.heads
            if L.type == "mlstm":
                for seg, n in (("q", H * s.dim), ("k", H * s.dim), ("v", H * s.vdim), ("g", H * s.vdim)):
                    sd[m + seg] = M.w_in[M.rows.off[seg]:M.rows.off[seg] + n]
                sd.update({m + "i": M.w_gates[:H], m + "f": M.w_gates[H:], m + "i.b": M.gate_bias[:H], m + "f.b": M.gate_bias[H:],
                           m + "norm": M.norm, m + "o": M.o})
            else:
                qd = s.dim + s.rot_dim
                sd.update({m + "dq": M.w_in[M.rows.off["dq"]:M.rows.off["dq"] + s.q_rank], m + "dq.norm": M.dq_norm,
                           m + "uq": M.w_uq.view(H, s.qdim, s.q_rank)[:, :qd].reshape(H * qd, s.q_rank),
                           m + "uk": M.w_uk[:, :s.kv_rank, :s.dim].transpose(1, 2).reshape(H * s.dim, s.kv_rank),
                           m + "uv": M.w_uv[:, :s.vdim, :s.kv_rank].reshape(H * s.vdim, s.kv_rank), m + "sink": M.sink,
                           m + "o": M.o.view(W, H, s.vdim_p)[:, :, :s.vdim].reshape(W, -1)})
                if s.kv_from is None:
                    o = M.rows.off["dkv"]
                    sd.update({m + "dkv": M.w_in[o:o + s.kv_rank + s.rot_dim], m + "dkv.norm": M.dkv_norm})
            if L.kind is None:
                continue
            X = L.mlp
            if L.kind == "dense":
                sd.update({b + "mlp.up": X.up[:X.ff], b + "mlp.down": X.down[:, :X.ff]})
            else:
                sd.update({b + "mlp.router": X.router, b + "mlp.correction": X.correction})
                for j in range(X.experts):
                    glu_out(X.gate_up[j], X.down[j], f"{b}mlp.e{j}.", X.ff, X.ffp)
                if X.sff:
                    glu_out(X.shared_gate_up, X.shared_down, b + "mlp.shared.", X.sff, X.sffp)
        return {k: v.detach().clone().contiguous() for k, v in sd.items()}

    def decode_gemm_shapes(self):
        """(weight, swiglu) of the dense projections a decode step runs, one per distinct shape, for the
        engine's decode GEMM routing (ops.tune_decode)."""
        if self.dtype != torch.bfloat16:
            return []   # f32 activations run on the vendor library: nothing to route
        seen, out = set(), []

        def add(w, sw=False):
            if (tuple(w.shape), sw) not in seen:
                seen.add((tuple(w.shape), sw))
                out.append((w, sw))

        for L in self.layers:
            M = L.mix
            for w in [M.w_in, M.o] + ([M.w_uq] if L.type == "latent_attention" else []):
                add(w)
            if L.kind == "dense":
                add(L.mlp.up)
                add(L.mlp.down)
            elif L.kind == "moe" and L.mlp.sff:
                add(L.mlp.shared_gate_up, True)
                add(L.mlp.shared_down)
        add(self.lm_head)
        return [(w, sw) for w, sw in out if w.numel() >= 1 << 20]

    # ------------------------------------------------------------------ caches
    def make_caches(self, num_blocks: int, block_size: int, num_slots: int) -> list:
        """One entry per layer: an mLSTM layer's state over the slots, a latent layer's paged rows, or -- the same tensor --
        the rows of the layer it shares.  Zero-filled: a masked row or a padding column may be read (and multiplied by
        zero), never a NaN pattern left by the allocator."""
        if block_size % 16:
            raise ValueError("the latent attention kernels read pages of a multiple of 16 tokens")
        caches = []
        for L in self.layers:
            s = L.mix.spec
            if L.type == "mlstm":
                caches.append(s.make_state(num_slots, self.dtype, self.device))
            elif s.kv_from is not None:
                caches.append(caches[s.kv_from])
            else:
                caches.append(s.make_cache(num_blocks, block_size, self.dtype, self.device))
        return caches

    def cache_block_bytes(self, block_size: int) -> int:
        return sum(L.mix.spec.bytes_per_token(self.dtype) for L in self.layers if L.type == "latent_attention") * block_size

    def state_slot_bytes(self) -> int:
        return sum(L.mix.spec.state_bytes(self.dtype) for L in self.layers if L.type == "mlstm")

    def kv_bytes_per_token(self) -> int:
        return self.cache_block_bytes(1)

    # ------------------------------------------------------------------ forward
    def _mixer(self, L: KafilornLayer, h, meta: AttnMeta, cache):
        M, eps = L.mix, self.cfg.norm_eps
        if L.type == "mlstm":
            return mlstm_mixer(h, M.w_in, M.w_gates, M.gate_bias, M.rows, M.norm, M.o, M.spec, eps, cache, meta, self.dtype)
        att = cached_latent_attention(h, M.w_in, M.rows, M.w_uq, M.w_uk, M.w_uv, M.dq_norm, M.dkv_norm, M.sink, cache, meta, M.spec, M.freq, eps)
        return ops.linear(att, M.o)

    def _ff(self, L: KafilornLayer, h):
        """-> (dense rows [T, W] or None, expert rows [T * top, W] or None, their weights f32 [T, top] or None)."""
        X = L.mlp
        if L.kind == "dense":
            return ops.linear(ops.relu_sq_(ops.linear(h, X.up)), X.down), None, None
        experts, weights = ops.router_choice(h, X.router, X.top, X.groups, X.keep, correction=X.correction)
        y = ops.routed_experts(h, experts, X.gate_up, X.down)
        b = ops.linear(ops.linear_swiglu_any(h, X.shared_gate_up), X.shared_down) if X.sff else None
        return b, y, weights

    def forward(self, ids: torch.Tensor, meta: AttnMeta, caches, taps: list = None) -> torch.Tensor:
        """-> normed hidden rows [R, W] that feed the LM head (``meta.logits_idx``, or every row).
        ``taps``: a list that receives the sum of the f32 streams after every layer (debugging and tests)."""
        eps, S, n = self.cfg.norm_eps, self.cfg.streams, len(self.layers)
        x, _ = ops.embed_stream(ids, self.embed, self.dtype, self.cfg.embed_scale)
        L0 = self.layers[0]
        x, h = ops.stream_hyper_norm(x, S, w_in=L0.hc1.w_in, norm_w=L0.norm1, eps=eps, out_dtype=self.dtype)
        for i, L in enumerate(self.layers):
            a = self._mixer(L, h, meta, caches[i])
            nxt = self.layers[i + 1] if i + 1 < n else None
            to_next = (nxt.hc1.w_in, nxt.norm1) if nxt is not None else (None, None)
            w_in, norm_w = (L.hc2.w_in, L.norm2) if L.kind else to_next
            x, h = ops.stream_hyper_norm(x, S, a, None, None, None, L.hc1.mix, L.hc1.w_out, w_in, norm_w, eps, self.dtype)
            if L.kind:
                b, y, yw = self._ff(L, h)
                x, h = ops.stream_hyper_norm(x, S, None, b, y, yw, L.hc2.mix, L.hc2.w_out, *to_next, eps, self.dtype)
            if taps is not None:
                taps.append(x.sum(1))
        idx = meta.logits_idx
        if idx is None:
            idx = torch.arange(x.shape[0], dtype=torch.long, device=x.device)
        # the LM head is linear: the logit scale goes into the f32 rows it reads
        return ops.stream_hyper_norm(x, S, norm_w=self.final_norm, eps=eps, out_dtype=self.dtype, idx=idx, out_scale=self.cfg.logit_scale)[1]

    def head(self, hidden):
        return ops.linear(hidden, self.lm_head)[:, : self.cfg.vocab_size]

    def logits(self, hidden, gather: bool = True, dtype=torch.float32):
        lg = self.head(hidden)
        return lg if dtype is None else lg.to(dtype)

    def greedy(self, hidden):
        return self.tp.greedy_ids(self.head(hidden), self.vocab_lo)


def random_state_dict(cfg: KafilornConfig, seed: int = 0) -> dict:
    """Random f32 tensors under the checkpoint names for ``cfg`` (presets, benchmarks, tests)."""
    g = torch.Generator().manual_seed(seed)
    W, S = cfg.hidden, cfg.streams

    def rn(*shape, scale=1.0, shift=0.0):
        return torch.randn(*shape, generator=g) * scale + shift

    def lin(out, inp, gain=1.0):
        return rn(out, inp, scale=gain / math.sqrt(inp))

    def glu(prefix, ff):
        return {prefix + "gate": lin(ff, W), prefix + "up": lin(ff, W), prefix + "down": lin(W, ff)}

    sd = {"embed": rn(cfg.vocab_size, W), "head": lin(cfg.vocab_size, W, 2.0), "final.norm": rn(W, scale=0.1, shift=1.0)}
    for i, l in enumerate(cfg.layers):
        b, m = f"l{i}.", f"l{i}.mix."
        for q in (1, 2) if l.mlp else (1,):
            sd[f"{b}norm{q}"] = rn(W, scale=0.1, shift=1.0)
            sd[f"{b}hc{q}.in"] = rn(S, scale=0.3, shift=1.0 / S)
            sd[f"{b}hc{q}.out"] = rn(S, scale=0.3, shift=1.0)
            sd[f"{b}hc{q}.mix"] = torch.eye(S) * 0.9 + rn(S, S, scale=0.1 / S)
        if l.type == "mlstm":
            s = MLSTMSpec.from_dict(l.mixer)
            H = s.heads
            sd.update({m + "q": lin(H * s.dim, W), m + "k": lin(H * s.dim, W), m + "v": lin(H * s.vdim, W), m + "g": lin(H * s.vdim, W),
                       m + "o": lin(W, H * s.vdim, 2.0), m + "norm": rn(H * s.vdim, scale=0.1, shift=1.0), m + "i": lin(H, W, 1.5),
                       m + "f": lin(H, W, 1.5), m + "i.b": rn(H, scale=0.5), m + "f.b": rn(H, scale=1.0, shift=3.0)})
        else:
            s = CachedLatentAttnSpec.from_dict(l.mixer)
            H = s.heads
            sd.update({m + "dq": lin(s.q_rank, W), m + "dq.norm": rn(s.q_rank, scale=0.1, shift=1.0),
                       m + "uq": lin(H * (s.dim + s.rot_dim), s.q_rank, 1.5), m + "uk": lin(H * s.dim, s.kv_rank, 1.5),
                       m + "uv": lin(H * s.vdim, s.kv_rank), m + "sink": rn(H), m + "o": lin(W, H * s.vdim, 2.0)})
            if s.kv_from is None:
                sd.update({m + "dkv": lin(s.kv_rank + s.rot_dim, W, 1.5), m + "dkv.norm": rn(s.kv_rank, scale=0.1, shift=1.0)})
        if not l.mlp:
            continue
        if l.mlp["kind"] == "dense":
            F = int(l.mlp["ff"])
            sd.update({b + "mlp.up": lin(F, W), b + "mlp.down": lin(W, F)})
        else:
            E = int(l.mlp["router"]["experts"])
            sd[b + "mlp.router"] = lin(E, W, 2.0)
            sd[b + "mlp.correction"] = rn(E, scale=0.1)
            for j in range(E):
                sd.update(glu(f"{b}mlp.e{j}.", int(l.mlp["expert"]["ff"])))
            if l.mlp.get("shared"):
                sd.update(glu(b + "mlp.shared.", int(l.mlp["shared"]["ff"])))
    return sd
