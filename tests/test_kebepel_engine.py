"""The Kebepel decoder through the framework's engine (model registry, loader, runner, paged cache, state
slots, scheduler, hipGraph decode, replay and generation entry points) against the plain float64 forward
of ``kebepel_oracle``.  Small random models of several shapes; CPU path and (``gpu`` marker) HIP kernels
in f32 and bf16."""
import io
import json

import pytest
import torch

import kebepel_oracle as O
from llm_kubernetes_minikube_sharp4dev_amd.engine.llm_engine import LLMEngine
from llm_kubernetes_minikube_sharp4dev_amd.engine.sampling import SamplingParams
from llm_kubernetes_minikube_sharp4dev_amd.models import KebepelConfig, KebepelModel, build_decoder, load_decoder_dir
from llm_kubernetes_minikube_sharp4dev_amd.models.configs import DECODERS, param_count

CPU32 = pytest.param("cpu", torch.float32, id="cpu-f32")
GPU32 = pytest.param("cuda", torch.float32, id="gpu-f32", marks=pytest.mark.gpu)
GPU16 = pytest.param("cuda", torch.bfloat16, id="gpu-bf16", marks=pytest.mark.gpu)
ALL = [CPU32, GPU32, GPU16]


def att(heads, kv, dim, vdim, scale, diff, temp=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if temp:
        m["q_temp"] = {"coef": temp[0], "every": temp[1]}
    return {"type": "attention", "mixer": m}


def par(heads, kv, dim, vdim, scale, rot, cap, rh, rkv, rdim, rvdim, conv, ls=0.7, rs=1.3):
    left = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if cap:
        left["softcap"] = cap
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": rh, "kv_heads": rkv, "dim": rdim, "vdim": rvdim, "conv": conv},
                                          "left_scale": ls, "right_scale": rs}}


def yarn(dims, base, factor, original, fast, slow):
    return {"dims": dims, "base": base, "scaling": {"factor": factor, "original": original, "fast": fast, "slow": slow}}


def ff(layer, n):
    return dict(layer, mlp={"kind": "dense", "ff": n} if n else None)


def config(layers, width, loop=None, vocab=97, eps=1e-5):
    d = {"architecture": "Kebepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


CONFIGS = {
    # both mixers, GQA on every side, the first two layers (one without a feed-forward) run three times
    "three": config([ff(par(4, 2, 24, 16, 0.2, yarn(16, 100.0, 4.0, 32, 8.0, 1.0), 5.0, 4, 2, 16, 8, 3), 80), ff(att(4, 2, 12, 20, 0.4, 0.25, (0.7, 5)), 0),
                     ff(par(3, 3, 16, 8, 0.3, {"dims": 8, "base": 1000.0}, 0.0, 2, 2, 12, 20, 4, 1.2, 0.5), 50)], 64, (0, 2, 3)),
    # one head / one kv head, a loop of one pass over the last layer alone (its step vector is added all the same), two taps, no
    # temperature, no cap, sizes that are multiples of nothing convenient
    "odd": config([ff(att(1, 1, 10, 14, 0.35, 0.6), 50), ff(par(3, 1, 20, 12, 0.3, {"dims": 20, "base": 1000.0}, 0.0, 3, 3, 10, 14, 2), 27),
                   ff(att(3, 1, 7, 9, 0.5, 0.1, (0.4, 1)), 0)], 36, (2, 3, 1), vocab=61, eps=1e-6),
    # no loop; more heads of a kv group than a tile of the attention kernels holds, wide key heads, a long convolution, every dimension rotated
    "wide": config([ff(par(18, 1, 40, 24, 0.15, yarn(40, 10000.0, 8.0, 64, 32.0, 1.0), 20.0, 2, 1, 72, 100, 7, 0.3, 2.0), 64),
                    ff(att(17, 1, 12, 40, 0.3, 0.5, (2.0, 64)), 30), ff(par(2, 2, 10, 136, 0.4, {"dims": 2, "base": 10.0}, 1.5, 1, 1, 130, 9, 1), 0)],
                   56, vocab=130),
    # differential attention alone: pages only
    "pages": config([ff(att(2, 2, 6, 8, 0.5, 0.2, (0.3, 3)), 0), ff(att(6, 2, 16, 10, 0.3, 0.7), 40)], 44, (0, 1, 2)),
    # projections the MFMA / weight-streaming kernels tile: no vendor GEMM, decode steps captured in hipGraphs
    "mid": config([ff(att(8, 4, 16, 32, 0.25, 0.3, (0.5, 32)), 512), ff(par(4, 1, 64, 64, 0.125, yarn(64, 10000.0, 4.0, 64, 32.0, 1.0), 30.0, 4, 2, 64, 64, 4), 256)],
                  256, (1, 2, 2), vocab=768),
}
_models = {}


def model_and_weights(name, device, dtype, seed=3):
    key = (name, device, dtype)
    if key not in _models:
        m = build_decoder(KebepelConfig.from_json(CONFIGS[name], name), device=device, dtype=dtype, seed=seed)
        _models[key] = (m, {k: v.cpu() for k, v in m.native_state_dict().items()})
    return _models[key]


def engine(m, tokens=512, seqs=4, **kw):
    return LLMEngine(m, None, block_size=16, max_model_len=tokens, max_num_seqs=seqs, num_blocks=-(-tokens // 16), eos_ids=set(), **kw)


def toks(n, vocab, seed):
    return torch.randint(0, vocab, (n,), generator=torch.Generator().manual_seed(seed)).tolist()


def close(got, want, dtype):
    """f32: every position within 1e-4 of the oracle.  bf16: the first tokens of a sequence are ill-conditioned
    in any 16-bit run of this design (a read-out of a state that holds one or two writes is a near-zero dot
    product times a value, and the per-head unit norm blows its rounding -- even its sign -- up to order one),
    so half of the positions must be within 3e-2 and none may be further off than half the logits' range;
    the f32 runs of the same kernels carry the sharp comparison."""
    want = want.double()
    err = (got.double().cpu() - want).abs().reshape(want.shape[0], -1).amax(1) / want.abs().max()
    if dtype == torch.float32:
        return float(err.max()) < 1e-4, float(err.max())
    return float(err.median()) < 3e-2 and float(err.max()) < 0.5, (float(err.median()), float(err.max()))


def replay(eng, rid, tokens, cuts, end=True):
    """Feed ``tokens`` in portions of the sizes ``cuts`` (the rest one by one); logits of every position."""
    out, at = [], 0
    sizes = list(cuts)
    while at < len(tokens):
        n = min(sizes.pop(0) if sizes else 1, len(tokens) - at)
        last = at + n == len(tokens)
        out.append(eng.replay_step([(rid, tokens[at:at + n], list(range(n)))], [rid] if last and end else []))
        at += n
    return torch.cat(out)


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_streams_and_logits(name, device, dtype):
    m, sd = model_and_weights(name, device, dtype)
    t = toks(45, m.cfg.vocab_size, 1)
    want, streams = O.forward(CONFIGS[name], sd, t, True)
    eng = engine(m)
    from llm_kubernetes_minikube_sharp4dev_amd.engine.sequence import Sequence
    sq = Sequence(list(t), SamplingParams(max_tokens=1))
    assert eng.scheduler.admit_forced(sq, len(t))
    si, _ = eng.runner.prepare([(sq, 0, len(t))], want={id(sq): list(range(len(t)))})
    ids, meta = eng.runner._meta(si)
    taps = []
    with torch.inference_mode():
        m(ids, meta, eng.runner.kv_caches, taps=taps)
    eng.scheduler.finish(sq, "stop")
    assert len(taps) == len(streams) == m.cfg.num_layers
    for r, (a, b) in enumerate(zip(taps, streams)):     # the f32 stream after every layer run
        ok, err = close(a, b, dtype)
        assert ok, (r, err)
    ok, err = close(replay(eng, "w", t, [len(t)]), want, dtype)
    assert ok, err


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("name", ["three", "odd", "wide", "pages"])
def test_prefill_equals_token_by_token_and_portions(name, device, dtype):
    """One step for the whole prompt, one token per step, and portions of changing size down to two tokens
    (cut inside pages and inside the recurrence's chunks) give the same logits at every position."""
    m, sd = model_and_weights(name, device, dtype)
    t = toks(70, m.cfg.vocab_size, 2)
    want = O.forward(CONFIGS[name], sd, t)
    eng = engine(m)
    for cuts in ([70], [], [1, 2, 2, 3, 16, 17, 5, 2], [33, 2, 31], [6, 7, 8]):
        ok, err = close(replay(eng, "r", t, cuts), want, dtype)
        assert ok, (cuts, err)


@pytest.mark.parametrize("device,dtype", ALL)
def test_mixed_batches_equal_each_request_alone(device, dtype):
    """Five requests of unequal lengths share steps: portions of some beside single tokens of others, a
    request sitting out steps, requests ending and a new one taking the freed pages and slot."""
    name = "three"
    m, sd = model_and_weights(name, device, dtype)
    V = m.cfg.vocab_size
    T = {"a": toks(60, V, 10), "b": toks(21, V, 11), "c": toks(9, V, 12), "d": toks(40, V, 13), "e": toks(33, V, 14)}
    want = {k: O.forward(CONFIGS[name], sd, v) for k, v in T.items()}
    plan = [[("a", 17)], [("a", 15), ("b", 20), ("c", 1)], [("a", 1), ("b", 1), ("c", 2), ("d", 31)],
            [("a", 1), ("c", 6), ("d", 1)], [("a", 26), ("d", 1)], [("d", 7), ("e", 2)], [("e", 30)], [("e", 1)]]
    eng = engine(m, tokens=160, seqs=4)   # a + b + c + d live together need 64 + 32 + 16 + 48 tokens of pages
    at = {k: 0 for k in T}
    got = {k: [] for k in T}
    for step in plan:
        entries, end = [], []
        for k, n in step:
            entries.append((k, T[k][at[k]:at[k] + n], list(range(n))))
            at[k] += n
            if at[k] == len(T[k]):
                end.append(k)
        lg = eng.replay_step(entries, end)
        r = 0
        for k, n in step:
            got[k].append(lg[r:r + n])
            r += n
    assert at == {k: len(v) for k, v in T.items()}
    assert eng.allocator.num_free == eng.runner.num_blocks and eng.state_pool.num_free == 4
    for k in T:
        ok, err = close(torch.cat(got[k]), want[k], dtype)
        assert ok, (k, err)
        # the same portions alone, in the same number format: nothing but rounding may separate the two runs
        alone = replay(eng, k + "-alone", T[k], [n for step in plan for kk, n in step if kk == k])
        d = float((alone.double() - torch.cat(got[k]).double()).abs().max() / want[k].abs().max())
        assert d < (1e-5 if dtype == torch.float32 else 6e-2), (k, d)


@pytest.mark.parametrize("device,dtype", ALL)
def test_freed_pages_and_slots_are_used_again(device, dtype):
    """A pool of exactly one request's size and ONE state slot: every request runs in the pages and the
    slot its predecessor left, and repeats its own first run bit for bit; a second live request is refused."""
    m, sd = model_and_weights("wide", device, dtype)
    V = m.cfg.vocab_size
    a, b = toks(48, V, 20), toks(41, V, 21)
    eng = engine(m, tokens=48, seqs=1)
    first = replay(eng, "a", a, [20, 5])
    other = replay(eng, "b", b, [3, 30])
    again = replay(eng, "a2", a, [20, 5])
    assert torch.equal(first, again)
    assert close(first, O.forward(CONFIGS["wide"], sd, a), dtype)[0]
    assert close(other, O.forward(CONFIGS["wide"], sd, b), dtype)[0]
    eng.replay_step([("x", a[:5], [])])
    with pytest.raises(RuntimeError):
        eng.replay_step([("y", b[:5], [])])


@pytest.mark.parametrize("device,dtype", ALL)
def test_long_decode_through_pages_and_temperature_steps(device, dtype):
    """150 single-token steps after a short prompt (across many page borders and steps of the query temperature), two requests side
    by side."""
    m, sd = model_and_weights("odd", device, dtype)
    V = m.cfg.vocab_size
    a, b = toks(170, V, 30), toks(158, V, 31)
    eng = engine(m, tokens=352, seqs=2)
    ga, gb = [eng.replay_step([("a", a[:20], list(range(20)))])], [eng.replay_step([("b", b[:8], list(range(8)))])]
    for i in range(150):
        lg = eng.replay_step([("a", [a[20 + i]], [0]), ("b", [b[8 + i]], [0])])
        ga.append(lg[:1])
        gb.append(lg[1:])
    for got, t in ((ga, a), (gb, b)):
        ok, err = close(torch.cat(got), O.forward(CONFIGS["odd"], sd, t), dtype)
        assert ok, err


@pytest.mark.parametrize("device,dtype", ALL)
@pytest.mark.parametrize("name", ["three", "wide", "pages"])
def test_greedy_generation_through_the_scheduler(name, device, dtype):
    """``LLMEngine.generate``: the scheduler admits, chunks (a 24-token step budget) and batches three
    prompts; every generated token must be the oracle's argmax for its prefix (or within a near tie)."""
    m, sd = model_and_weights(name, device, dtype)
    V = m.cfg.vocab_size
    prompts = [toks(50, V, 40), toks(7, V, 41), toks(1, V, 42)]
    eng = LLMEngine(m, None, block_size=16, max_model_len=256, max_num_seqs=3, num_blocks=16, eos_ids=set(),
                    max_num_batched_tokens=24)
    seqs = eng.generate(prompts, SamplingParams.greedy(12))
    assert eng.allocator.num_free == 16 and eng.state_pool.num_free == 3
    for p, s in zip(prompts, seqs):
        assert len(s.output_ids) == 12
        full = p + list(s.output_ids)
        lg = O.forward(CONFIGS[name], sd, full[:-1])[len(p) - 1:]
        for i, tid in enumerate(s.output_ids):
            gap = float(lg[i].max() - lg[i, tid])
            assert gap <= (1e-3 if dtype == torch.float32 else 0.25) * float(lg[i].max() - lg[i].min()), (i, gap)


def test_checkpoint_directory_selects_the_model_and_replays(tmp_path):
    """config.json + model.safetensors on disk: the registry picks the class by the architecture name, every tensor is used and
    its shape checked, and the trace command writes the logits it is asked for."""
    import numpy as np
    from safetensors.torch import save_file

    from llm_kubernetes_minikube_sharp4dev_amd.engine.replay import run_trace

    m, sd = model_and_weights("odd", "cpu", torch.float32)
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    sd16 = {k: v.to(torch.bfloat16) for k, v in sd.items()}
    save_file(sd16, str(d / "model.safetensors"))
    m2 = load_decoder_dir(str(d), dtype=torch.float32)
    assert isinstance(m2, KebepelModel) and m2.cfg.num_layers == 3
    t = toks(30, 61, 50)
    want = O.forward(CONFIGS["odd"], sd16, t)
    steps = [{"step": 0, "entries": [{"id": "q", "tokens": t[:19], "want": [0, 18]}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": t[19:20], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "q", "tokens": t[20:], "want": [9]}, {"id": "p", "tokens": t[:4], "want": [3]}],
              "end": ["q", "p"]}]
    out = io.StringIO()
    assert run_trace(str(d), "float32", str(tmp_path / "o"), 64, lines=[json.dumps(s) for s in steps], out=out, device="cpu") == 0
    assert out.getvalue().split() == ["done", "0", "done", "1", "done", "2"]
    l0 = torch.from_numpy(np.fromfile(tmp_path / "o" / "0.f32", dtype="<f4")).view(2, 61)
    l2 = torch.from_numpy(np.fromfile(tmp_path / "o" / "2.f32", dtype="<f4")).view(2, 61)
    assert not (tmp_path / "o" / "1.f32").exists()
    assert close(l0, want[[0, 18]], torch.float32)[0] and close(l2, want[[29, 3]], torch.float32)[0]
    for name in ("l0.mix.q", "l1.mix.left.k.norm", "l1.mix.right.v.conv", "l2.norm1b.b", "loop.step", "l1.mix.right.dt_bias"):
        with pytest.raises(ValueError):
            KebepelModel(m2.cfg, dtype=torch.float32).load_state_dict_native(dict(sd16, **{name: sd16[name][:-1]}))
    # every tensor of the checkpoint matters to the model
    for name in sd16:
        other = KebepelModel(m2.cfg, dtype=torch.float32).load_state_dict_native(dict(sd16, **{name: sd16[name] * 1.25 + 0.1}))
        assert any(not torch.equal(a, b) for a, b in zip(other.parameters(), m2.parameters())), name


def test_config_round_trip_and_refusals():
    for name, d in CONFIGS.items():
        cfg = KebepelConfig.from_json(d, name)
        assert KebepelConfig.from_json(json.loads(json.dumps(cfg.to_json())), name) == cfg
        m, sd = model_and_weights(name, "cpu", torch.float32)
        assert param_count(cfg) == sum(v.numel() for v in sd.values())
        again = KebepelModel(cfg, dtype=torch.float32).load_state_dict_native(sd)
        assert all(torch.equal(a, b) for a, b in zip(again.parameters(), m.parameters()))
    three = KebepelConfig.from_json(CONFIGS["three"])
    assert three.layer_runs() == [(0, 0), (1, None), (0, 1), (1, None), (0, 2), (1, None), (2, None)] and three.num_layers == 7
    assert KebepelConfig.from_json(CONFIGS["wide"]).layer_runs() == [(0, None), (1, None), (2, None)]
    for name in ("kebepel-tiny", "kebepel-1b"):
        assert param_count(DECODERS[name]) > 0
    for layer in ({"type": "mamba2", "mixer": {}}, dict(att(2, 2, 8, 8, 1.0, 0.1), mlp={"kind": "moe"})):
        with pytest.raises(ValueError):
            KebepelConfig.from_json(config([layer], 32))
    for loop in ((0, 2, 2), (1, 1, 2), (-1, 1, 2)):
        with pytest.raises(ValueError):
            KebepelConfig.from_json(config([ff(att(2, 2, 8, 8, 1.0, 0.1), 0)], 32, loop))
    for layer in (att(3, 2, 8, 8, 1.0, 0.1), att(2, 2, 300, 8, 1.0, 0.1), par(2, 2, 8, 8, 1.0, {"dims": 10, "base": 10.0}, 0, 2, 2, 8, 8, 2),
                  par(2, 2, 8, 8, 1.0, {"dims": 8, "base": 10.0}, 0, 3, 2, 8, 8, 2), par(2, 2, 8, 8, 1.0, {"dims": 8, "base": 10.0}, 0, 2, 2, 8, 8, 9)):
        with pytest.raises(ValueError):
            KebepelModel(KebepelConfig.from_json(config([ff(layer, 0)], 32)))


def test_every_layer_run_owns_its_caches():
    """A looped layer's passes have caches and states of their own, and the pool counts them."""
    m, _ = model_and_weights("three", "cpu", torch.float32)
    caches = m.make_caches(4, 16, 2)
    assert [len(c) for c in caches] == [4, 2, 4, 2, 4, 2, 4]
    ptrs = [t.data_ptr() for c in caches for t in c]
    assert len(set(ptrs)) == len(ptrs)
    assert m.cache_block_bytes(16) == sum(t[0].numel() * 4 for c in caches for t in c[:2])
    assert m.state_slot_bytes() == sum(t[0].numel() * 4 for c in caches for t in c[2:])


@pytest.mark.gpu
def test_captured_decode_graph_matches_the_oracle():
    """bf16 on the GPU with sizes the framework's own GEMM kernels tile: decode steps replay a captured
    hipGraph (state slots and block tables in its static buffers); prompt portions, then 60 single tokens
    (past a page's end) for two requests that start at different times, against the float64 forward."""
    m, sd = model_and_weights("mid", "cuda", torch.bfloat16)
    V = m.cfg.vocab_size
    a, b = toks(110, V, 60), toks(95, V, 61)
    wa, wb = O.forward(CONFIGS["mid"], sd, a), O.forward(CONFIGS["mid"], sd, b)
    eng = engine(m, tokens=256, seqs=2)
    ga = [eng.replay_step([("a", a[:33], list(range(33)))]), eng.replay_step([("a", a[33:50], list(range(17)))])]
    gb = []
    for i in range(60):
        entries = [("a", [a[50 + i]], [0])]
        if i == 5:
            entries.append(("b", b[:35], list(range(35))))
        elif i > 5:
            entries.append(("b", [b[35 + i - 6]], [0]))
        lg = eng.replay_step(entries)
        ga.append(lg[:1])
        if i >= 5:
            gb.append(lg[1:])
    captured = [k for k, st in eng.runner.graphs.items() if st.get("graph") is not None]
    assert captured, "no decode bucket was captured"
    for got, want, n in ((ga, wa, 110), (gb, wb, 35 + 54)):
        ok, err = close(torch.cat(got), want[:n], torch.bfloat16)
        assert ok, err


def test_served_through_the_model_manager(tmp_path):
    """The serving stack's model manager builds the preset, wraps it in an engine with state slots and
    prefix caching off, and generates through the server's pipelined step loop; a checkpoint directory
    given for a served name brings its own config."""
    import asyncio

    from safetensors.torch import save_file

    from llm_kubernetes_minikube_sharp4dev_amd.config import Config
    from llm_kubernetes_minikube_sharp4dev_amd.serving.model_manager import ModelManager

    cfg = Config()
    cfg.engine.dtype, cfg.engine.max_num_seqs, cfg.engine.max_model_len = "float32", 4, 256
    mgr = ModelManager(cfg, device="cpu", engine_overrides={"num_blocks": 32})
    h = mgr.generator("kebepel-tiny")
    eng = h.engine
    assert isinstance(eng.model, KebepelModel) and eng.state_pool.num_slots == 4 and not eng.allocator.prefix_caching

    async def both():
        return await asyncio.gather(h.async_engine.generate([5, 6, 7, 8, 9, 10, 11], SamplingParams.greedy(5)),
                                    h.async_engine.generate([3], SamplingParams.greedy(5)))

    try:
        seqs = asyncio.run(both())
    finally:
        h.async_engine.shutdown()
    assert [len(s.output_ids) for s in seqs] == [5, 5]
    assert eng.state_pool.num_free == 4
    sd = {k: v.cpu() for k, v in eng.model.native_state_dict().items()}
    for prompt, sq in zip(([5, 6, 7, 8, 9, 10, 11], [3]), seqs):
        full = prompt + list(sq.output_ids)
        lg = O.forward(eng.model.cfg.to_json(), sd, full[:-1])[len(prompt) - 1:]
        assert [int(x) for x in lg.argmax(-1)] == list(sq.output_ids)
    _, sd_odd = model_and_weights("odd", "cpu", torch.float32)
    d = tmp_path / "ckpt"
    d.mkdir()
    (d / "config.json").write_text(json.dumps(CONFIGS["odd"]))
    save_file({k: v.to(torch.bfloat16) for k, v in sd_odd.items()}, str(d / "model.safetensors"))
    mgr2 = ModelManager(cfg, device="cpu", checkpoints={"kebepel-tiny": str(d)}, engine_overrides={"num_blocks": 32})
    h2 = mgr2.generator("kebepel-tiny")
    try:
        assert isinstance(h2.engine.model, KebepelModel) and h2.engine.model.cfg.hidden == 36 and h2.engine.model.cfg.vocab_size == 61
    finally:
        h2.async_engine.shutdown()


@pytest.mark.gpu
def test_pipelined_generation_on_captured_graphs():
    """The server's step loop on the GPU in bf16: pipelined steps whose decode inputs are gathered on the
    device from the previous step's ids, decode graphs replayed, three requests of different lengths that
    decode across page borders; every token must be the oracle's argmax for its prefix, or within a near tie."""
    import asyncio

    from llm_kubernetes_minikube_sharp4dev_amd.engine.llm_engine import AsyncLLMEngine

    m, sd = model_and_weights("mid", "cuda", torch.bfloat16)
    V = m.cfg.vocab_size
    prompts = [toks(40, V, 70), toks(3, V, 71), toks(18, V, 72)]
    eng = LLMEngine(m, None, block_size=16, max_model_len=256, max_num_seqs=4, num_blocks=24, eos_ids=set(),
                    max_num_batched_tokens=32)
    aeng = AsyncLLMEngine(eng)

    async def run():
        return await asyncio.gather(*[aeng.generate(p, SamplingParams.greedy(16)) for p in prompts])

    try:
        seqs = asyncio.run(run())
    finally:
        aeng.shutdown()
    assert any(st.get("graph") is not None for st in eng.runner.graphs.values())
    assert eng.state_pool.num_free == 4 and eng.allocator.num_free == 24
    for p, sq in zip(prompts, seqs):
        assert len(sq.output_ids) == 16
        full = p + list(sq.output_ids)
        lg = O.forward(CONFIGS["mid"], sd, full[:-1])[len(p) - 1:]
        for i, tid in enumerate(sq.output_ids):
            gap = float(lg[i].max() - lg[i, tid])
            assert gap <= 0.25 * float(lg[i].max() - lg[i].min()), (i, gap)
