"""Kefurax through the framework (loader, scheduler, block and state-slot bookkeeping, model runner, kernels on the
GPU / reference ops on the CPU) against the plain float64 model of ``tests/kefurax_oracle.py``.

Every test builds its own small configuration and random weights (stored as bfloat16, so the oracle and the framework
read the same numbers).  The schedules go through ``EngineCore.step_forced`` and generation goes through
``LLM.generate``.  The CPU tests run in float32; the GPU tests run the HIP kernels in float32 (tight tolerance: an index
that is one off shows) and in bfloat16.
"""
import json
import math
import os
import types

import numpy as np
import pytest
import torch

import kefurax_oracle as oracle
from test_tavulix import portions, run_schedule, tokens_for

F64 = torch.float64


# ------------------------------------------------------------------------------------------------ models
def yarn(dims, base, factor=None, original=64, fast=8.0, slow=1.0):
    r = {"dims": dims, "base": base}
    if factor:
        r["scaling"] = {"factor": factor, "original": original, "fast": fast, "slow": slow}
    return r


def dense(ff):
    return {"kind": "dense", "ff": ff} if ff else None


def parallel(left, right, scales=(0.7, 0.4), ff=0):
    """``left``: heads, kv heads, dim, vdim, score scale, rotation; ``right``: heads, q/k heads, dim, vdim, taps."""
    lh, lk, ld, lv, scale, rot = left
    rh, rk, rd, rv, conv = right
    return {"type": "parallel", "mlp": dense(ff),
            "mixer": {"left": {"heads": lh, "kv_heads": lk, "dim": ld, "vdim": lv, "scale": scale, "rot": rot},
                      "right": {"heads": rh, "kv_heads": rk, "dim": rd, "vdim": rv, "conv": conv},
                      "left_scale": scales[0], "right_scale": scales[1]}}


def rglru(width, blocks, conv, ff=0):
    return {"type": "rglru", "mixer": {"width": width, "blocks": blocks, "conv": conv}, "mlp": dense(ff)}


def mamba(inner, state, rank, conv, ff=0):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "dt_rank": rank, "conv": conv}, "mlp": dense(ff)}


def config(layers, width=48, vocab=97, eps=1e-5, scale=None, mult=0.6):
    return {"architecture": "Kefurax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "residual_mult": mult,
            "embedding": {"scale": width ** 0.5 if scale is None else scale}, "layers": layers}


CONFIGS = {
    # every layer of another shape and kind, attention first; value heads sharing q / k heads, query heads sharing key
    # heads; key and value sizes that differ; part of a head rotated and all of it; frequencies on both sides of the ramp
    "varied": config([
        parallel((4, 2, 16, 12, 0.9, yarn(8, 100.0, 4.0)), (4, 2, 8, 12, 4), (0.7, 0.4), 40),
        mamba(36, 6, 5, 3),
        rglru(40, 5, 4, 24),
        parallel((3, 1, 8, 20, 1.3, yarn(8, 1000.0, 2.0, 256, 16.0, 2.0)), (6, 3, 12, 8, 2), (0.3, 1.1)),
        mamba(28, 10, 3, 4, 32)]),
    # values a model can make equal or one: one head, kv heads = heads, one block and as many blocks as channels, one
    # state, rank one, one tap everywhere, scales and multiplier of exactly one, no frequency scaling
    "degenerate": config([
        rglru(8, 8, 1),
        parallel((1, 1, 16, 16, 0.5, yarn(16, 50.0)), (1, 1, 8, 8, 1), (1.0, 1.0)),
        mamba(12, 1, 1, 1, 8),
        rglru(16, 1, 1, 8)], width=32, vocab=50, scale=1.0, mult=1.0),
    # sequences over several pages of 16 tokens
    "paged": config([
        rglru(48, 3, 4),
        parallel((4, 1, 16, 16, 1.1, yarn(12, 500.0, 8.0, 48, 4.0)), (4, 2, 16, 16, 3), (0.5, 0.9), 64),
        mamba(64, 8, 4, 4),
        parallel((2, 2, 32, 24, 0.8, yarn(32, 2000.0, 4.0, 512)), (2, 2, 24, 16, 4), (0.8, 0.6))], width=64),
    # sizes the 16-bit kernels' 16-byte and matrix-core paths take
    "wide": config([
        mamba(128, 16, 8, 4, 128),
        parallel((4, 2, 64, 64, 0.7, yarn(32, 10000.0, 4.0, 128)), (4, 4, 32, 32, 4), (0.6, 0.8), 128),
        rglru(192, 3, 4, 64),
        parallel((8, 2, 32, 32, 1.0, yarn(32, 300.0, 2.0, 96)), (2, 1, 64, 32, 2), (0.9, 0.5)),
        rglru(96, 3, 2),
        mamba(64, 40, 16, 2)], width=128),
    # a width, a vocabulary and sizes that are no multiples of 8 (no 16-byte access fits a 16-bit row)
    "uneven": config([
        mamba(54, 7, 9, 3),
        rglru(42, 3, 3, 30),
        parallel((3, 3, 20, 10, 0.9, yarn(14, 80.0, 3.0)), (3, 1, 10, 14, 3), (0.6, 0.7), 26)], width=100, vocab=211),
    # no layer attends: pages only count positions
    "recurrent": config([mamba(32, 4, 3, 3), rglru(32, 2, 2, 16), mamba(24, 12, 2, 2)], width=40),
}


def random_weights(cfg, seed):
    g = torch.Generator().manual_seed(seed)
    width = cfg["width"]

    def rnd(*shape, lo=-1.0, hi=1.0):
        return lo + (hi - lo) * torch.rand(shape, generator=g)

    def proj(rows, cols, gain=1.0):
        return rnd(rows, cols) * gain * (3.0 / cols) ** 0.5

    w = {"embed": rnd(cfg["vocab"], width), "head": proj(cfg["vocab"], width), "final.norm": rnd(width, lo=0.6, hi=1.4)}
    for i, spec in enumerate(cfg["layers"]):
        m, p, q = spec["mixer"], f"l{i}.", f"l{i}.mix."
        w[p + "norm1"] = rnd(width, lo=0.6, hi=1.4)
        if spec["type"] == "rglru":
            inner, nb = m["width"], m["blocks"]
            n = inner // nb
            for nm in ("y", "x"):
                w[q + nm], w[q + nm + ".b"] = proj(inner, width, 0.5), rnd(inner, lo=-0.5, hi=0.5)
            w[q + "conv"], w[q + "conv.b"] = rnd(inner, m["conv"], lo=-0.7, hi=0.7), rnd(inner, lo=-0.3, hi=0.3)
            for nm in ("ra", "ri"):
                w[q + nm], w[q + nm + ".b"] = proj(nb * n, n, 1.5).view(nb, n, n), rnd(nb, n)
            w[q + "lam"], w[q + "o"] = rnd(inner, lo=-7.0, hi=0.0), proj(width, inner)
        elif spec["type"] == "mamba1":
            inner, n, rank = m["inner"], m["state"], m["dt_rank"]
            w[q + "in"] = proj(2 * inner, width, 0.5)
            w[q + "conv"], w[q + "conv.b"] = rnd(inner, m["conv"], lo=-0.7, hi=0.7), rnd(inner, lo=-0.3, hi=0.3)
            w[q + "x"], w[q + "dt"], w[q + "dt.b"] = proj(rank + 2 * n, inner, 2.0), proj(inner, rank), rnd(inner, lo=-4.0, hi=-0.5)
            w[q + "A_log"], w[q + "D"], w[q + "o"] = rnd(inner, n, lo=-2.0, hi=1.5), rnd(inner, lo=0.3, hi=1.0), proj(width, inner)
        else:
            l, r, q = m["left"], m["right"], q + "left."
            w[q + "q"], w[q + "k"] = proj(l["heads"] * l["dim"], width), proj(l["kv_heads"] * l["dim"], width)
            w[q + "v"], w[q + "g"] = proj(l["kv_heads"] * l["vdim"], width), proj(l["heads"] * l["vdim"], width)
            w[q + "o"] = proj(width, l["heads"] * l["vdim"])
            q = p + "mix.right."
            heads, kv, dim, vdim = r["heads"], r["kv_heads"], r["dim"], r["vdim"]
            for nm, rows in (("q", kv * dim), ("k", kv * dim), ("v", heads * vdim)):
                w[q + nm], w[q + nm + ".conv"] = proj(rows, width), rnd(rows, r["conv"])
            w[q + "b"], w[q + "a"] = proj(heads, width), proj(heads, width)
            w[q + "A_log"], w[q + "dt_bias"], w[q + "norm"] = rnd(heads, lo=-2.5, hi=0.5), rnd(heads), rnd(vdim, lo=0.6, hi=1.4)
            w[q + "g"], w[q + "o"] = proj(heads * vdim, width), proj(width, heads * vdim)
        if spec["mlp"]:
            ff = spec["mlp"]["ff"]
            w[p + "norm2"] = rnd(width, lo=0.6, hi=1.4)
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = proj(ff, width), proj(ff, width), proj(width, ff)
    return {k: v.to(torch.bfloat16) for k, v in w.items()}


_MODELS, _ORACLE = {}, {}


def save_model(d, cfg, w):
    from safetensors.torch import save_file
    save_file({k: v.contiguous() for k, v in w.items()}, str(d / "model.safetensors"))
    (d / "config.json").write_text(json.dumps(cfg))
    return str(d)


def model_dir(name, tmp_path_factory):
    if name not in _MODELS:
        cfg = CONFIGS[name]
        w = random_weights(cfg, sum(map(ord, name)))
        _MODELS[name] = (save_model(tmp_path_factory.mktemp("kefurax_" + name), cfg, w), cfg, w)
    return _MODELS[name]


def oracle_logits(cfg, w, tokens, single=False):
    """The float64 model's logits; ``single``: the same equations evaluated in float32."""
    key = (id(w), tuple(tokens), single)
    if key not in _ORACLE:
        kind = torch.float32 if single else torch.float64
        saved = oracle.F64, oracle.f64
        oracle.F64, oracle.f64 = kind, (lambda t: t.to(kind))
        try:
            _ORACLE[key] = oracle.forward(cfg, w, list(tokens)).double().numpy()
        finally:
            oracle.F64, oracle.f64 = saved
    return _ORACLE[key]


def check(got, cfg, w, reqs, tol):
    """Every row the run produced against the oracle.  Every sublayer's output is normed, so at a position where an
    output nearly cancels, the rounding of its inputs is multiplied up.  How much a row multiplies rounding is measured,
    not guessed: the oracle's own equations evaluated in float32 differ from float64 by some ``e32`` at that row (a few
    1e-6 where nothing cancels), and the row is allowed ``8 e32`` in float32 and ``2^14 e32`` in bfloat16 where that is
    more than the tolerance.  A wrong index or a lost state shows in many rows, none of them of that kind."""
    assert got
    room = 8.0 if tol < 1e-2 else 16384.0
    over = []
    for (rid, p), row in got.items():
        want = oracle_logits(cfg, w, reqs[rid])[p]
        e32 = float(np.abs(oracle_logits(cfg, w, reqs[rid], single=True)[p] - want).max())
        ratio = float(np.abs(row - want).max()) / max(tol, room * e32)
        if ratio > 1.0:
            over.append((ratio, rid, p, e32))
    over.sort(reverse=True)
    # (in bfloat16 a row in fifty may lie outside, by a factor of three at most: the tolerance is a typical worst row)
    assert not over or (tol > 1e-2 and over[0][0] <= 3.0), over[:5]
    assert len(over) <= max(1, len(got) // 50), over[:5]


DEVICES = [pytest.param("cpu", "float32", 1e-4, id="cpu-f32"),
           pytest.param("cuda", "float32", 1e-4, id="gpu-f32", marks=pytest.mark.gpu),
           pytest.param("cuda", "bfloat16", 0.25, id="gpu-bf16", marks=pytest.mark.gpu)]
OP_DEVICES = [pytest.param("cpu", "float32", id="cpu-f32"),
              pytest.param("cuda", "float32", id="gpu-f32", marks=pytest.mark.gpu),
              pytest.param("cuda", "bfloat16", id="gpu-bf16", marks=pytest.mark.gpu)]


def i32(device, *values):
    return torch.tensor(list(values), dtype=torch.int32, device=device)


# ------------------------------------------------------------------------------------------------ schedules
@pytest.mark.parametrize("device,dtype,tol", DEVICES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_and_first_tokens(name, device, dtype, tol, tmp_path_factory, tmp_path):
    path, cfg, w = model_dir(name, tmp_path_factory)
    reqs = {"a": tokens_for(cfg, 70, 1), "b": tokens_for(cfg, 1, 2), "c": tokens_for(cfg, 2, 3)}
    steps = [[(r, t, list(range(len(t)))), {"end": [r]}] for r, t in reqs.items()]
    got = run_schedule(path, steps, dtype, device, max_tokens=128, tmp=tmp_path)
    assert len(got) == 73
    check(got, cfg, w, reqs, tol)


@pytest.mark.parametrize("device,dtype,tol", DEVICES)
@pytest.mark.parametrize("name", ["varied", "uneven"])
def test_residual_stream_after_every_layer(name, device, dtype, tol, tmp_path_factory):
    if dtype != "float32":
        pytest.skip("the per-layer comparison is the float32 one")
    from vllm_distributed_amd.engine.request import Request
    from vllm_distributed_amd.entrypoints import trace_replay
    from vllm_distributed_amd.sampling_params import SamplingParams
    path, cfg, w = model_dir(name, tmp_path_factory)
    toks = tokens_for(cfg, 37, 8)
    args = types.SimpleNamespace(model=path, dtype=dtype, out="", max_tokens=64, max_seqs=2, device=device,
                                 block_size=16, enforce_eager=True)
    core = trace_replay.make_core(args)
    try:
        model = core.executor.driver.worker.model_runner.model
        model.trace_residual = []
        core.add_request(Request("r", toks, SamplingParams(temperature=0.0, max_tokens=None, score_only=True, ignore_eos=True)))
        core.step_forced({"r": len(toks)}, {})
        got = [t.cpu().double() for t in model.trace_residual]
    finally:
        core.shutdown()
    want = []
    oracle.forward(cfg, w, toks, want)
    assert len(got) == len(want) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(got, want)):
        assert (a - b).abs().max().item() <= 5e-5 * max(1.0, b.abs().max().item()), i


@pytest.mark.parametrize("device,dtype,tol", DEVICES)
@pytest.mark.parametrize("name", ["varied", "paged", "wide", "recurrent"])
def test_prefill_then_long_token_by_token_decoding(name, device, dtype, tol, tmp_path_factory, tmp_path):
    """A prompt, then 120 tokens one at a time: recurrent states and convolution tails are carried through 120
    single-row steps, the cache grows over several pages."""
    path, cfg, w = model_dir(name, tmp_path_factory)
    toks = tokens_for(cfg, 150, 4)
    got = run_schedule(path, portions(toks, [30, 1], "r"), dtype, device, max_tokens=192, tmp=tmp_path)
    assert len(got) == 150
    check(got, cfg, w, {"r": toks}, tol)


@pytest.mark.gpu
@pytest.mark.parametrize("dtype,tol", [("float32", 1e-4), ("bfloat16", 0.25)])
@pytest.mark.parametrize("name", ["paged", "wide"])
def test_pages_of_64_tokens(name, dtype, tol, tmp_path_factory, tmp_path):
    """The page size a GPU engine uses by default: two requests in turn, portions that end inside, at and just
    behind a page's border, then single rows across the next border."""
    path, cfg, w = model_dir(name, tmp_path_factory)
    a, b = tokens_for(cfg, 150, 60), tokens_for(cfg, 70, 61)
    steps = [[("a", a[:63], [0, 62])], [("a", a[63:64], [0]), ("b", b[:64], [63])], [("a", a[64:66], [0, 1]), ("b", b[64:65], [0])],
             [("a", a[66:127], [60]), ("b", b[65:70], [4]), {"end": ["b"]}]]
    steps += [[("a", a[i:i + 1], [0])] for i in range(127, 150)]
    steps[-1].append({"end": ["a"]})
    got = run_schedule(path, steps, dtype, "cuda", max_tokens=256, block_size=64, tmp=tmp_path)
    assert len(got) == 2 + 1 + 1 + 2 + 1 + 1 + 1 + 23
    check(got, cfg, w, {"a": a, "b": b}, tol)


@pytest.mark.parametrize("device,dtype,tol", DEVICES)
@pytest.mark.parametrize("sizes", [[2], [3, 2, 7, 1, 16, 17, 2, 2, 31, 5], [1], [64, 2, 1]])
@pytest.mark.parametrize("name", ["varied", "wide"])
def test_portions_of_any_size(name, sizes, device, dtype, tol, tmp_path_factory, tmp_path):
    """Portions cut inside pages, convolution tails and the scans' chunks, down to two tokens and one."""
    path, cfg, w = model_dir(name, tmp_path_factory)
    toks = tokens_for(cfg, 75 if sizes != [1] else 40, 5)
    got = run_schedule(path, portions(toks, sizes, "r"), dtype, device, max_tokens=128, tmp=tmp_path)
    assert len(got) == len(toks)
    check(got, cfg, w, {"r": toks}, tol)


def unequal_requests(cfg):
    """Seven unequal requests for three sequence slots and 10 pages of 16: portions of prompts beside single tokens,
    requests that sit steps out, slots and pages handed on as requests end."""
    reqs = {f"q{i}": tokens_for(cfg, n, 10 + i) for i, n in enumerate([50, 33, 1, 47, 20, 48, 9])}
    at = {r: 0 for r in reqs}
    pattern = {"q0": [7, 1, 1, 2, 30, 1], "q1": [2, 16, 1, 1, 1], "q2": [1], "q3": [17, 1, 15, 1], "q4": [1, 1, 5],
               "q5": [30, 2, 1], "q6": [2, 1]}
    waiting, live, steps, turn = list(reqs), [], [], 0
    while waiting or live:
        while waiting and len(live) < 3 and \
                sum(-(-len(reqs[r]) // 64) * 64 for r in live + waiting[:1]) <= 160:
            live.append(waiting.pop(0))
        step, ended = [], []
        for k, r in enumerate(list(live)):
            if (turn + k) % 4 == 3 and len(live) > 1:
                continue                                    # sits this step out
            sizes = pattern[r]
            n = min(sizes[min(at[r] and (turn % len(sizes)), len(sizes) - 1)], len(reqs[r]) - at[r])
            step.append((r, reqs[r][at[r]:at[r] + n], list(range(n))))
            at[r] += n
            if at[r] == len(reqs[r]):
                ended.append(r)
                live.remove(r)
        if step:
            steps.append(step + ([{"end": ended}] if ended else []))
        turn += 1
    return reqs, steps


@pytest.mark.parametrize("eager", [False, True])
@pytest.mark.parametrize("device,dtype,tol", DEVICES)
@pytest.mark.parametrize("name", ["paged", "wide", "recurrent"])
def test_mixed_batches_reuse_pages_and_slots(name, device, dtype, tol, eager, tmp_path_factory, tmp_path):
    """A new owner of a page or slot must not see what the old one left; every row against the request run alone by the
    oracle."""
    if eager and device == "cpu":
        pytest.skip("graphs exist on the GPU only")
    path, cfg, w = model_dir(name, tmp_path_factory)
    reqs, steps = unequal_requests(cfg)
    got = run_schedule(path, steps, dtype, device, max_tokens=160, max_seqs=3, eager=eager, tmp=tmp_path)
    assert len(got) == sum(len(t) for t in reqs.values())
    check(got, cfg, w, reqs, tol)


@pytest.mark.parametrize("device,dtype,tol", DEVICES)
def test_batch_rows_equal_single_runs(device, dtype, tol, tmp_path_factory, tmp_path):
    """The same rows run alone and inside a batch of unequal neighbours agree far inside the oracle tolerance."""
    path, cfg, w = model_dir("varied", tmp_path_factory)
    a, b, c = tokens_for(cfg, 30, 20), tokens_for(cfg, 11, 21), tokens_for(cfg, 64, 22)
    alone = run_schedule(path, portions(a, [13, 1], "a"), dtype, device, max_tokens=64, tmp=tmp_path / "x")
    steps = [[("c", c[:50], []), ("a", a[:13], list(range(13))), ("b", b[:2], [])]]
    for i in range(13, 30):
        step = [("a", a[i:i + 1], [0])]
        if i < 22:
            step.append(("b", b[i - 11:i - 10], []))
        if i < 27:
            step.insert(0, ("c", c[50 + i - 13:51 + i - 13], []))
        steps.append(step)
    both = run_schedule(path, steps, dtype, device, max_tokens=192, tmp=tmp_path / "y")
    worst = sorted(float(np.abs(alone[("a", p)] - both[("a", p)]).max()) for p in range(30))
    assert worst[-1 if dtype == "float32" else -2] <= (5e-5 if dtype == "float32" else 0.15), worst[-3:]


@pytest.mark.parametrize("device,dtype,tol", DEVICES)
def test_one_far_token_decides_the_logits(device, dtype, tol, tmp_path_factory, tmp_path):
    """A model whose attention can be aimed: the one attention layer's queries read a coordinate of the embedding that only
    one token has, its keys one that only another token has, so the first of them puts nearly all of its weight on the
    second wherever that lies, and its value marks the logits.  The earlier token sits at page borders, at the start and among hundreds of others,
    the later one in the prompt, at a portion's start or decoded alone.  Without rotation (a rotated part of two
    dimensions with a frequency of one in a million) distance plays no role."""
    width, dim = 64, 32
    cfg = config([parallel((2, 1, dim, 16, 0.6, yarn(2, 1e6)), (2, 1, 8, 8, 2), (1.0, 0.3)), rglru(32, 2, 2)], width=width,
                 vocab=80, scale=2.0, mult=1.0)
    w = {k: v.float() for k, v in random_weights(cfg, 5).items()}
    g = torch.Generator().manual_seed(6)
    w["embed"][:, :4] = 0.02 * torch.randn(80, 4, generator=g)
    w["embed"][78, 0], w["embed"][79, 2] = 6.0, 6.0                  # 78: the far token, 79: the one that asks for it
    w["embed"][78, 1] = 4.0                                          # what the far token's value carries
    # those coordinates go into dimension 3 of every head (the other dimensions: little)
    for nm, c in (("q", 2), ("k", 0)):
        m = 0.05 * torch.randn(w["l0.mix.left." + nm].shape, generator=g)
        m[3::dim, c] = 3.0
        w["l0.mix.left." + nm] = m
    v = 0.1 * torch.randn(w["l0.mix.left.v"].shape, generator=g)
    v[:, 1] = torch.linspace(1.0, 3.0, 16)
    w["l0.mix.left.v"] = v
    w = {k: x.to(torch.bfloat16) for k, x in w.items()}
    d = tmp_path_factory.mktemp("kefurax_far")
    path = save_model(d, cfg, w)
    base = [int(t) % 78 for t in tokens_for(cfg, 260, 9)]
    for far, late, cut in ((0, 250, 250), (15, 200, 64), (16, 255, 255), (31, 129, 100), (143, 144, 144), (47, 255, 128)):
        toks = list(base)
        toks[far], toks[late] = 78, 79
        steps = [[("r", toks[:cut], [0])]] if cut == late else [[("r", toks[:cut], [0])], [("r", toks[cut:late], [0])]]
        steps += [[("r", toks[late:late + 1], [0]), {"end": ["r"]}]]
        steps += [[("s", toks[:late + 1], [late]), {"end": ["s"]}]]
        got = run_schedule(path, steps, dtype, device, max_tokens=320, tmp=tmp_path)
        want = oracle_logits(cfg, w, toks[:late + 1])[late]
        blank = list(toks)
        blank[far] = 3
        other = oracle_logits(cfg, w, blank[:late + 1])[late]
        shows = np.abs(want - other).max()
        assert shows > 0.4, (far, late, shows)                       # (the far token's presence does decide)
        for key in (("r", late), ("s", late)):
            assert np.abs(got[key] - want).max() < (1e-4 if dtype == "float32" else 0.15 * shows), (far, late, key)


# --------------------------------------------------------------------------- mechanisms alone, made to show
def _paged(keys, vals, table, nblk, bs, dt):
    n, hkv, dim = keys.shape
    kc = torch.zeros(nblk, hkv, bs, dim, dtype=dt)
    vc = torch.zeros(nblk, hkv, bs // 8, vals.shape[2], 8, dtype=dt)
    for j in range(n):
        b, o = int(table[0, j // bs]), j % bs
        kc[b, :, o] = keys[j].to(dt)
        vc[b, :, o // 8, :, o % 8] = vals[j].to(dt)
    return kc, vc


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("dim,vdim", [(8, 12), (32, 16), (64, 64)])
def test_a_far_key_stands_out_and_the_denominator_has_one_more(device, dtype, dim, vdim):
    """Attention as the layer runs it, over shuffled pages: a query aimed at one key gets ``e^s / (1 + e^s + rest)`` of
    that key's value wherever it lies (first token, page borders, the row itself), nothing from a key behind the row;
    with all scores far below zero the output vanishes instead of averaging the values."""
    from vllm_distributed_amd.models.layers.attention import AttentionMetadata, WindowBiasAttention, set_forward_context
    dt = getattr(torch, dtype)
    n, bs, hq, hkv = 330, 16, 4, 2
    g = torch.Generator().manual_seed(dim)
    nblk = -(-n // bs) + 2
    table = torch.randperm(nblk, generator=g)[:-(-n // bs)].to(torch.int32).view(1, -1)
    with torch.device(device):
        attn = WindowBiasAttention(hq, dim, vdim, hkv, 1.0, 0, distance_bias=False, sink=0.0)
    assert "sink" not in dict(attn.named_parameters()) and attn.sink.abs().max().item() == 0.0
    vals = torch.randn(n, hkv, vdim, generator=g)

    def run(keys, q, pos, rows):
        kc, vc = _paged(keys, vals, table, nblk, bs, dt)
        attn.bind_kv_cache(kc.to(device), vc.to(device))
        qsl = i32(device, 0, rows)
        md = AttentionMetadata(num_decodes=1 if rows == 1 else 0, num_decode_tokens=1 if rows == 1 else 0,
                               num_prefills=0 if rows == 1 else 1, num_prefill_tokens=0 if rows == 1 else rows,
                               slot_mapping=i32(device, *([-1] * rows)), block_table=table.to(device),
                               seq_lens=i32(device, pos + 1), query_start_loc=qsl, max_query_len=rows, max_seq_len=pos + 1,
                               prefill_query_start_loc=qsl, max_prefill_query_len=rows)
        set_forward_context(md, torch.arange(pos - rows + 1, pos + 1, dtype=torch.int32, device=device))
        try:
            return attn.forward_cached(q.to(dt).to(device)).view(rows, hq, vdim)[-1].float().cpu(), vc
        finally:
            set_forward_context(None)
    for pos in (329, 200, 16, 15, 0):
        for target in sorted({0, 1, pos, pos - 1, pos // bs * bs, pos // bs * bs - 1, 16, pos + 1, pos // 2}):
            if target < 0 or target >= n:
                continue
            keys = torch.zeros(n, hkv, dim)
            keys[:, :, 0], keys[:, :, 1] = -40.0, 0.0          # everything else far below
            keys[target, :, 0] = 0.0
            keys[target, :, 1] = 1.0
            for rows in (1, min(9, pos + 1)):
                q = torch.zeros(rows, hq, dim)
                q[-1, :, 0], q[-1, :, 1] = 1.0, torch.tensor([-1.0, 0.0, 1.0, 3.0])
                o, vc = run(keys, q, pos, rows)
                for h in range(hq):
                    s = float(q[-1, h, 1])
                    share = math.exp(s) / (1.0 + math.exp(s)) if target <= pos else 0.0
                    want = share * vc[table[0, target // bs], h // 2, (target % bs) // 8, :, target % 8].float()
                    assert (o[h] - want).abs().max().item() < (1e-5 if dtype == "float32" else 0.02), (pos, target, rows, h)


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("dim,rot", [(16, yarn(8, 100.0, 4.0)), (32, yarn(32, 10000.0, 8.0, 128, 16.0)), (20, yarn(6, 30.0)),
                                     (64, yarn(64, 500.0, 2.0, 2048, 32.0)), (48, yarn(2, 10.0, 16.0, 32, 4.0, 0.5))])
def test_rotation_pairs_neighbours_and_comes_before_the_norm(device, dtype, dim, rot):
    """Rows at far positions against the oracle's rotation and norm; rotating behind the norm, or pairing values half a
    width apart, gives something else; the scale on cos and sin survives the norm where part of a head is not rotated."""
    from vllm_distributed_amd import ops
    from vllm_distributed_amd.models.layers.attention import rotary_frequencies
    dt = getattr(torch, dtype)
    freq, mul = rotary_frequencies(rot["dims"], rot["base"], rot.get("scaling"))
    want_f, want_mul = oracle.rotation(rot)
    assert torch.allclose(freq.double(), torch.tensor(want_f, dtype=F64), rtol=1e-6) and abs(mul - want_mul) < 1e-12
    n, h, kv, vdim = 700, 2, 1, 8
    g = torch.Generator().manual_seed(dim)
    x = torch.randn(n, h * dim + kv * (dim + vdim), generator=g).to(dt)
    want = oracle.unit_rms(oracle.rotate(x[:, :h * dim].double().view(n, h, dim), rot), 1e-5)
    late = oracle.rotate(oracle.unit_rms(x[:, :h * dim].double().view(n, h, dim), 1e-5), rot)
    got = ops.rotate_norm_cache(x.to(device), h, kv, dim, vdim, freq.to(device), mul, True, 1e-5, None, None,
                                torch.arange(n, dtype=torch.int32, device=device), None, None, None).double().cpu()
    half = ops.rotate_norm_cache(x.to(device), h, kv, dim, vdim, freq.to(device), mul, False, 1e-5, None, None,
                                 torch.arange(n, dtype=torch.int32, device=device), None, None, None).double().cpu()
    tol = 2e-4 if dtype == "float32" else 0.03
    assert (got - want).abs().max().item() < tol
    if rot["dims"] > 2:
        assert (half - want).abs().max().item() > 0.3
    if mul > 1.0:
        assert (late - want).abs().max().item() > 2 * tol


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("n_state,channels", [(6, 10), (16, 64), (1, 3), (40, 20)])
def test_the_channel_scan_remembers_far_tokens_and_stale_slots_do_not_show(device, dtype, n_state, channels):
    """Token 0 writes along one state; 300 tokens later a read-out along it returns what the decays left, from a channel
    that keeps and nothing from a channel that forgets.  Portions of many sizes through a slot another sequence left
    full; the whole against the token-by-token float64 recurrence."""
    from vllm_distributed_amd import ops
    dt = getattr(torch, dtype)
    n, far = 301, n_state // 2
    g = torch.Generator().manual_seed(n_state)
    x = 0.05 * torch.randn(n, channels, generator=g)
    bc = 0.02 * torch.randn(n, 2 * n_state, generator=g)
    bc[0, far], bc[n - 1, n_state + far] = 3.0, 2.0
    x[0] = 4.0
    step = torch.full((n, channels), -6.0)                     # softplus(-6) ~ 0.0025: next to no write, slow decay
    step[0] = 3.0
    a_log = torch.full((channels, n_state), math.log(0.4))
    a_log[1] = math.log(60.0)                                  # channel 1 forgets
    bias, skip = torch.zeros(channels), torch.full((channels,), 0.5)
    gate = torch.randn(n, channels, generator=g)
    x, bc, gate = x.to(dt), bc.to(dt), gate.to(dt)
    xd, bd = x.double(), bc.double()
    y, last = oracle.channel_scan(xd, oracle.softplus(step.double()), bd[:, :n_state], bd[:, n_state:],
                                  torch.exp(a_log.double()), skip.double())
    keeps = float(y[n - 1, 0] - 0.5 * xd[n - 1, 0])
    d0 = math.log1p(math.exp(3.0))
    assert abs(keeps - d0 * 4.0 * 3.0 * 2.0 * math.exp(-0.4 * 300 * math.log1p(math.exp(-6.0)))) < 0.6
    assert abs(float(y[n - 1, 1] - 0.5 * xd[n - 1, 1])) < 0.05
    want = y * oracle.silu(gate.double())
    state = torch.full((3, channels, n_state), 7.0, device=device)                 # what an earlier owner left
    out, at, sizes = [], 0, [1, 2, 64, 17, 1, 1, 100, 3, 2, 16]
    for i in range(100):
        m = min(sizes[i % len(sizes)], n - at)
        if m == 0:
            break
        out.append(ops.channel_scan(*(t[at:at + m].to(device) for t in (x, step, bc)), n_state, a_log.to(device),
                                    bias.to(device), skip.to(device), gate[at:at + m].to(device), state, i32(device, 2),
                                    i32(device, 0, m), i32(device, at + m), m).cpu())
        at += m
    got = torch.cat(out).double()
    assert (got - want).abs().max().item() < (1e-5 if dtype == "float32" else 6e-3) * float(want.abs().max())
    assert (state[2].cpu().double() - last).abs().max().item() < 2e-5 * float(last.abs().max())
    assert float(state[0].min()) == 7.0 and float(state[1].max()) == 7.0


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
def test_small_steps_and_slow_decays_keep_their_precision(device, dtype):
    """Step sizes and decays near the ends of their range: softplus of -14 (8e-7), a retention of all but 1e-6 per
    token, and the input's share ``sqrt(1 - a^2)`` of such a decay, to a few units in the last place."""
    from vllm_distributed_amd import ops
    raw = torch.tensor([-14.0, -9.0, -4.0, -1.0, -0.01, 0.0, 0.5, 3.0, 11.0, 19.9, 20.1, 80.0])
    c = raw.numel()
    one = torch.ones(1, c, device=device)
    state = torch.zeros(1, c, 1, device=device)
    ops.channel_scan(one, raw.view(1, c).to(device), torch.ones(1, 2, device=device), 1, torch.zeros(c, 1, device=device),
                     torch.zeros(c, device=device), None, None, state, i32(device, 0), i32(device, 0, 1), i32(device, 1), 1)
    want = torch.log1p(torch.exp(raw.double()))
    assert ((state[0, :, 0].cpu().double() - want) / want).abs().max().item() < 2e-6
    rate = torch.tensor([2e-6, 1e-4, 1e-2, 0.2, 0.4999, 0.5001, 1.0, 3.0, 16.0, 80.0])
    w = rate.numel()
    zero = torch.zeros(1, w, w, device=device)
    state = torch.full((1, w), 2.0, device=device)
    bias = torch.full((w,), 40.0, device=device)               # both gates fully open
    for ctx in (0, 1):
        out = ops.gated_unit_step(torch.ones(1, w, device=device), zero, bias, zero, bias, rate.to(device),
                                  torch.full((1, w), 30.0, device=device), None, state, i32(device, 0), i32(device, 0, 1),
                                  i32(device, 1 + ctx), 1)
        share = torch.sqrt(-torch.expm1(-2 * rate.double()))
        want = share if ctx == 0 else torch.exp(-rate.double()) * share + share       # (the stale 2.0 does not show)
        assert ((state[0].cpu().double() - want) / want).abs().max().item() < 3e-6
        assert ((out[0].cpu().double() - 30.0 * want) / (30.0 * want)).abs().max().item() < 5e-6


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("blocks,n", [(3, 8), (2, 32), (1, 96)])
def test_the_gated_unit_carries_its_state_and_blocks_do_not_mix(device, dtype, blocks, n):
    """A token written 300 tokens back is still in the channels that retain and gone from those that do not; portions of
    many sizes, decoded rows between them, through a slot another sequence left full; a block's gates do not depend on
    the channels of another block."""
    from vllm_distributed_amd import ops
    from vllm_distributed_amd.models.layers.linear_attention import GatedUnitRecurrence
    dt = getattr(torch, dtype)
    width, t = blocks * n, 301
    g = torch.Generator().manual_seed(width)
    w = {"ra": torch.randn(blocks, n, n, generator=g) * n ** -0.5, "ri": torch.randn(blocks, n, n, generator=g) * 0.1 / n,
         "ra.b": torch.randn(blocks, n, generator=g), "ri.b": torch.randn(blocks, n, generator=g),
         "lam": torch.empty(width).uniform_(-12.0, -9.0, generator=g)}
    w["lam"][1::2] = 1.0                                       # the odd channels forget within a few tokens
    w = {k: v.to(torch.bfloat16) for k, v in w.items()}
    u = 0.02 * torch.randn(t, width, generator=g)
    u[0] = 1.0
    y = torch.randn(t, width, generator=g)
    u, y = u.to(dt), y.to(dt)
    yb = torch.randn(width, generator=g)
    ud = u.double()
    r, i = oracle.gated_unit_gates(ud, w, "", blocks)
    states, last = oracle.gated_unit_scan(-8.0 * r * oracle.softplus(oracle.f64(w["lam"])), i * ud)
    want = states * oracle.gelu_tanh(y.double() + yb.double())
    no_first, _ = oracle.gated_unit_scan(-8.0 * r * oracle.softplus(oracle.f64(w["lam"])), i * ud * (torch.arange(t) > 0).view(-1, 1))
    share = (states - no_first)[-1].abs()
    assert share[0::2].median() > 1e-3 and share[1::2].max() < 1e-6
    with torch.device(device):
        unit = GatedUnitRecurrence(width, blocks, 0, dt)
    unit.ra.data.copy_(w["ra"]), unit.ri.data.copy_(w["ri"])
    unit.ra_bias.data.copy_(w["ra.b"].reshape(-1)), unit.ri_bias.data.copy_(w["ri.b"].reshape(-1))
    unit.lam.data.copy_(w["lam"])
    unit.finalize_weights()
    state = torch.full((3, width), 7.0, device=device)
    out, at, sizes = [], 0, [1, 2, 64, 17, 1, 1, 130, 3, 2, 8]
    for k in range(100):
        m = min(sizes[k % len(sizes)], t - at)
        if m == 0:
            break
        out.append(ops.gated_unit_step(u[at:at + m].to(device), unit.ra, unit.ra_bias, unit.ri, unit.ri_bias, unit.rate,
                                       y[at:at + m].to(device), yb.to(device), state, i32(device, 1), i32(device, 0, m),
                                       i32(device, at + m), m).cpu())
        at += m
    got = torch.cat(out).double()
    assert (got - want).abs().max().item() < (5e-6 if dtype == "float32" else 6e-3) * float(want.abs().max())
    assert (state[1].cpu().double() - last).abs().max().item() < 5e-6 * max(1.0, float(last.abs().max()))
    assert float(state[0].min()) == 7.0 and float(state[2].max()) == 7.0
    if blocks > 1:                                             # other channels of another block: the first block's result stays
        u2 = u.clone()
        u2[:, n:] = 3.0
        st = torch.zeros(1, width, device=device)
        both = [ops.gated_unit_step(v.to(device), unit.ra, unit.ra_bias, unit.ri, unit.ri_bias, unit.rate, y.to(device), None,
                                    st, i32(device, 0), i32(device, 0, t), i32(device, t), t)[:, :n].cpu() for v in (u, u2)]
        assert torch.equal(both[0], both[1])


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("heads,groups,dim,vdim", [(4, 2, 8, 12), (2, 2, 32, 32), (3, 1, 20, 6)])
def test_delta_rule_with_one_decay_per_head(device, dtype, heads, groups, dim, vdim):
    """The read-out sees the current token's write; a far token written along a key nobody else touches comes back from
    the head that keeps and not from the one that forgets; portions, a stale slot, neighbouring heads' shared q / k."""
    from vllm_distributed_amd import ops
    dt = getattr(torch, dtype)
    t = 161
    g = torch.Generator().manual_seed(heads * dim)
    q, k = torch.randn(t, groups, dim, generator=g), torch.randn(t, groups, dim, generator=g)
    v = 0.1 * torch.randn(t, heads, vdim, generator=g)
    k[1:, :, 2], k[0], q[-1] = 0.0, 0.0, 0.0
    k[0, :, 2], q[-1, :, 2], v[0] = 5.0, 1.0, 3.0              # token 0 writes along dimension 2, the last one reads it
    beta, dta = torch.full((t, heads), 2.0), torch.full((t, heads), -6.0)
    a_log, dtb = torch.zeros(heads), torch.zeros(heads)
    a_log[1] = math.log(80.0)                                  # head 1 forgets
    x = torch.cat([q.reshape(t, -1), k.reshape(t, -1), v.reshape(t, -1)], 1).to(dt)
    ba = torch.cat([beta, dta], 1).to(dt)
    xd, rep = x.double(), heads // groups
    qd, kd = xd[:, :groups * dim].view(t, groups, dim), xd[:, groups * dim:2 * groups * dim].view(t, groups, dim)
    qd = qd / torch.sqrt((qd * qd).sum(-1, keepdim=True) + 1e-6) * dim ** -0.5
    kd = kd / torch.sqrt((kd * kd).sum(-1, keepdim=True) + 1e-6)
    decay = torch.exp(-torch.exp(a_log.double()) * oracle.softplus(ba[:, heads:].double()))
    want, last = oracle.delta_heads(qd.repeat_interleave(rep, 1), kd.repeat_interleave(rep, 1),
                                    xd[:, 2 * groups * dim:].view(t, heads, vdim), oracle.sigmoid(ba[:, :heads].double()), decay)
    assert float(want[-1, 0].abs().min()) > 1.0 * dim ** -0.5 and float(want[-1, 1].abs().max()) < 0.2
    state = torch.full((2, heads, dim, vdim), 7.0, device=device)
    out, at, sizes = [], 0, [1, 2, 30, 9, 1, 1, 40, 3, 2, 8]
    for i in range(100):
        m = min(sizes[i % len(sizes)], t - at)
        if m == 0:
            break
        out.append(ops.gated_delta_rule(x[at:at + m].to(device), heads, groups, dim, vdim, ba[at:at + m, :heads].to(device),
                                        ba[at:at + m, heads:].to(device), dtb.to(device), a_log.to(device), state,
                                        i32(device, 1), i32(device, 0, m), i32(device, at + m), 1e-6, m).cpu())
        at += m
    got = torch.cat(out).double().view(t, heads, vdim)
    assert (got - want).abs().max().item() < 2e-5 * float(want.abs().max())
    assert (state[1].cpu().double() - last).abs().max().item() < 2e-5 * float(last.abs().max())
    assert float(state[0].min()) == 7.0


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("taps,channels", [(4, 24), (2, 10), (1, 16), (3, 64)])
def test_convolution_with_biases_first_tokens_and_tails(device, dtype, taps, channels):
    """The projection's bias belongs to inputs that exist only: in front of the first token there is nothing, not a bias.
    Portions beside a stranger's rows, through a slot another sequence left full."""
    from vllm_distributed_amd import ops
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(taps)
    t = 40
    x, other = torch.randn(t, channels, generator=g).to(dt), torch.randn(3, channels, generator=g).to(dt)
    w = torch.randn(channels, taps, generator=g).to(dt)
    bias, ib = torch.randn(channels, generator=g), 2.0 + torch.rand(channels, generator=g)
    want = oracle.causal_conv(x.double() + ib.double(), w.double(), bias.double())
    state = torch.full((3, max(taps - 1, 1), channels), 9.0, dtype=dt, device=device)
    out, at = [], 0
    for m in (1, 1, 2, 5, 1, 16, 3, 1, 10):
        rows = torch.cat([x[at:at + m], other])
        pos = torch.cat([torch.arange(at, at + m), torch.arange(3)]).int()
        y = ops.short_conv_act(rows.to(device), channels, w.t().contiguous().to(device), state, i32(device, 2, 0),
                               i32(device, 0, m, m + 3), i32(device, at + m, 3), i32(device, *([0] * m + [1] * 3)),
                               pos.to(device), False, True, bias.to(device), False, ib.to(device))
        out.append(y[:m].cpu())
        at += m
    assert at == t
    got = torch.cat(out).double()
    assert (got - want).abs().max().item() < (1e-5 if dtype == "float32" else 0.12)


@pytest.mark.parametrize("device,dtype", OP_DEVICES)
def test_norms_on_the_way_out(device, dtype):
    """``x += m * norm(y)``: the stream grows by a vector of length ``m * gain`` whatever the size of ``y``, the next
    sublayer reads the stream itself, and only the final norm reads it normed."""
    from vllm_distributed_amd.models.layers.attention import ResidualRMSNorm
    dt = getattr(torch, dtype)
    g = torch.Generator().manual_seed(2)
    width = 72
    with torch.device(device):
        post, final = ResidualRMSNorm(width, 1e-5, dt), ResidualRMSNorm(width, 1e-5, dt)
    gain, fg = torch.rand(width, generator=g) + 0.5, torch.rand(width, generator=g) + 0.5
    post.weight.data.copy_(gain), final.weight.data.copy_(fg)
    x0 = 3 * torch.randn(5, width, generator=g)
    y = (torch.randn(5, width, generator=g) * torch.tensor([1e-4, 0.1, 1.0, 30.0, 300.0]).view(-1, 1)).to(dt)
    want = x0.double() + 0.7 * oracle.unit_rms(y.double(), 1e-5) * gain.double()
    for then in (None, final):
        x = x0.clone().to(device)
        out = post.fold(y.to(device), x, 0.7, then)
        assert (x.cpu().double() - want).abs().max().item() < 3e-6 and x.dtype == torch.float32
        w2 = want if then is None else oracle.unit_rms(want, 1e-5) * fg.double()
        assert out.dtype == dt and (out.cpu().double() - w2).abs().max().item() < (1e-5 if dtype == "float32" else 0.05)
    with pytest.raises(NotImplementedError):
        ResidualRMSNorm(width, 1e-5, dt, offset=1.0).fold(y, x0)


# ------------------------------------------------------------------------------------------- bookkeeping
def test_layers_caches_and_state(tmp_path_factory):
    """Every recurrent part has a convolution tail (model dtype) and an fp32 state; only the left halves of parallel
    layers own cache rows; nothing is windowed, so no page is given back while a request runs."""
    from vllm_distributed_amd.entrypoints import trace_replay
    path, cfg, w = model_dir("varied", tmp_path_factory)
    args = types.SimpleNamespace(model=path, dtype="bfloat16", out="", max_tokens=64, max_seqs=3, device="cpu",
                                 block_size=16, enforce_eager=True)
    core = trace_replay.make_core(args)
    try:
        mr = core.executor.driver.worker.model_runner
        owners = mr.model.attention_layers()
        assert [a.layer_idx for a in owners] == [0, 3]
        assert tuple(owners[0].k_cache.shape[1:]) == (2, 16, 16) and tuple(owners[0].v_cache.shape[1:]) == (2, 2, 12, 8)
        shapes = [tuple(s.shape) for s in mr.state_tensors]
        assert shapes == [(4, 3, 2 * 16 + 48), (4, 4, 8, 12), (4, 2, 36), (4, 36, 6), (4, 3, 40), (4, 40),
                          (4, 1, 2 * 36 + 48), (4, 6, 12, 8), (4, 3, 28), (4, 28, 10)]
        assert [s.dtype for s in mr.state_tensors] == [torch.bfloat16, torch.float32] * 5
        spec = mr.get_kv_cache_spec()
        assert spec.sliding_window is None and spec.bytes_per_token == 2 * (2 * (16 + 12) + 1 * (8 + 20))
        names = [n for n, _ in mr.model.named_parameters()]
        assert len(names) == len(set(names)) and "head.weight" in names
    finally:
        core.shutdown()


def test_config_errors():
    from vllm_distributed_amd.models.kefurax import KefuraxLayer
    f32 = torch.float32
    good = parallel((4, 2, 8, 8, 0.5, yarn(4, 10.0)), (4, 2, 8, 8, 2))
    KefuraxLayer(32, good, 1e-5, 1.0, 0, f32, {})
    bad_mlp = rglru(16, 2, 2, 8)
    bad_mlp["mlp"]["kind"] = "other"
    no_size = mamba(16, 4, 2, 2)
    no_size["mixer"].pop("state")
    for bad in (parallel((4, 3, 8, 8, 0.5, yarn(4, 10.0)), (4, 2, 8, 8, 2)), parallel((4, 2, 8, 8, 0.5, yarn(4, 10.0)), (4, 3, 8, 8, 2)),
                parallel((4, 2, 8, 8, 0.5, yarn(10, 10.0)), (4, 2, 8, 8, 2)), parallel((4, 2, 8, 8, 0.5, yarn(3, 10.0)), (4, 2, 8, 8, 2)),
                rglru(16, 3, 2), dict(good, type="other"), bad_mlp, no_size):
        with pytest.raises(ValueError):
            KefuraxLayer(32, bad, 1e-5, 1.0, 0, f32, {})


def test_a_missing_tensor_is_an_error(tmp_path_factory, tmp_path):
    path, cfg, w = model_dir("degenerate", tmp_path_factory)
    for name in ("l0.mix.lam", "l1.mix.right.o", "l2.mix.x", "l2.norm2"):
        d = tmp_path / name
        d.mkdir()
        save_model(d, cfg, {k: v for k, v in w.items() if k != name})
        with pytest.raises(Exception):
            run_schedule(str(d), [[("r", [1, 2], [1]), {"end": ["r"]}]], "float32", "cpu", max_tokens=64, tmp=tmp_path)


def test_dummy_weights_and_config_keys():
    """Random-weight loading (the benchmark's path): every parameter is filled, the derived keys are there."""
    import tempfile
    from vllm_distributed_amd import LLM, SamplingParams
    from vllm_distributed_amd.config import normalize_hf_config
    from vllm_distributed_amd.models.kefurax import weight_shapes
    cfg = json.loads(json.dumps(CONFIGS["paged"]))
    assert weight_shapes(cfg) == {k: tuple(v.shape) for k, v in random_weights(cfg, 1).items()}
    n = dict(cfg)
    normalize_hf_config(n)
    assert n["hidden_size"] == 64 and n["vocab_size"] == 97 and n["num_hidden_layers"] == 4 and n["num_attention_heads"] == 4
    assert n["num_key_value_heads"] == 1 and n["head_dim"] == 16 and n["architectures"] == ["KefuraxForCausalLM"]
    with tempfile.TemporaryDirectory() as d:
        with open(os.path.join(d, "config.json"), "w") as f:
            json.dump(cfg, f)
        llm = LLM(model=d, device="cpu", dtype="float32", max_model_len=64, max_num_seqs=2, block_size=16,
                  load_format="dummy", enforce_eager=True)
        try:
            out = llm.generate([[1, 2, 3]], SamplingParams(temperature=0.0, max_tokens=4, ignore_eos=True))
        finally:
            llm.shutdown()
        assert len(out[0].outputs[0].token_ids) == 4


def test_sizes_that_tensor_shapes_state_as_well(tmp_path_factory, tmp_path):
    """A config that leaves out what the tensors' shapes say anyway loads and computes the same model."""
    path, cfg, w = model_dir("varied", tmp_path_factory)
    bare = json.loads(json.dumps(cfg))
    for spec in bare["layers"]:
        for key in ("conv", "width", "blocks", "inner", "state", "dt_rank"):
            spec["mixer"].pop(key, None)
        spec["mixer"].get("right", {}).pop("conv", None)
        if spec["mlp"]:
            spec["mlp"].pop("ff")
    d = tmp_path / "bare"
    d.mkdir()
    save_model(d, bare, w)
    toks = tokens_for(cfg, 40, 70)
    got = run_schedule(str(d), portions(toks, [17, 1], "r"), "float32", "cpu", max_tokens=64, tmp=tmp_path)
    check(got, cfg, w, {"r": toks}, 1e-4)


def test_the_trace_runner_as_a_program(tmp_path_factory, tmp_path):
    import subprocess
    import sys
    path, cfg, w = model_dir("degenerate", tmp_path_factory)
    a, b = tokens_for(cfg, 9, 50), tokens_for(cfg, 5, 51)
    lines = [{"step": 0, "entries": [{"id": "a", "tokens": a[:6], "want": [0, 5]}, {"id": "b", "tokens": b[:2], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "b", "tokens": b[2:], "want": []}], "end": ["b"]},
             {"step": 2, "entries": [{"id": "a", "tokens": a[6:], "want": [2]}], "end": ["a"]}]
    exe = os.path.join(os.path.dirname(os.path.dirname(os.path.abspath(__file__))), "bin", "trace_run")
    r = subprocess.run([sys.executable, exe, "--model", path, "--dtype", "float32", "--out", str(tmp_path), "--max-tokens", "128",
                        "--device", "cpu"], input="".join(json.dumps(x) + "\n" for x in lines), text=True,
                       capture_output=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = oracle_logits(cfg, w, a)
    got0 = np.fromfile(tmp_path / "0.f32", dtype="<f4").reshape(2, cfg["vocab"])
    got2 = np.fromfile(tmp_path / "2.f32", dtype="<f4").reshape(1, cfg["vocab"])
    assert np.abs(got0 - want[[0, 5]]).max() < 1e-4 and np.abs(got2 - want[[8]]).max() < 1e-4


# ------------------------------------------------------------------------------------------- generation
@pytest.mark.parametrize("device,dtype", OP_DEVICES)
@pytest.mark.parametrize("name", ["varied", "recurrent"])
def test_greedy_generation_through_the_scheduler(name, device, dtype, tmp_path_factory):
    """``LLM.generate`` on five prompts with two sequence slots and small prefill chunks: the scheduler's own batching,
    chunking and sampling.  Every generated token is the oracle's argmax given the tokens before it (in bfloat16: or
    its logit is within rounding of the oracle's best)."""
    from vllm_distributed_amd import LLM, SamplingParams
    path, cfg, w = model_dir(name, tmp_path_factory)
    prompts = [tokens_for(cfg, n, 40 + n) for n in (3, 30, 1, 17, 45)]
    llm = LLM(model=path, device=device, dtype=dtype, max_model_len=128, max_num_seqs=2, max_num_batched_tokens=16,
              block_size=16, load_format="safetensors", enforce_eager=False)
    try:
        outs = llm.generate(prompts, SamplingParams(temperature=0.0, max_tokens=24, ignore_eos=True))
    finally:
        llm.shutdown()
    for prompt, o in zip(prompts, outs):
        gen = list(o.outputs[0].token_ids)
        assert len(gen) == 24
        logits = oracle.forward(cfg, w, prompt + gen).numpy()
        for i, tok in enumerate(gen):
            row = logits[len(prompt) + i - 1]
            if dtype == "float32":
                assert tok == int(row.argmax()), (len(prompt), i)
            else:
                assert row.max() - row[tok] < 0.2, (len(prompt), i, float(row.max() - row[tok]))
