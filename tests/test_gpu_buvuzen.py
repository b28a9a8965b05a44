"""Buvuzen models through the engine against the plain implementation (tests/plain/buvuzen_plain.py):
every way of cutting the work, batches, pages used again, keys far back, keys just inside and just
outside a window, sinks and gates that matter, identity experts and groups, layers with the weights of
another one, the first tokens, long decoding, and greedy generation through ``Engine.generate``.
Small configurations of the tests' own, random weights; where random weights would hide a fault,
tokens and projections are made so that one key is found."""
import copy
import json
import os
import subprocess

import numpy as np
import pytest

from buvuzen_util import CFG_A, CFG_B, CFG_C, again, config, layer, moe, random_weights, write_model
from conftest import ROOT
from gpu_util import chunked_steps, make_runner, mixed_steps, run_steps, tail_decode_steps, whole_steps
from plain import buvuzen_plain as P

pytestmark = pytest.mark.gpu

CONFIGS = {"A": (CFG_A, 21), "B": (CFG_B, 22), "C": (CFG_C, 23)}
LENGTHS = {"A": [70, 1, 45, 2, 90, 33, 58], "B": [40, 75, 3, 52, 21], "C": [30, 64, 17, 49, 5]}
PAGE = {"A": 4, "B": 8, "C": 16}
CLOSE_CALL = 0.02      # a gap between two choice scores that bfloat16 rounding of what came before may close


def tokens_of(vocab, n, seed):
    return np.random.default_rng(seed).integers(0, vocab, n).tolist()


class Logits(np.ndarray):
    """Plain logits [T, vocab] that also know which rows' routers made no close call."""
    calm = None


def reference(cfg, w, tokens):
    close = np.zeros(len(tokens))
    z = P.forward(cfg, w, tokens, np.float64, close=close).view(Logits)
    z.calm = close > CLOSE_CALL
    return z


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for name, (cfg, seed) in CONFIGS.items():
        w = random_weights(cfg, seed)
        streams = {f"r{i}": tokens_of(cfg["vocab"], n, 50 + i) for i, n in enumerate(LENGTHS[name])}
        refs = {r: reference(cfg, w, t) for r, t in streams.items()}
        for dtype in ("float32", "bfloat16"):
            folder = write_model(str(tmp_path_factory.mktemp(f"buvuzen{name}_{dtype}")), cfg, w, dtype)
            out[(name, dtype)] = (folder, streams, refs)
    return out


def assert_close(got, want, dtype, what=""):
    """Against the float64 values, relative to the largest logit.  float32 differs by the order of
    its sums alone.  bfloat16 rounds every product's inputs: three rows in four within 5 %, every row
    whose routers made no close call in the plain run within 30 %; a wrong key, a lost sink or a wrong
    expert moves most rows by the logits' own size."""
    calm = getattr(want, "calm", None)
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape, f"{what}: shape {got.shape} vs {want.shape}"
    err = np.abs(got - want).reshape(len(want), -1).max(axis=1) / max(1.0, np.abs(want).max())
    if dtype == "float32":
        ok = err.max() <= 3e-5
    else:
        held = err if calm is None or len(calm) != len(err) else err[calm]
        ok = (held.size == 0 or held.max() <= 0.30) and np.quantile(err, 0.75) <= 0.05
    if not ok:
        raise AssertionError(f"{what}: largest relative error {err.max():.3e} at row {int(np.argmax(err))}, "
                             f"three in four below {np.quantile(err, 0.75):.3e}")


def check(rows, refs, dtype, what):
    assert set(rows) == set(refs)
    for r in refs:
        assert_close(rows[r], refs[r], dtype, f"{what} {r}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_every_split_matches_the_plain_implementation(models, name, dtype):
    folder, streams, refs = models[(name, dtype)]
    runner = make_runner(folder, dtype, page_size=PAGE[name], cache_tokens=128, max_seqs=2, max_batch_tokens=128,
                         max_model_len=128)
    whole = run_steps(runner, streams, whole_steps(streams))
    check(whole, refs, dtype, "whole")
    tail = run_steps(runner, streams, tail_decode_steps(streams, tail=40))
    check(tail, refs, dtype, "last 40 one by one")
    one = run_steps(runner, streams, tail_decode_steps(streams, tail=1000))
    check(one, refs, dtype, "token by token")
    chunk = run_steps(runner, streams, chunked_steps(streams))
    check(chunk, refs, dtype, "portions")
    pairs = run_steps(runner, streams, chunked_steps(streams, sizes=(2,)))
    check(pairs, refs, dtype, "portions of two")
    if dtype == "float32":
        # every sum runs in an order fixed by positions and channels alone: the cuts change nothing
        for r in streams:
            for other in (tail, one, chunk, pairs):
                assert np.array_equal(whole[r], other[r]), r
    assert all(p.free_pages == p.num_pages for p in runner.manager.pools)
    assert runner.manager.slots.free_slots == 2


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C"])
def test_mixed_batches_with_pages_used_again(models, name, dtype):
    folder, streams, refs = models[(name, dtype)]
    page = PAGE[name]
    pages_of = lambda n: -(-n // page)
    room = sum(sorted((pages_of(len(t)) for t in streams.values()), reverse=True)[:3])
    runner = make_runner(folder, dtype, page_size=page, num_pages=room, max_seqs=3, max_batch_tokens=128,
                         max_model_len=128)
    alone = run_steps(runner, streams, whole_steps(streams))
    for seed in (0, 1):
        steps = mixed_steps(streams, seed=seed, max_live=3, room=room, page=page, decode_tail=9)
        assert any(any(n > 1 for _, n in e) and any(n == 1 for _, n in e) for e, _ in steps)
        slots_seen = {}

        def observe(_):
            for r in runner.manager.live():
                slots_seen.setdefault(runner.manager.slot(r), set()).add(r)

        rows = run_steps(runner, streams, steps, observe)
        check(rows, refs, dtype, f"mixed seed {seed}")
        assert any(len(v) >= 2 for v in slots_seen.values()), "no slot was used again"
        if dtype == "float32":
            for r in streams:
                assert np.array_equal(rows[r], alone[r]), f"{r} differs from its run alone"
    assert all(p.free_pages == p.num_pages for p in runner.manager.pools)


def test_layers_are_right_one_by_one(models):
    """The stream after every entry of the order, so that a fault names its layer."""
    cfg, seed = CONFIGS["A"]
    folder = models[("A", "float32")][0]
    w = random_weights(cfg, seed)
    toks = tokens_of(cfg["vocab"], 37, 9)
    want = []
    P.forward(cfg, w, toks, np.float64, layers_out=want)
    runner = make_runner(folder, "float32", page_size=4, cache_tokens=64, max_seqs=1, max_batch_tokens=64, max_model_len=64,
                         use_steplists=False)
    got = []
    for b in runner.model.blocks:
        real = b.forward

        def spied(ctx, h, *a, _real=real, **k):
            out = _real(ctx, h, *a, **k)
            got.append(runner.rt.download(h))
            return out

        b.forward = spied
    run_steps(runner, {"r": toks}, whole_steps({"r": toks}))
    assert len(got) == len(want) == len(cfg["layers"])
    for i, (a, b) in enumerate(zip(got, want)):
        assert np.abs(a - b).max() <= 3e-5 * np.abs(b).max(), f"entry {i}"


# ---------------------------------------------------------------- keys far back, and a window's edge
MARK = 49          # two tokens, MARK and MARK - 1, that stand only where a test puts them


def one_layer(window, sizes):
    if sizes == "small":
        return layer(heads=2, kv_heads=1, dim=48, vdim=20, window=window)
    if sizes == "uneven":
        return layer(heads=4, kv_heads=2, dim=32, vdim=64, window=window)
    return layer(heads=2, kv_heads=1, dim=64, vdim=64, window=window)       # sizes that the matrix-core kernels take


def round16(a):
    from zse_amd.weights.safetensors import bf16_bits_to_f32, f32_to_bf16_bits
    return bf16_bits_to_f32(f32_to_bf16_bits(np.asarray(a, np.float32)))


def a_key_that_is_found(cfg, w, scores=14.0):
    """Random weights spread a softmax over hundreds of keys, and no single key matters.  Here the
    one layer is taken apart so that one does: keys read the first half of the width and values
    the second; queries are the keys' own projection, with gains of 1; and the tokens MARK and MARK - 1
    share the first half of their embeddings and differ in the second.  A query of the one then
    scores a key of the other as high as its own, ``scores``, far above every other key, and what it
    gets from there is another value.  Sinks lie below that score and above most others."""
    w = dict(w)
    mx, m = cfg["layers"][0]["mixer"], "l0.mix."
    H, G, D, half = mx["heads"], mx["kv_heads"], mx["dim"], cfg["width"] // 2
    e = w["embed"].copy()
    e[MARK, :half] = e[MARK - 1, :half]
    w["embed"] = round16(e)
    k, v = w[m + "k"].copy(), w[m + "v"].copy()
    k[:, half:], v[:, :half] = 0.0, 0.0
    w[m + "k"], w[m + "v"] = k, v
    w[m + "q"] = k.reshape(G, D, -1)[[h // (H // G) for h in range(H)]].reshape(H * D, -1).copy()
    w[m + "q.norm"], w[m + "k.norm"] = np.ones(D, np.float32), np.ones(D, np.float32)
    w[m + "sink"] = round16(np.linspace(scores - 8.0, scores - 3.0, H))
    mx["scale"] = scores / D                     # a unit-RMS query times itself is D
    return w


def unmarked(n, seed):
    return np.random.default_rng(seed).integers(0, MARK - 1, n).tolist()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", ["small", "big", "uneven"])
def test_a_key_hundreds_of_tokens_back(tmp_path, sizes, dtype):
    cfg = config([one_layer(None, sizes)], vocab=MARK + 1, width=32)
    w = a_key_that_is_found(cfg, random_weights(cfg, 11))
    n, far = 330, 17
    base = unmarked(n, 21)
    base[far], base[-1] = MARK, MARK - 1
    other = list(base)
    other[far] = 3
    ref, ref_other = P.forward(cfg, w, base), P.forward(cfg, w, other)
    effect = np.abs(ref_other[-1] - ref[-1]).max()
    assert effect > 0.1 * np.abs(ref[-1]).max(), "the key does not matter in this draw"
    folder = write_model(str(tmp_path / f"far_{sizes}_{dtype}"), cfg, w, dtype)
    runner = make_runner(folder, dtype, page_size=16, cache_tokens=2 * 384, max_seqs=2, max_batch_tokens=512, max_model_len=384)
    streams = {"base": base, "other": other}
    for how, steps in (("prompt", whole_steps(streams)), ("decoded", tail_decode_steps(streams, tail=20)),
                       ("portions", chunked_steps(streams, sizes=(64, 3, 31, 2)))):
        rows = run_steps(runner, streams, steps)
        assert_close(rows["base"], ref, dtype, f"{how} base")
        assert_close(rows["other"], ref_other, dtype, f"{how} other")
        assert np.abs(rows["other"][-1] - rows["base"][-1]).max() > 0.6 * effect, how


@pytest.mark.parametrize("sizes", ["small", "big", "uneven"])
@pytest.mark.parametrize("window,page", [(19, 4), (16, 16), (33, 8), (1, 4), (2, 16), (64, 16)])
def test_keys_just_inside_and_just_outside_the_window(tmp_path, sizes, window, page):
    """One layer: the logits at position p depend on the tokens p - window + 1 .. p and on nothing else.
    The key that the last token finds, put just outside the window, must not move a single bit of the
    last row, in a prompt, in portions that end before, at and behind the edge, and token by token;
    just inside it takes about half of the row's weight."""
    cfg = config([one_layer(window, sizes)], vocab=MARK + 1, width=32)
    w = a_key_that_is_found(cfg, random_weights(cfg, 5))
    n = 3 * window + 41
    base = unmarked(n, 3)
    p = n - 1
    base[p] = MARK - 1
    outside, inside = list(base), list(base)
    outside[p - window] = MARK
    if window > 1:
        inside[p - window + 1] = MARK
    refs = {"base": P.forward(cfg, w, base), "outside": P.forward(cfg, w, outside), "inside": P.forward(cfg, w, inside)}
    assert np.abs(refs["outside"][p] - refs["base"][p]).max() < 1e-12
    effect = np.abs(refs["inside"][p] - refs["base"][p]).max()
    assert window == 1 or effect > 0.1 * np.abs(refs["base"][p]).max(), "the key does not matter in this draw"
    streams = {"base": base, "outside": outside, "inside": inside}
    for dtype in ("float32", "bfloat16"):
        folder = write_model(str(tmp_path / f"edge_{dtype}"), cfg, w, dtype)
        runner = make_runner(folder, dtype, page_size=page, cache_tokens=3 * 256, max_seqs=3, max_batch_tokens=256,
                             max_model_len=256)
        edge = p - window
        ways = {"prompt": whole_steps(streams), "decoded": tail_decode_steps(streams, tail=window + 9),
                "portions to the edge": chunked_steps(streams, sizes=(edge, 2, 5)),
                "portions over the edge": chunked_steps(streams, sizes=(edge - 1, 3, 2, 7)),
                "portions behind the edge": chunked_steps(streams, sizes=(edge + 1, 2)),
                "portions of two": chunked_steps(streams, sizes=(2,))}
        for how, steps in ways.items():
            rows = run_steps(runner, streams, steps)
            for r in streams:
                assert_close(rows[r], refs[r], dtype, f"{how} {r}")
            if dtype == "float32":
                assert np.array_equal(rows["outside"][p], rows["base"][p]), f"{how}: a key outside the window was seen"
            if window > 1:
                assert np.abs(rows["inside"][p] - rows["base"][p]).max() > 0.6 * effect, f"{how}: a key inside the window was lost"


def in_every_way(tmp_path, cfg, w, toks, ref, name, dtypes=("float32", "bfloat16")):
    for dtype in dtypes:
        folder = write_model(str(tmp_path / f"{name}_{dtype}"), cfg, w, dtype)
        runner = make_runner(folder, dtype, page_size=8, cache_tokens=128, max_seqs=1, max_batch_tokens=128, max_model_len=128)
        for how, steps in (("whole", whole_steps({"r": toks})), ("decoded", tail_decode_steps({"r": toks}, tail=len(toks) - 9)),
                           ("portions", chunked_steps({"r": toks}))):
            assert_close(run_steps(runner, {"r": toks}, steps)["r"], ref, dtype, f"{name} {dtype} {how}")


# ---------------------------------------------------------------- sinks, gates
@pytest.mark.parametrize("sizes", ["small", "big"])
def test_sinks_and_gates_that_differ_from_head_to_head(tmp_path, sizes):
    """The norm behind the mixer takes out what all heads share: here the sinks and gates of one layer
    take away nearly everything of some heads and nothing of others, so a sink or a gate that is left
    out, scaled or given to another head moves every row."""
    dim = 64 if sizes == "big" else 20
    cfg = config([layer(heads=4, kv_heads=2, dim=dim, vdim=dim, scale=0.5 / dim, window=24)], vocab=80, width=32)
    w = random_weights(cfg, 3)
    w["l0.mix.sink"] = np.array([-6.0, 5.0, 0.0, 8.0], np.float32)
    w["l0.mix.g"] = round16(w["l0.mix.g"] * 3.0)
    toks = tokens_of(80, 70, 4)
    ref = P.forward(cfg, w, toks)
    for name, value in (("l0.mix.sink", np.full(4, -60.0)), ("l0.mix.sink", w["l0.mix.sink"][::-1]),
                        ("l0.mix.sink", w["l0.mix.sink"] * 0.5 / dim), ("l0.mix.g", w["l0.mix.g"] * 0.0)):
        assert np.abs(P.forward(cfg, dict(w, **{name: value.astype(np.float32)}), toks) - ref).max() > 0.2 * np.abs(ref).max()
    in_every_way(tmp_path, cfg, w, toks, ref, sizes)


# ---------------------------------------------------------------- experts
@pytest.mark.parametrize("W,ff", [(64, 32), (36, 20)])
def test_identity_experts_groups_and_the_shared_experts_gate(tmp_path, W, ff):
    """In bfloat16 through the grouped products where the width allows it, else row by row.  Left out, each of the mechanisms moves most rows by much."""
    cfg = config([layer(heads=1, kv_heads=1, dim=16, window=4, mlp=moe(7, 3, ff, 24, identity=2, scale=2.0, groups=(3, 2)))], vocab=90, width=W, scale=1.5)
    w = random_weights(cfg, 12)
    w["l0.mlp.router"] = round16(w["l0.mlp.router"] * 2.0)
    w["l0.mlp.correction"] = round16(np.array([-0.3, 0.1, -0.2, -0.4, 0.0, -0.35, -0.1, 0.05, -0.5]))
    w["l0.mlp.shared.sg"] = round16(w["l0.mlp.shared.sg"] * 4.0)
    toks = tokens_of(90, 100, 6)
    ref = reference(cfg, w, toks)
    moved = lambda c, ww: np.abs(P.forward(c, ww, toks) - ref).max(axis=1) > 0.05 * np.abs(ref).max()
    changed = {}
    for what, path, value in (("scale", ("router", "scale"), 1.0), ("groups", ("router", "groups"), None)):
        c = copy.deepcopy(cfg)
        c["layers"][0]["mlp"][path[0]][path[1]] = value
        changed[what] = moved(c, w).mean()
    changed["correction"] = moved(cfg, dict(w, **{"l0.mlp.correction": np.zeros(9, np.float32)})).mean()
    changed["gate"] = moved(cfg, dict(w, **{"l0.mlp.shared.sg": np.zeros((1, W), np.float32)})).mean()
    ids = []
    real, P.choose = P.choose, lambda *a: (ids.append(real(*a)), ids[-1])[1]
    try:
        P.forward(cfg, w, toks)
    finally:
        P.choose = real
    chosen = np.stack([i for i, _ in ids])
    changed["identity"] = (chosen >= 7).any(axis=1).mean()
    assert all(v > 0.1 for v in changed.values()), changed
    in_every_way(tmp_path, cfg, w, toks, ref, f"moe{W}")


def test_every_choice_an_identity_expert(tmp_path):
    """Corrections that leave no real expert in the race: the feed-forward is the weighted stream and the
    shared expert alone, and a batch has no rows for the experts' products."""
    cfg = config([layer(heads=1, kv_heads=1, dim=16, window=4, mlp=moe(2, 2, 16, 16, identity=2, scale=1.5, groups=(2, 1)))], vocab=50, width=64)
    w = random_weights(cfg, 2)
    w["l0.mlp.correction"] = np.array([-4.0, -4.0, 4.0, 4.0], np.float32)
    toks = tokens_of(50, 90, 1)
    in_every_way(tmp_path, cfg, w, toks, reference(cfg, w, toks), "identity")


# ---------------------------------------------------------------- weights used again
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_runs_of_one_layers_weights_do_not_share_keys(tmp_path, dtype):
    """Three layers on one set of weights: each writes keys of its own, and what a later one computes for
    a token is not what an earlier one did."""
    cfg = config(again([layer(heads=2, kv_heads=1, dim=32, window=11, mlp=moe(3, 2, 16, 16, identity=1, groups=(2, 2)))], 0, 0), vocab=70, width=32)
    w = random_weights(cfg, 14)
    streams = {f"r{i}": tokens_of(70, n, i) for i, n in enumerate([40, 9, 61])}
    refs = {r: reference(cfg, w, t) for r, t in streams.items()}
    folder = write_model(str(tmp_path / f"again_{dtype}"), cfg, w, dtype)
    runner = make_runner(folder, dtype, page_size=4, num_pages=40, max_seqs=3, max_batch_tokens=128, max_model_len=64)
    assert len({c.k.ptr for c in runner.caches}) == 3
    for steps in (whole_steps(streams), tail_decode_steps(streams, tail=50), mixed_steps(streams, seed=3, max_live=3, room=40, page=4)):
        check(run_steps(runner, streams, steps), refs, dtype, "weights used again")


# ---------------------------------------------------------------- both ends of a sequence
@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("A", "bfloat16"), ("B", "bfloat16")])
def test_long_decoding(models, name, dtype):
    cfg, seed = CONFIGS[name]
    folder = models[(name, dtype)][0]
    w = random_weights(cfg, seed)
    toks = tokens_of(cfg["vocab"], 240, 77)
    ref = reference(cfg, w, toks)
    runner = make_runner(folder, dtype, page_size=PAGE[name], cache_tokens=256, max_seqs=1, max_batch_tokens=64, max_model_len=256)
    rows = run_steps(runner, {"r": toks}, tail_decode_steps({"r": toks}, tail=230))
    assert_close(rows["r"], ref, dtype, "230 tokens one by one")


def test_the_first_tokens_of_a_sequence(models):
    """Positions 0 to 3: windows larger than what there is, a sink beside a single key."""
    for name in ("A", "B", "C"):
        cfg, seed = CONFIGS[name]
        folder = models[(name, "float32")][0]
        w = random_weights(cfg, seed)
        runner = make_runner(folder, "float32", page_size=4, cache_tokens=64, max_seqs=2, max_batch_tokens=64, max_model_len=64)
        for n in (1, 2, 3, 4):
            toks = tokens_of(cfg["vocab"], n, 200 + n)
            ref = P.forward(cfg, w, toks, np.float64)
            for steps in (whole_steps({"r": toks}), tail_decode_steps({"r": toks}, tail=10)):
                rows = run_steps(runner, {"r": toks}, steps)
                assert_close(rows["r"], ref, "float32", f"{name}: {n} tokens")


# ---------------------------------------------------------------- the engine's own entry point
def plain_greedy(cfg, w, prompt, n):
    toks = list(prompt)
    for _ in range(n):
        toks.append(int(np.argmax(P.forward(cfg, w, toks, np.float64)[-1])))
    return toks[len(prompt):]


def test_greedy_generation_through_the_engine(models):
    from zse_amd.engine.engine import Engine
    from zse_amd.sampling.sampler import SamplingParams
    cfg, seed = CONFIGS["A"]
    folder = models[("A", "float32")][0]
    w = random_weights(cfg, seed)
    prompts = [tokens_of(cfg["vocab"], n, 300 + n) for n in (5, 23, 1, 40, 12, 31)]
    want = [plain_greedy(cfg, w, p, 12) for p in prompts]
    # four places for six requests, portions of 16: prompts are cut, requests wait for a slot
    with Engine(folder, dtype="float32", block_size=4, num_blocks=64, max_batch_tokens=32, max_batch_seqs=4,
                prefill_chunk_size=16, max_seq_len=128) as eng:
        got = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0))
        assert got == want
        again_ = eng.generate(prompts[:2], SamplingParams(max_tokens=12, temperature=0.0))
        assert again_ == want[:2]
    with Engine(folder, dtype="float32", block_size=4, num_blocks=64, max_batch_tokens=32, max_batch_seqs=4,
                prefill_chunk_size=16, max_seq_len=128, use_graphs=False) as eng:
        assert eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0)) == want


@pytest.mark.parametrize("name", ["A", "B"])
def test_generation_in_bfloat16_through_graphs_does_not_depend_on_the_company(models, name):
    from zse_amd.engine.engine import Engine
    from zse_amd.sampling.sampler import SamplingParams
    cfg, _ = CONFIGS[name]
    folder = models[(name, "bfloat16")][0]
    prompts = [tokens_of(cfg["vocab"], n, 400 + n) for n in (9, 30, 17)]
    sp = SamplingParams(max_tokens=10, temperature=0.0)
    with Engine(folder, dtype="bfloat16", block_size=8, num_blocks=64, max_batch_tokens=64, max_batch_seqs=4,
                prefill_chunk_size=64, max_seq_len=128) as eng:
        together = eng.generate(prompts, sp)
        alone = [eng.generate([p], sp)[0] for p in prompts]
        assert eng.runner.graph_runs > 0, "no decode step was replayed from a graph"
    assert together == alone
    with Engine(folder, dtype="bfloat16", block_size=8, num_blocks=64, max_batch_tokens=64, max_batch_seqs=4,
                prefill_chunk_size=64, max_seq_len=128, use_graphs=False) as eng:
        assert eng.generate(prompts, sp) == together


def test_the_trace_program_serves_the_design(models, tmp_path):
    cfg, seed = CONFIGS["A"]
    folder, streams, refs = models[("A", "float32")]
    out = tmp_path / "out"
    a, b = streams["r0"], streams["r2"]
    steps = [
        {"step": 0, "entries": [{"id": "a", "tokens": a[:7], "want": [0, 6]}], "end": []},
        {"step": 1, "entries": [{"id": "a", "tokens": a[7:9], "want": []}, {"id": "b", "tokens": b[:40], "want": [39]}], "end": []},
        {"step": 2, "entries": [{"id": "b", "tokens": b[40:41], "want": [0]}, {"id": "a", "tokens": a[9:], "want": [len(a) - 10]}],
         "end": ["a"]},
        {"step": 3, "entries": [{"id": "b", "tokens": b[41:], "want": [len(b) - 42]}], "end": ["b"]},
    ]
    p = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "128"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == [f"done {i}" for i in range(4)]
    V = cfg["vocab"]
    read = lambda i: np.fromfile(str(out / f"{i}.f32"), dtype="<f4").reshape(-1, V)
    assert_close(read(0), refs["r0"][[0, 6]], "float32", "step 0")
    assert_close(read(1), refs["r2"][[39]], "float32", "step 1")
    assert_close(read(2), np.stack([refs["r2"][40], refs["r0"][len(a) - 1]]), "float32", "step 2")
    assert_close(read(3), refs["r2"][[len(b) - 1]], "float32", "step 3")
