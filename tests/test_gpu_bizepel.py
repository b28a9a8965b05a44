"""Bizepel models through the engine against the plain implementation (tests/plain/bizepel_plain.py):
every way of cutting the work, batches, pages and state slots used again, keys far back, keys just
inside and just outside a window and just among and just behind the kept first ones, recurrences
that remember, values lent from layer to layer, the first tokens, long decoding, and greedy
generation through ``Engine.generate``.  Small configurations of the tests' own, random weights;
where random weights would hide a fault, tokens and projections are made so that one key is found."""
import json
import os
import subprocess

import numpy as np
import pytest

from bizepel_util import (CFG_A, CFG_B, CFG_C, attention_layer, config, delta_layer, dense, file_config, moe, random_weights,
                          scan_layer, write_model)
from conftest import ROOT
from gpu_util import chunked_steps, make_runner, mixed_steps, run_steps, tail_decode_steps, whole_steps
from plain import bizepel_plain as P

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
            folder = write_model(str(tmp_path_factory.mktemp(f"bizepel{name}_{dtype}")), file_config(cfg), w, dtype)
            out[(name, dtype)] = (folder, streams, refs)
    return out


def assert_close(got, want, dtype, what=""):
    """Against the float64 values, relative to the largest logit.  float32 differs by the order of
    its sums alone.  bfloat16 rounds every product's inputs, and narrow random models with
    recurrences amplify that: nine rows in ten within 6 %, every row within 30 %; a wrong key, a lost
    state or a wrong expert moves most rows by the logits' own size.  A token whose choice of
    experts was a close call in the plain run may go to another expert in bfloat16; such rows count
    among the nine in ten but are not held to the bound for every row."""
    calm = getattr(want, "calm", None)
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    assert got.shape == want.shape, f"{what}: shape {got.shape} vs {want.shape}"
    err = np.abs(got - want).reshape(len(want), -1).max(axis=1) / max(1.0, np.abs(want).max())
    if dtype == "float32":
        ok = err.max() <= 3e-5
    else:
        held = err if calm is None or len(calm) != len(err) else err[calm]
        ok = (held.size == 0 or held.max() <= 0.30) and np.quantile(err, 0.9) <= 0.06
    if not ok:
        raise AssertionError(f"{what}: largest relative error {err.max():.3e} at row {int(np.argmax(err))}, "
                             f"nine in ten below {np.quantile(err, 0.9):.3e}")


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
def test_mixed_batches_with_pages_and_slots_used_again(models, name, dtype):
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
        assert any(len(v) >= 2 for v in slots_seen.values()), "no state slot was used again"
        if dtype == "float32":
            for r in streams:
                assert np.array_equal(rows[r], alone[r]), f"{r} differs from its run alone"
    assert all(p.free_pages == p.num_pages for p in runner.manager.pools)


# ---------------------------------------------------------------- a key that is found
MARK = 49          # two tokens, MARK and MARK - 1, that stand only where a test puts them


def round16(a):
    from zse_amd.weights.safetensors import bf16_bits_to_f32, f32_to_bf16_bits
    return bf16_bits_to_f32(f32_to_bf16_bits(np.ascontiguousarray(a, np.float32)))


def one_attention(dim, vdim, window, keep, scale=1.0):
    """One attention layer and nothing else that looks back: the layer's convolutions have only their
    last tap.  Random weights spread a softmax over hundreds of keys, and no single key matters.  Here
    the projections are made so that one does: keys read the first half of the width and values
    the second; queries are the keys' own projection (rotated channels emptied, so that distance
    takes nothing off a score); and the tokens MARK and MARK - 1 share the first half of their
    embeddings and differ in the second.  A query of the one then scores a key of the other as high
    as its own, far above every other key, and what it gets from there is another value."""
    H, G, R, W = 2, 1, 4, 32
    cfg = config([attention_layer(heads=H, kv_heads=G, dim=dim, vdim=vdim, rot_dims=R, base=30.0, scale=scale, window=window,
                                  keep=keep, conv=3, v_mix=False)], vocab=MARK + 1, width=W, taps=2, side=None, logit_scale=1.0)
    w = random_weights(cfg, 5)
    half, m = W // 2, "l0.mix."
    tidy = lambda v: (v - v.mean()) / np.sqrt(((v - v.mean()) ** 2).mean())
    e = w["embed"].copy()
    e[MARK, :half] = e[MARK - 1, :half] = tidy(e[MARK, :half])
    e[MARK, half:] = tidy(e[MARK, half:])
    e[MARK - 1, half:] = -e[MARK, half:]
    w["embed"] = round16(e)
    for n in ("embed.norm", "l0.norm1", "l0.ls1", m + "q.norm", m + "k.norm"):
        w[n] = np.ones_like(w[n])
    w["l0.canon1"] = np.zeros_like(w["l0.canon1"])
    for r in ("q", "k", "v"):
        w[f"{m}{r}.b"] = np.zeros_like(w[f"{m}{r}.b"])
        w[f"{m}{r}.conv"] = np.zeros_like(w[f"{m}{r}.conv"])
        w[f"{m}{r}.conv"][:, -1] = 1.0
    k, v = w[m + "k"].copy(), w[m + "v"].copy()
    k[:, half:], v[:, :half] = 0.0, 0.0
    q = np.tile(k.reshape(G, dim, W), (H // G, 1, 1))
    q[:, :R] = 0.0
    w[m + "k"], w[m + "v"], w[m + "q"], w[m + "o"] = k, v, q.reshape(H * dim, W), round16(3.0 * w[m + "o"])
    return cfg, w


def unmarked(n, seed):
    return np.random.default_rng(seed).integers(0, MARK - 1, n).tolist()


# head shapes: (24, 20) runs on the plain attention kernel in either type, the others on the
# matrix-core kernels in bfloat16
SHAPES = [(24, 20), (32, 32), (32, 16), (32, 64)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,vdim", SHAPES)
def test_a_key_hundreds_of_tokens_back(tmp_path, dim, vdim, dtype):
    cfg, w = one_attention(dim, vdim, None, 0)
    n = 390
    base = unmarked(n, 21)
    base[-1] = MARK
    other = list(base)
    other[41] = MARK - 1
    streams = {"base": base, "other": other}
    refs = {r: P.forward(cfg, w, t, np.float64) for r, t in streams.items()}
    size = np.abs(refs["base"][-1]).max()
    assert np.abs(refs["other"][-1] - refs["base"][-1]).max() > 0.1 * size
    folder = write_model(str(tmp_path / "far"), file_config(cfg), w, dtype)
    runner = make_runner(folder, dtype, page_size=16, cache_tokens=800, max_seqs=2, max_batch_tokens=512, max_model_len=400)
    for how, steps in (("prompt", whole_steps(streams)), ("decoded", tail_decode_steps(streams, tail=20)),
                       ("portions", chunked_steps(streams, sizes=(64, 3, 31, 2)))):
        rows = run_steps(runner, streams, steps)
        check(rows, refs, dtype, how)
        assert np.abs(rows["other"][-1] - rows["base"][-1]).max() > 0.08 * size, how


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,vdim", SHAPES)
@pytest.mark.parametrize("window,keep,page", [(12, 3, 8), (7, 0, 4), (40, 5, 16), (33, 17, 4), (1, 1, 8), (65, 40, 8)])
def test_keys_just_inside_and_just_outside_the_window_and_the_kept_ones(tmp_path, window, keep, page, dim, vdim, dtype):
    """The marked key at j and queries for it at j + window - 1 (the last that sees it) and j + window
    (which must not move by a bit); and the marked key last among the kept ones or right behind
    them, with a query for it far away.  In prompts, in portions that end at and around the places, and
    token by token."""
    cfg, w = one_attention(dim, vdim, window, keep)
    j = max(keep, 3) + 2 * window + 5
    inside, outside = j + window - 1, j + window
    n = outside + 6
    base = unmarked(n, 3)
    far = n - 2
    base[inside] = base[outside] = base[far] = MARK
    edge, kept, behind = list(base), list(base), list(base)
    edge[j] = MARK - 1 if window > 1 else base[j]
    behind[keep] = MARK - 1
    if keep:
        kept[keep - 1] = MARK - 1
    streams = {"base": base, "edge": edge, "kept": kept, "behind": behind}
    refs = {r: P.forward(cfg, w, t, np.float64) for r, t in streams.items()}
    size = np.abs(refs["base"]).max()
    moved = lambda rows, r, i: np.abs(rows[r][i] - rows["base"][i]).max()
    if window > 1:
        assert moved(refs, "edge", inside) > 0.1 * size
    assert not keep or moved(refs, "kept", far) > 0.1 * size
    folder = write_model(str(tmp_path / "edge"), file_config(cfg), w, dtype)
    runner = make_runner(folder, dtype, page_size=page, cache_tokens=4 * 256, max_seqs=4, max_batch_tokens=1024, max_model_len=256)
    ways = [("prompt", whole_steps(streams)), ("decoded", tail_decode_steps(streams, tail=n - j + 2)),
            ("token by token", tail_decode_steps(streams, tail=1000)),
            ("portions", chunked_steps(streams, sizes=(max(keep, 1), j, 2, max(window - 2, 1), 1, 2))),
            ("portions of two and three", chunked_steps(streams, sizes=(2, 3)))]
    for how, steps in ways:
        rows = run_steps(runner, streams, steps)
        check(rows, refs, dtype, how)
        if window > 1:
            assert moved(rows, "edge", inside) > 0.08 * size, how
        assert np.array_equal(rows["edge"][outside], rows["base"][outside]), f"{how}: a key outside the window was read"
        if keep:
            assert moved(rows, "kept", far) > 0.08 * size, how
        assert np.array_equal(rows["behind"][far], rows["base"][far]), f"{how}: a key behind the kept ones was read"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_windowed_attention_gives_pages_back_and_keeps_the_first(tmp_path, dtype):
    """A pool too small for a request's whole length serves it all the same, and pages that come back
    are handed out again while the kept ones stay."""
    cfg, w = one_attention(32, 16, 16, 6)
    base = unmarked(150, 1)
    base[-1], base[140], base[5] = MARK, MARK, MARK - 1
    ref = P.forward(cfg, w, base, np.float64)
    folder = write_model(str(tmp_path / "small"), file_config(cfg), w, dtype)
    runner = make_runner(folder, dtype, page_size=4, num_pages=16, max_seqs=1, max_batch_tokens=32, max_model_len=160)
    rows = run_steps(runner, {"r": base}, chunked_steps({"r": base}, sizes=(9, 1, 1, 30, 2, 7)))
    assert_close(rows["r"], ref, dtype, "a small pool")
    assert all(p.free_pages == p.num_pages for p in runner.manager.pools)


# ---------------------------------------------------------------- recurrences, convolutions, lent values
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["delta", "delta by heads of 32", "scan"])
def test_the_recurrence_remembers_the_first_tokens(tmp_path, kind, dtype):
    """Decays close to one and little removed: what the recurrence took in at the start still shows two
    hundred tokens later, through a state carried over portions and single tokens."""
    layer = scan_layer(24, 8, 4, 3) if kind == "scan" else delta_layer(2, 32, 4) if "32" in kind else delta_layer(3, 12, 4)
    cfg = config([layer], vocab=50, width=32, taps=2, side=None)
    w = random_weights(cfg, 41)
    if kind == "scan":
        w["l0.mix.A_log"][:] = -5.0
    else:
        w["l0.mix.w0"][:], w["l0.mix.w2"][:], w["l0.mix.a.b"][:] = -9.0, 0.0, -7.0
    n = 200
    base = tokens_of(cfg["vocab"], n, 9)
    other = [(t + 11) % cfg["vocab"] for t in base[:6]] + base[6:]
    streams = {"base": base, "other": other}
    refs = {r: P.forward(cfg, w, t, np.float64) for r, t in streams.items()}
    assert np.abs(refs["other"][-1] - refs["base"][-1]).max() > 0.01 * np.abs(refs["base"][-1]).max(), "the start is forgotten"
    folder = write_model(str(tmp_path / "memory"), file_config(cfg), w, dtype)
    runner = make_runner(folder, dtype, page_size=16, cache_tokens=1024, max_seqs=2, max_batch_tokens=512, max_model_len=512)
    for how, steps in (("prompt", whole_steps(streams)), ("decoded", tail_decode_steps(streams, tail=180)),
                       ("portions", chunked_steps(streams, sizes=(17, 2, 40, 1, 16)))):
        check(run_steps(runner, streams, steps), refs, dtype, how)


def test_decays_and_rates_at_both_ends(tmp_path):
    """Removal rates near one and near zero, decays at both ends of their range (exp(-exp(-1/2)) and 1), keys
    of very different lengths: the 32-bit arithmetic holds."""
    cfg = config([delta_layer(2, 16, 3, mlp=dense(16)), scan_layer(16, 4, 3, 2)], vocab=40, width=32, taps=2, side=4)
    w = random_weights(cfg, 8)
    w["l0.mix.w0"][:] = np.linspace(-14.0, 14.0, 32)
    w["l0.mix.a.b"][:] = np.linspace(9.0, -9.0, 32)
    w["l0.mix.k"] *= np.linspace(0.001, 3.0, 32)[:, None].astype(np.float32)
    w["l1.mix.dt.b"][:] = np.linspace(-9.0, 6.0, 16)
    w["l1.mix.A_log"][:] = np.linspace(-4.0, 2.5, 64).reshape(16, 4)
    toks = tokens_of(40, 60, 4)
    ref = P.forward(cfg, w, toks, np.float64)
    folder = write_model(str(tmp_path / "ends"), file_config(cfg), w, "float32")
    runner = make_runner(folder, "float32", page_size=8, cache_tokens=64, max_seqs=1, max_batch_tokens=64, max_model_len=64)
    for steps in (whole_steps({"r": toks}), tail_decode_steps({"r": toks}, tail=50), chunked_steps({"r": toks}, sizes=(19, 2, 3))):
        assert_close(run_steps(runner, {"r": toks}, steps)["r"], ref, "float32", "both ends")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_portions(tmp_path, dtype):
    """Portions of several hundred tokens (whose recurrences may run in other kernels than short ones'):
    one request alone, unequal ones in one step, later portions that start from carried states."""
    cfg = config([delta_layer(2, 64, 8, mlp=dense(24)), scan_layer(72, 5, 3, 3), delta_layer(1, 24, 4), delta_layer(1, 128, 4)],
                 vocab=70, width=40, taps=3, side=6)
    w = random_weights(cfg, 31)
    w["l0.mix.w0"][:] = np.linspace(-8.0, 8.0, 128)
    lengths = {"a": 263, "b": 128, "c": 129, "d": 5, "e": 191}
    streams = {r: tokens_of(cfg["vocab"], n, 60 + i) for i, (r, n) in enumerate(lengths.items())}
    refs = {r: P.forward(cfg, w, t, np.float64) for r, t in streams.items()}
    folder = write_model(str(tmp_path / "long"), file_config(cfg), w, dtype)
    runner = make_runner(folder, dtype, page_size=8, cache_tokens=1024, max_seqs=3, max_batch_tokens=1024, max_model_len=512)
    check(run_steps(runner, streams, whole_steps(streams)), refs, dtype, "whole")
    together = [([("a", 263), ("b", 128), ("d", 5)], ["a", "b", "d"]), ([("c", 129), ("e", 191)], ["c", "e"])]
    check(run_steps(runner, streams, together), refs, dtype, "unequal requests together")
    check(run_steps(runner, streams, chunked_steps(streams, sizes=(131, 2, 64, 1, 66))), refs, dtype, "long portions one after the other")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_values_lent_to_later_layers(tmp_path, dtype):
    """A large share: the later layers' values are mostly the first mixing layer's.  Without the mixing
    the logits would be others."""
    layers = [scan_layer(16, 4, 2, 2, mlp=dense(16)), attention_layer(2, 2, 16, 16, 8, window=9, keep=2, conv=2, mlp=dense(16)),
              attention_layer(2, 2, 16, 16, 8, window=None, conv=None, v_mix=False), attention_layer(4, 1, 16, 32, 16, window=5, keep=1, conv=3)]
    cfg = config(layers, vocab=60, width=32, taps=2, side=4)
    w = random_weights(cfg, 6)
    w["l3.mix.vmix"] = np.array(0.875, np.float32)
    streams = {f"r{i}": tokens_of(60, n, 90 + i) for i, n in enumerate((50, 33, 7, 41))}
    refs = {r: P.forward(cfg, w, t, np.float64) for r, t in streams.items()}
    none = dict(w)
    none["l3.mix.vmix"] = np.array(0.0, np.float32)
    assert np.abs(P.forward(cfg, none, streams["r0"], np.float64) - refs["r0"]).max() > 0.05 * np.abs(refs["r0"]).max()
    folder = write_model(str(tmp_path / "lent"), file_config(cfg), w, dtype)
    runner = make_runner(folder, dtype, page_size=8, cache_tokens=256, max_seqs=3, max_batch_tokens=128, max_model_len=128)
    for how, steps in (("whole", whole_steps(streams)), ("one by one", tail_decode_steps(streams, tail=100)),
                       ("portions", chunked_steps(streams)), ("mixed", mixed_steps(streams, seed=3, max_live=3))):
        check(run_steps(runner, streams, steps), refs, dtype, how)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_through_every_kind_of_layer(models, dtype):
    cfg, seed = CONFIGS["A"]
    folder = models[("A", dtype)][0]
    w = random_weights(cfg, seed)
    toks = tokens_of(cfg["vocab"], 240, 77)
    ref = reference(cfg, w, toks)
    runner = make_runner(folder, dtype, page_size=4, cache_tokens=256, max_seqs=1, max_batch_tokens=64, max_model_len=256)
    rows = run_steps(runner, {"r": toks}, tail_decode_steps({"r": toks}, tail=230))
    assert_close(rows["r"], ref, dtype, "230 tokens one by one")


def test_the_first_tokens_of_a_sequence(models):
    """Positions 0 to 3: the convolutions read rows before the sequence (zeros, without the projections'
    biases), the recurrences start from zero states."""
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


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_slot_taken_over_starts_from_zero(models, dtype):
    """One slot, requests one after the other: none must see what the one before left in the
    states or in the convolutions' rows."""
    folder, streams, refs = models[("A", dtype)]
    runner = make_runner(folder, dtype, page_size=4, cache_tokens=128, max_seqs=1, max_batch_tokens=128, max_model_len=128)
    for r in ("r0", "r4", "r2", "r0"):
        rows = run_steps(runner, {r: streams[r]}, chunked_steps({r: streams[r]}, sizes=(9, 1, 4)))
        assert_close(rows[r], refs[r], dtype, r)


def test_what_a_layer_keeps_lies_one_behind_the_other(models):
    folder = models[("A", "float32")][0]
    runner = make_runner(folder, "float32", page_size=4, cache_tokens=64, max_seqs=2, max_batch_tokens=64, max_model_len=64)
    spans = [(c.state_offset, c.state_offset + c.state_bytes) for c in runner.caches if c.state_bytes]
    spans += [(at, at + n) for c in runner.caches for at, n in c.extra.values()]
    spans.sort()
    assert len(spans) == 5 + 10                # a mixer's state and two input convolutions in each of five layers
    assert all(a[1] <= b[0] for a, b in zip(spans, spans[1:])) and spans[-1][1] <= runner.slot_bytes


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
    for graphs in (True, False):
        with Engine(folder, dtype="float32", block_size=4, num_blocks=64, max_batch_tokens=32, max_batch_seqs=4,
                    prefill_chunk_size=16, max_seq_len=128, use_graphs=graphs) as eng:
            assert eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0)) == want
            assert eng.generate(prompts[:2], SamplingParams(max_tokens=12, temperature=0.0)) == want[:2]


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


def test_the_engines_pools_hold_the_kept_pages(models):
    """The engine sizes a windowed group's pool by what its requests can hold: window, step and kept tokens."""
    from zse_amd.engine.engine import Engine
    from zse_amd.sampling.sampler import SamplingParams
    cfg, w = one_attention(32, 16, 8, 30)
    import tempfile
    with tempfile.TemporaryDirectory() as d:
        folder = write_model(d, file_config(cfg), w, "float32")
        prompts = [unmarked(n, n) for n in (90, 70, 80)]
        with Engine(folder, dtype="float32", block_size=4, max_batch_tokens=24, max_batch_seqs=3, prefill_chunk_size=8,
                    max_seq_len=120) as eng:
            got = eng.generate(prompts, SamplingParams(max_tokens=6, temperature=0.0))
            assert eng.stats().preemptions == 0
        assert got == [plain_greedy(cfg, w, p, 6) for p in prompts]


def test_the_trace_program_serves_the_design(models, tmp_path):
    cfg, seed = CONFIGS["B"]
    folder, streams, refs = models[("B", "float32")]
    out = tmp_path / "out"
    a, b = streams["r0"], streams["r1"]
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
    assert_close(read(1), refs["r1"][[39]], "float32", "step 1")
    assert_close(read(2), np.stack([refs["r1"][40], refs["r0"][len(a) - 1]]), "float32", "step 2")
    assert_close(read(3), refs["r1"][[len(b) - 1]], "float32", "step 3")
