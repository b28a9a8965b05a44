"""Kernels that Bizepel added or added to, each alone against the plain function of the same mechanism
or a few lines of NumPy: the short convolution over steps of two requests; the kernel between two
sublayers; the embedding's norm; the token gate; gelu as the products' epilogue; lent and mixed
values in the head preparation; the router with corrections and groups; experts without a gate; the
generalized delta rule, walked and by single tokens, with its gates; the attention kernels with kept
first keys and values of another width."""
import numpy as np
import pytest

from plain import bizepel_plain as P

pytestmark = pytest.mark.gpu

_alive = []


@pytest.fixture(autouse=True)
def _operands():
    yield
    _alive.clear()


def lib(dtype="float32"):
    from zse_amd.runtime.device import Runtime
    rt = Runtime.get()
    return rt, rt.kernels(dtype)


def bf16(a):
    from zse_amd.weights.safetensors import bf16_bits_to_f32, f32_to_bf16_bits
    return bf16_bits_to_f32(f32_to_bf16_bits(np.ascontiguousarray(a, np.float32)))


def up(rt, a, dtype="float32"):
    from zse_amd.weights.safetensors import f32_to_bf16_bits
    a = np.ascontiguousarray(a, np.float32)
    _alive.append(rt.upload(f32_to_bf16_bits(a), "bfloat16") if dtype == "bfloat16" else rt.upload(a))
    return _alive[-1]


def i32(rt, a):
    _alive.append(rt.upload(np.ascontiguousarray(a, np.int32)))
    return _alive[-1]


def new(rt, shape, dtype="float32"):
    _alive.append(rt.zeros(shape, dtype))
    return _alive[-1]


STEPS = ([3, 1], [1, 1], [2, 17], [1, 0], [9, 8], [1, 2], [0, 1], [33, 1])       # tokens of requests 0 and 1


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("C,taps,pad,kind", [(40, 4, 8, "bias"), (7, 3, 5, "plain"), (64, 2, 0, "in_bias"), (24, 1, 8, "plain"),
                                             (600, 9, 0, "in_bias"), (33, 5, 2, "bias"), (2056, 4, 0, "plain"), (16, 3, 0, "in_bias")])
def test_short_convolution_over_steps(C, taps, pad, kind, dtype):
    rt, k = lib(dtype)
    rng = np.random.default_rng(C + taps)
    total = [sum(s[r] for s in STEPS) for r in range(2)]
    w = rng.normal(0, 0.7, (C, taps)).astype(np.float32)
    b, ib = rng.normal(size=C).astype(np.float32), rng.normal(size=C).astype(np.float32)
    xs = [rng.normal(size=(n, C)).astype(np.float32) for n in total]
    if dtype == "bfloat16":
        xs = [bf16(x) for x in xs]
    want = []
    for x in xs:
        u = x + (ib if kind == "in_bias" else 0)
        y = P.causal_conv(u, w, np.float64)
        want.append(P.silu(y + b) if kind == "bias" else u + y if kind == "plain" else y)
    offset, slot_words = 8, (12 + (taps - 1) * C + 7) // 4 * 4
    state, done = new(rt, (2, slot_words)), [0, 0]
    for st in STEPS:
        T, padding = sum(st), 2                       # two rows of padding behind the last request
        rows = np.concatenate([xs[r][done[r]:done[r] + st[r]] for r in range(2)])
        wide = np.concatenate([rows, rng.normal(size=(T, pad))], axis=1) if pad else rows
        wide = np.concatenate([wide, np.full((padding, C + pad), np.nan)])
        out = up(rt, np.full((T + padding, C), 7.0), dtype)
        k.zk_conv_rows(up(rt, wide, dtype).ptr, C + pad, up(rt, ib).ptr if kind == "in_bias" else None, up(rt, w).ptr,
                       up(rt, b).ptr if kind == "bias" else None, state.ptr, slot_words, offset, i32(rt, [0, st[0], T]).ptr,
                       i32(rt, [1, 0]).ptr, out.ptr, C, T + padding, 2, max(st), C, taps, 1 if kind == "plain" else 0,
                       1 if kind == "bias" else 0, rt.stream)
        got = rt.download_f32(out)
        assert not got[T:].any(), "padding rows come out as zeros"
        at = 0
        for r in range(2):
            ref = want[r][done[r]:done[r] + st[r]]
            if st[r]:
                tol = 3e-5 if dtype == "float32" else 0.006 * np.abs(ref).max() + 1e-3
                assert np.abs(got[at:at + st[r]] - ref).max() <= tol, (st, r)
            at += st[r]
            done[r] += st[r]
    words = rt.download(state)
    assert not words[:, :offset].any() and not words[:, offset + (taps - 1) * C:].any()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("W,parts,unit,taps", [(64, 0, 0, 0), (64, 3, 0, 4), (50, 1, 1, 3), (2048, 2, 1, 4), (36, 0, 1, 1), (4100, 0, 0, 2), (4100, 2, 1, 4), (300, 0, 1, 2),
                                                (300, 2, 0, 6), (4096, 4, 1, 3)])
def test_the_kernel_between_two_sublayers(W, parts, unit, taps, dtype):
    """h += g y (or g times the unit root mean square of y), the stream as activations, the next layer norm, and in
    a step of single tokens the convolution over the rows that the state holds."""
    rt, k = lib(dtype)
    rng = np.random.default_rng(W + parts)
    R = 5
    act = bf16 if dtype == "bfloat16" else lambda a: a.astype(np.float32)
    h = rng.normal(1.0, 2.0, (R, W)).astype(np.float32)
    planes = rng.normal(size=(max(parts, 1), R, W)).astype(np.float32)
    if parts == 0:
        planes = act(planes)
    g, nw = rng.normal(1, 0.4, W).astype(np.float32), rng.normal(1, 0.3, W).astype(np.float32)
    cw = rng.normal(0, 0.6, (W, max(taps, 1))).astype(np.float32)
    eps, yeps = 1e-4, 1e-3
    slots = [3, 0, 4, 1, 2]
    slot_words, offset = 8 + max(taps - 1, 0) * W + 8, 8
    st = act(rng.normal(size=(R, max(taps - 1, 1), W)))
    words = np.zeros((R, slot_words), np.float32)
    for r in range(R):
        words[slots[r], offset:offset + max(taps - 1, 0) * W] = st[r, :taps - 1].reshape(-1) if taps > 1 else []
    state = up(rt, words)
    positions = np.array([9, 3, 0, -1, 4])              # row 3 is padding
    hd = up(rt, h)
    raw, out = new(rt, (R, W), dtype), new(rt, (R, W), dtype)
    y = up(rt, planes if parts else planes[0], "float32" if parts else dtype)
    k.zk_sublayer_step(hd.ptr, y.ptr, parts, up(rt, g).ptr, unit, yeps, raw.ptr, up(rt, nw).ptr, None, eps, out.ptr,
                       up(rt, cw).ptr if taps else None, taps, state.ptr, slot_words, offset, i32(rt, positions).ptr,
                       i32(rt, range(R)).ptr, i32(rt, slots).ptr, R, W, rt.stream)
    s = planes.astype(np.float64).sum(axis=0)
    if unit:
        s = P.unit_rms(s, yeps, np.float64)
    hn = h + s * g
    n = P.layer_norm(hn, nw, eps, np.float64)
    assert np.abs(rt.download(hd) - hn).max() < 1e-4
    tol = 2e-4 if dtype == "float32" else 0.01 * max(1.0, np.abs(hn).max())
    assert np.abs(rt.download_f32(raw) - hn).max() < tol
    got = rt.download_f32(out)
    if not taps:
        assert np.abs(got - n).max() < tol
        return
    after = rt.download(state)
    for r in range(R):
        mine = after[slots[r], offset:offset + (taps - 1) * W].reshape(taps - 1, W)
        if positions[r] < 0:
            assert not got[r].any() and np.array_equal(mine, st[r, :taps - 1])
            continue
        ref = n[r] + cw[:, taps - 1] * n[r]
        for a in range(taps - 1):
            ref = ref + cw[:, taps - 2 - a] * st[r, a]
        assert np.abs(got[r] - ref).max() < 4 * tol, r
        if taps > 1:
            assert np.abs(mine[0] - n[r]).max() < tol and np.array_equal(mine[1:], st[r, :taps - 2])
    assert not after[:, :offset].any() and not after[:, offset + (taps - 1) * W:].any()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_single_tokens_and_portions_give_the_convolution_the_same_rows(dtype):
    """The norm with the convolution in one launch, and the norm followed by the convolution's own
    kernel, to the bit."""
    rt, k = lib(dtype)
    rng = np.random.default_rng(3)
    W, taps, R = 96, 4, 3
    h, nw, cw = rng.normal(size=(R, W)), rng.normal(1, 0.2, W), rng.normal(0, 0.5, (W, taps))
    st = bf16(rng.normal(size=(R, (taps - 1) * W)))
    one, two = up(rt, st), up(rt, st)
    a, n, b = new(rt, (R, W), dtype), new(rt, (R, W), dtype), new(rt, (R, W), dtype)
    ids, hd = i32(rt, range(R)), up(rt, h)
    k.zk_sublayer_step(hd.ptr, None, 0, None, 0, 0.0, None, up(rt, nw).ptr, None, 1e-5, a.ptr, up(rt, cw).ptr, taps, one.ptr,
                       (taps - 1) * W, 0, ids.ptr, ids.ptr, ids.ptr, R, W, rt.stream)
    k.zk_sublayer_step(hd.ptr, None, 0, None, 0, 0.0, None, up(rt, nw).ptr, None, 1e-5, n.ptr, None, 0, None, 0, 0, ids.ptr,
                       ids.ptr, ids.ptr, R, W, rt.stream)
    k.zk_conv_rows(n.ptr, W, None, up(rt, cw).ptr, None, two.ptr, (taps - 1) * W, 0, i32(rt, range(R + 1)).ptr, ids.ptr, b.ptr, W,
                   R, R, 1, W, taps, 1, 0, rt.stream)
    assert np.array_equal(rt.download(a), rt.download(b))
    assert np.array_equal(rt.download(one), rt.download(two))


def test_the_norm_of_the_stream_and_the_token_gate():
    rt, k = lib()
    rng = np.random.default_rng(5)
    h, w = rng.normal(2.0, 3.0, (4, 77)), rng.normal(1, 0.3, 77)
    hd = up(rt, h)
    k.zk_norm_stream(hd.ptr, up(rt, w).ptr, None, 0.3, 4, 77, rt.stream)
    assert np.abs(rt.download(hd) - P.layer_norm(h, w, 0.3, np.float64)).max() < 1e-5
    for dtype in ("float32", "bfloat16"):
        rt, k = lib(dtype)
        z, table, toks = rng.normal(0, 2, (6, 13)), bf16(rng.normal(size=(20, 60))), [3, 19, 0, 3, 7, 11]
        out = new(rt, (6, 13), dtype)
        k.zk_token_gate(up(rt, z).ptr, up(rt, table, dtype).ptr, i32(rt, toks).ptr, 60, 26, out.ptr, 6, 13, rt.stream)
        want = P.gelu_tanh(z) * table[toks, 26:39]
        assert np.abs(rt.download_f32(out) - want).max() < (1e-5 if dtype == "float32" else 0.02)


@pytest.mark.parametrize("M,K,N", [(3, 96, 80), (16, 96, 80), (40, 256, 144), (200, 96, 80), (700, 1024, 320), (2048, 512, 1024)])
def test_gelu_in_the_products_epilogue(M, K, N):
    rt, k = lib("bfloat16")
    rng = np.random.default_rng(M)
    x, w = bf16(rng.normal(size=(M, K))), bf16(rng.normal(0, 1.5 / np.sqrt(K), (N, K)))
    z = x.astype(np.float64) @ w.T.astype(np.float64)
    out = new(rt, (M, N), "bfloat16")
    k.zk_gemm_bf16(up(rt, x, "bfloat16").ptr, K, up(rt, w, "bfloat16").ptr, out.ptr, N, 0, M, N, K, 8, 0.0, 0, None, 0, None, rt.stream)
    want = np.where(np.abs(z) < 30, P.gelu_exact(z), np.maximum(z, 0))
    assert np.abs(rt.download_f32(out) - want).max() < 0.005 * np.abs(want).max()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_gelu_element_by_element(dtype):
    rt, k = lib(dtype)
    z = bf16(np.random.default_rng(1).normal(0, 2, 1000))
    out = new(rt, (1000,), dtype)
    k.zk_unary_act(up(rt, z, dtype).ptr, out.ptr, 1000, 1, rt.stream)
    assert np.abs(rt.download_f32(out) - P.gelu_exact(z.astype(np.float64))).max() < (1e-6 if dtype == "float32" else 0.02)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("D,E", [(12, 20), (32, 16)])
def test_values_lent_and_mixed(D, E, dtype):
    """One launch lends its values, another takes its share of them before it stores its own; queries
    and keys get their norms and the rotation of neighbouring channels."""
    rt, k = lib(dtype)
    rng = np.random.default_rng(D)
    T, H, G, bs = 5, 2, 2, 4
    ld = (H + G) * D + G * E
    pos = np.array([7, 3, 0, 12, -1])
    slot = np.array([5, 9, 2, 14, -1])
    gq, gk, share = rng.normal(1, 0.3, D), rng.normal(1, 0.3, D), np.array([0.3], np.float32)
    freqs = P.rotary_frequencies(8, 100.0)
    a, b = (bf16(rng.normal(size=(T, ld))) for _ in range(2))
    kc, vc = new(rt, (4, G, bs, D), dtype), new(rt, (4, G, bs, E), dtype)
    lent = new(rt, (T, G * E), dtype)
    for rows, lend, take in ((a, lent.ptr, None), (b, None, lent.ptr)):
        q = up(rt, rows, dtype)
        k.zk_head_prep_values(q.ptr, i32(rt, pos).ptr, i32(rt, slot).ptr, up(rt, gq).ptr, up(rt, gk).ptr, None, 1e-5,
                              up(rt, freqs).ptr, 8, None, 0, kc.ptr, vc.ptr, T, H, G, D, E, bs, 0, None, 1.0, 1, ld, 0,
                              lend, take, up(rt, share).ptr if take else None, rt.stream)
    tol = 2e-5 if dtype == "float32" else 0.02
    va, vb = a[:, (H + G) * D:], b[:, (H + G) * D:]
    assert np.abs(rt.download_f32(lent)[:4] - va[:4]).max() < tol
    mixed = (0.7 * vb + 0.3 * va).reshape(T, G, E)
    prep = lambda x, g: P.rotate_neighbours(P.unit_rms(x, 1e-5, np.float64) * g, pos, freqs, np.float64)
    want_q, want_k = prep(b[:, :H * D].reshape(T, H, D), gq), prep(b[:, H * D:(H + G) * D].reshape(T, G, D), gk)
    got_q = rt.download_f32(q)[:, :H * D].reshape(T, H, D)
    K, V = rt.download_f32(kc), rt.download_f32(vc)
    for t in range(4):
        assert np.abs(got_q[t] - want_q[t]).max() < 3 * tol
        assert np.abs(K[slot[t] // bs, :, slot[t] % bs] - want_k[t]).max() < 3 * tol
        assert np.abs(V[slot[t] // bs, :, slot[t] % bs] - mixed[t]).max() < tol


@pytest.mark.parametrize("E,top,groups,keep", [(8, 4, 4, 3), (6, 2, 3, 2), (5, 5, 5, 5), (130, 16, 13, 4), (1024, 8, 128, 2), (12, 3, 1, 1),
                                               (4, 1, 2, 1), (64, 6, 64, 9)])
def test_the_router_with_corrections_and_groups(E, top, groups, keep):
    rt, k = lib()
    rng = np.random.default_rng(E + top)
    T, ld = 40, E + 3
    z = np.zeros((T, ld), np.float32)
    z[:, :E] = rng.normal(0, 2, (T, E))
    z[3, :E] = 0.5                                     # equal scores: the lower number
    corr = rng.normal(0, 0.5, E).astype(np.float32)
    corr[rng.random(E) < 0.3] -= 2.0                   # choice scores below zero
    for with_corr, normalise, scale in ((True, 1, 1.7), (False, 0, 1.0)):
        ids, wts = i32(rt, np.zeros((T, top))), new(rt, (T, top))
        k.zk_moe_route_groups(up(rt, z).ptr, ld, up(rt, corr).ptr if with_corr else None, ids.ptr, wts.ptr, T, E, top, groups, keep,
                              0, normalise, scale, rt.stream)
        got_i, got_w = rt.download(ids), rt.download(wts)
        for t in range(T):
            s = (1.0 / (1.0 + np.exp(-z[t, :E]))).astype(np.float32)
            c = corr if with_corr else np.zeros(E, np.float32)
            gr = {"count": groups, "keep": keep} if groups > 1 else None
            if P.closeness(s, c, top, gr) < 1e-6 and t != 3:
                continue                               # a tie that rounding decides
            want = P.choose(s, c, top, gr) if t != 3 or not with_corr else None
            if want is None:
                assert len(set(got_i[t])) == top
                continue
            assert got_i[t].tolist() == want.tolist(), t
            w = s[want].astype(np.float64)
            w = (w / (w.sum() + 1e-20) if normalise else w) * scale
            assert np.abs(got_w[t] - w).max() < 1e-6


def test_the_router_survives_numbers_that_are_none():
    """Rows of padding may hold anything: the chosen numbers stay below the number of experts."""
    rt, k = lib()
    z = np.full((3, 8), np.nan, np.float32)
    z[1] = np.inf
    z[2, ::2] = -np.inf
    ids, wts = i32(rt, np.full((3, 3), -7)), new(rt, (3, 3))
    k.zk_moe_route_groups(up(rt, z).ptr, 8, None, ids.ptr, wts.ptr, 3, 8, 3, 4, 2, 0, 1, 1.0, rt.stream)
    got = rt.download(ids)
    assert ((got >= 0) & (got < 8)).all()


@pytest.mark.parametrize("dtype,T", [("float32", 7), ("bfloat16", 5), ("bfloat16", 90)])
def test_experts_without_a_gate(dtype, T):
    """Row by row and (many pairs, bfloat16) grouped on the matrix cores, an expert without tokens among them."""
    rt, k = lib(dtype)
    rng = np.random.default_rng(T)
    E, top, W, F = 6, 3, 64, 40
    x = bf16(rng.normal(size=(T, W)))
    w_up, w_down = bf16(rng.normal(0, 0.2, (E, F, W))), bf16(rng.normal(0, 0.2, (E, W, F)))
    ids = np.stack([rng.permutation([0, 1, 3, 4, 5])[:top] for _ in range(T)]).astype(np.int32)
    wts = rng.random((T, top)).astype(np.float32)
    want = np.zeros((T, W))
    for t in range(T):
        for e, g in zip(ids[t], wts[t]):
            want[t] += g * (w_down[e].astype(np.float64) @ P.relu_squared(w_up[e].astype(np.float64) @ x[t]))
    out, y = new(rt, (T, W)), new(rt, (T * top, F), dtype)
    args = (up(rt, x, dtype).ptr, i32(rt, ids).ptr, up(rt, wts).ptr, up(rt, w_up, dtype).ptr, up(rt, w_down, dtype).ptr)
    if dtype == "bfloat16" and T > 20:
        work, xg, rows = i32(rt, np.zeros(E + 1 + 2 * T * top)), new(rt, (T * top, W), dtype), new(rt, (T * top, W))
        k.zk_moe_experts_grouped_ext(*args, work.ptr, xg.ptr, y.ptr, rows.ptr, out.ptr, T, E, top, W, F, 0.0, 2, 1, rt.stream)
    else:
        k.zk_moe_experts_ext(*args, y.ptr, out.ptr, T, top, W, F, 0.0, 2, 1, rt.stream)
    assert np.abs(rt.download(out) - want).max() < (1e-4 if dtype == "float32" else 0.01) * np.abs(want).max()


# ---------------------------------------------------------------- the generalized delta rule
@pytest.mark.parametrize("T,n,rank", [(5, 24, 3), (19, 300, 16), (1, 256, 64), (40, 512, 40)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_decays_and_removal_rates(T, n, rank, dtype):
    rt, k = lib(dtype)
    rng = np.random.default_rng(n)
    rows = rng.normal(0, 2, (T, n + rank + 2))
    w2, w0, a0 = bf16(rng.normal(0, 1, (n, rank))), rng.normal(size=n), rng.normal(size=n)
    decay, rate = new(rt, (T, n)), new(rt, (T, n))
    k.zk_gdelta_gates(up(rt, rows).ptr, n + rank + 2, n + 1, rank, up(rt, w2, dtype).ptr, up(rt, w0).ptr, up(rt, a0).ptr, decay.ptr,
                      rate.ptr, T, n, rt.stream)
    z = np.tanh(rows[:, n + 1:n + 1 + rank]) @ w2.T.astype(np.float64) + w0
    assert np.abs(rt.download(decay) - np.exp(-np.exp(-0.5) * P.sigmoid(z))).max() < 3e-6
    assert np.abs(rt.download(rate) - P.sigmoid(rows[:, :n] + a0)).max() < 1e-6


DELTA_STEPS = ([150, 37], [70, 1], [1, 129], [1, 1], [1, 1], [6, 2])


@pytest.mark.parametrize("dtype,how", [("float32", "walk"), ("bfloat16", "walk"), ("bfloat16", "chunks"), ("bfloat16", "chunks in passes")])
@pytest.mark.parametrize("H,D", [(3, 12), (2, 32), (2, 64), (1, 100), (2, 128), (1, 200), (1, 256), (9, 32)])
def test_the_generalized_delta_rule_over_steps(H, D, dtype, how):
    """Two requests over six steps, their states carried in slots; in bfloat16 steps of single tokens on the kernel
    of their own where there is one, and portions in chunks (with room for all of them, and for two at a time)."""
    rt, k = lib(dtype)
    if "chunks" in how and not k.zk_gdelta_chunk_floats(D):
        pytest.skip("head size not taken by the chunks")
    rng = np.random.default_rng(H * 1000 + D)
    total = [sum(s[r] for s in DELTA_STEPS) for r in range(2)]
    eps, offset = 1e-5, 16
    slot_words = offset + H * D * D + 8
    gain = rng.normal(1, 0.3, (H, D))
    data, want = [], []
    for n in total:
        r, kk, v, g = (bf16(rng.normal(size=(n, H, D))) for _ in range(4))
        z = rng.normal(-3, 2, (n, H, D))
        z[:, 0] = rng.normal(6, 3, (n, D))               # one head whose decays are about as strong as they can be
        w, a = np.exp(-np.exp(-0.5) * P.sigmoid(z)), P.sigmoid(rng.normal(0, 2, (n, H, D)))
        data.append((r, kk, v, g, w, a))
        o = np.stack([P.general_delta_rule(*(x[:, h].astype(np.float64) for x in (r, kk, v, w, a)), np.float64)
                      for h in range(H)], axis=1)
        want.append(P.unit_rms(o, eps, np.float64) * gain * P.sigmoid(g.astype(np.float64)))
    state, done = new(rt, (2, slot_words)), [0, 0]
    C = H * D
    for st in DELTA_STEPS:
        T = sum(st)
        cut = lambda i: np.concatenate([d[i][done[q]:done[q] + st[q]].reshape(st[q], C) for q, d in enumerate(data)])
        X = up(rt, np.concatenate([cut(i) for i in range(4)], axis=1), dtype)
        out, raw = new(rt, (T, C), dtype), new(rt, (T, C))
        gate = X.ptr + 3 * C * (2 if dtype == "bfloat16" else 4)
        W_, A_ = up(rt, cut(4)), up(rt, cut(5))
        if dtype == "bfloat16" and max(st) == 1 and k.zk_gdelta_token_supports(D):
            k.zk_gdelta_token(X.ptr, 4 * C, C, 2 * C, gate, 4 * C, W_.ptr, A_.ptr, up(rt, gain).ptr, state.ptr, slot_words, offset,
                              i32(rt, [5, 5]).ptr, i32(rt, [0, 1]).ptr, i32(rt, [1, 0]).ptr, out.ptr, T, H, D, eps, rt.stream)
        elif "chunks" in how:
            count = 2 if "passes" in how else -(-max(st) // 32)
            floats = count * 2 * H * k.zk_gdelta_chunk_floats(D)
            work = up(rt, np.full(floats, np.nan))
            k.zk_gdelta_chunked(X.ptr, 4 * C, C, 2 * C, gate, 4 * C, W_.ptr, A_.ptr, up(rt, gain).ptr, state.ptr, slot_words, offset,
                                i32(rt, [0, st[0], T]).ptr, i32(rt, [1, 0]).ptr, i32(rt, np.zeros(T)).ptr, out.ptr, raw.ptr, work.ptr,
                                floats, T, 2, max(st), H, D, eps, rt.stream)
        else:
            k.zk_gdelta(X.ptr, 4 * C, C, 2 * C, gate, 4 * C, W_.ptr, A_.ptr, up(rt, gain).ptr, state.ptr, slot_words, offset,
                        i32(rt, [0, st[0], T]).ptr, i32(rt, [1, 0]).ptr, i32(rt, np.zeros(T)).ptr, out.ptr, raw.ptr, T, 2,
                        max(st), H, D, eps, rt.stream)
        got = rt.download_f32(out).reshape(T, H, D)
        at = 0
        for q in range(2):
            ref = want[q][done[q]:done[q] + st[q]]
            tol = (3e-4 if dtype == "float32" else 0.01) * max(1.0, np.abs(ref).max())
            assert np.abs(got[at:at + st[q]] - ref).max() < tol, (st, q)
            at += st[q]
            done[q] += st[q]
    words = rt.download(state)
    assert not words[:, :offset].any() and not words[:, offset + H * D * D:].any()


# ---------------------------------------------------------------- attention with kept first keys, values of another width
def plain_attention(q, kk, v, pos0, scale, window, keep):
    n, H, _ = q.shape
    G = kk.shape[1]
    out = np.zeros((n, H, v.shape[2]))
    for i in range(n):
        p = pos0 + i
        j = np.arange(p + 1)
        seen = j[(p - j < window) | (j < keep)] if window else j
        for h in range(H):
            s = (kk[seen, h // (H // G)] @ q[i, h]) * scale
            e = np.exp(s - s.max())
            out[i, h] = (e / e.sum()) @ v[seen, h // (H // G)]
    return out


@pytest.mark.parametrize("D,E,H,G,bs,window,keep", [
    (16, 16, 4, 2, 4, 24, 3), (64, 64, 2, 1, 16, 100, 40), (128, 128, 8, 2, 16, 700, 4), (32, 32, 3, 3, 8, 1, 1),
    (128, 64, 4, 2, 16, 40, 4), (64, 32, 4, 1, 16, 33, 70), (32, 64, 4, 2, 8, 200, 5), (16, 32, 2, 2, 4, 31, 33), (256, 128, 2, 2, 32, 333, 300),
    (128, 256, 2, 1, 16, 64, 8), (64, 128, 34, 1, 16, 90, 7), (32, 16, 20, 1, 8, 50, 6), (64, 128, 2, 2, 8, 0, 0)])
@pytest.mark.parametrize("dtype,mode", [("bfloat16", 0), ("bfloat16", 1), ("bfloat16", 4), ("bfloat16", 5), ("float32", 0)])
def test_attention_with_kept_first_keys(D, E, H, G, bs, window, keep, dtype, mode):
    """Three requests of one step: a long portion from position 0, a portion behind a cached context
    and a single token far into its context.  Pages between the kept keys and the window hold what
    is not a number and their table entries name no page, as after they were given back.  ``mode``: which of the portions'
    kernels (0: chosen by the sizes)."""
    rt, k = lib(dtype)
    tuned = dtype == "bfloat16"
    if tuned and not k.zk_attention_bf16_supports_values(H, G, D, E, bs):
        if mode:
            pytest.skip("head shape not taken by the matrix-core kernel")
        tuned = False
    rng = np.random.default_rng(D + E + window)
    ctx, fresh = [420, 333, 1101], [420, 70, 1]
    R, T, max_ctx = 3, sum(fresh), 1280
    blocks = -(-max_ctx // bs)
    pages = R * blocks + 1
    kc = np.zeros((pages, G, bs, D), np.float32)
    vc = np.zeros((pages, G, E, bs) if tuned else (pages, G, bs, E), np.float32)
    table = (np.arange(R * blocks, dtype=np.int32).reshape(R, blocks)[:, ::-1] + 1).copy()     # pages in falling order
    keys, vals = [], []
    for r in range(R):
        kk = rng.normal(size=(ctx[r], G, D))
        kk = bf16(kk * np.sqrt(D) / np.linalg.norm(kk, axis=-1, keepdims=True))
        vv = bf16(rng.normal(size=(ctx[r], G, E)))
        keys.append(kk)
        vals.append(vv)
        for p in range(ctx[r]):
            pg = table[r, p // bs]
            kc[pg, :, p % bs] = kk[p]
            if tuned:
                vc[pg, :, :, p % bs] = vv[p]
            else:
                vc[pg, :, p % bs] = vv[p]
        first = ctx[r] - fresh[r] - window + 1 if window else 0       # the oldest key that a window of the step shows
        for j in range(blocks):
            gone = window and (j + 1) * bs - 1 < first and j * bs >= keep
            if gone or j * bs >= ctx[r]:
                if gone:
                    kc[table[r, j]], vc[table[r, j]] = np.nan, np.nan
                table[r, j] = -1
    q = rng.normal(size=(T, H, D))
    q = bf16(q * np.sqrt(D) / np.linalg.norm(q, axis=-1, keepdims=True))
    scale = 6.0 / D
    q_start = np.concatenate([[0], np.cumsum(fresh)]).astype(np.int32)
    want = np.concatenate([plain_attention(q[q_start[r]:q_start[r + 1]].astype(np.float64), keys[r].astype(np.float64),
                                           vals[r].astype(np.float64), ctx[r] - fresh[r], scale, window, keep) for r in range(R)])
    out = new(rt, (T, H * E), dtype)
    tab = i32(rt, table)
    if tuned:
        need = (int(k.zk_attention_bf16_workspace(R, H, E, max_ctx)) + 255) // 256 * 256
        need += int(k.zk_attention_bf16_portion_workspace(2 * (448 + 128), H, G, E))
        ws = new(rt, (need // 4 + 16,))
        before = k.zk_attention_bf16_portion_kernel(mode)
        try:
            k.zk_attention_bf16_sized(up(rt, q.reshape(T, H * D), dtype).ptr, H * D, up(rt, kc, dtype).ptr, up(rt, vc, dtype).ptr,
                                      tab.ptr, blocks, i32(rt, q_start).ptr, i32(rt, ctx).ptr, out.ptr, R, 2, 448, max_ctx, H, G, D,
                                      bs, scale, 0.0, window, 64, ws.ptr, ws.nbytes, 0, 0, 1, 0, E, keep, rt.stream)
        finally:
            k.zk_attention_bf16_portion_kernel(before)
    else:
        positions = np.concatenate([np.arange(ctx[r] - fresh[r], ctx[r]) for r in range(R)])
        owner = np.concatenate([np.full(fresh[r], r) for r in range(R)])
        k.zk_attention_plain_kept(up(rt, q.reshape(T, H * D), dtype).ptr, H * D, up(rt, kc, dtype).ptr, up(rt, vc, dtype).ptr,
                                  tab.ptr, blocks, i32(rt, owner).ptr, i32(rt, positions).ptr, out.ptr, T, H, G, D, E, bs, scale, 0.0,
                                  window, 0, None, 0, None, 0, 0, 0, keep, rt.stream)
    got = rt.download_f32(out).reshape(T, H, E)
    err = np.abs(got - want).max(axis=(1, 2))
    assert err.max() < (1e-5 if dtype == "float32" else 0.02), (int(np.argmax(err)), float(err.max()))
