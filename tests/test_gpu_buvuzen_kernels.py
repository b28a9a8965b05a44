"""Kernels that Buvuzen added or added to, each alone against the plain function of the same mechanism or
a few lines of NumPy: the attention kernels with a sink and a gate per head, by every way a portion or
a decoded token can take; the router with softmax scores and groups judged by their best; the experts
with identity experts among the choices, row by row and grouped; the kernel that joins a result and
hands on the stream itself; a product into wider rows; the factor in a norm's gain."""
import numpy as np
import pytest

from plain import buvuzen_plain as P

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


# ---------------------------------------------------------------- attention
def plain_attention(q, kk, v, pos0, scale, window, sinks, gate):
    n, H, _ = q.shape
    G = kk.shape[1]
    out = np.zeros((n, H, v.shape[2]))
    mask = P.visible(len(kk), window)[pos0:pos0 + n]
    for h in range(H):
        g = h // (H // G)
        p = P.sink_softmax((q[:, h] @ kk[:, g].T) * scale, mask, sinks[h] if sinks is not None else -np.inf)
        out[:, h] = (p @ v[:, g]) * (P.sigmoid(gate[:, h:h + 1]) if gate is not None else 1.0)
    return out


@pytest.mark.parametrize("D,E,H,G,bs,window,use", [
    (16, 16, 4, 2, 4, 24, "both"), (64, 64, 2, 1, 16, 100, "both"), (128, 128, 8, 2, 16, 700, "both"), (32, 32, 3, 3, 8, 1, "both"),
    (128, 64, 4, 2, 16, 40, "both"), (32, 64, 4, 2, 8, 200, "sinks"), (256, 128, 2, 2, 32, 333, "both"), (128, 256, 2, 1, 16, 64, "gate"),
    (64, 128, 34, 1, 16, 90, "both"), (32, 16, 20, 1, 8, 50, "both"), (64, 64, 6, 6, 16, 0, "both"), (256, 256, 4, 2, 16, 0, "both")])
@pytest.mark.parametrize("dtype,mode", [("bfloat16", 0), ("bfloat16", 1), ("bfloat16", 4), ("bfloat16", 5), ("bfloat16", 8), ("float32", 0)])
def test_attention_with_sinks_and_gates(D, E, H, G, bs, window, use, dtype, mode):
    """Three requests of one step: a long portion from position 0, a portion behind a cached context
    and a single token far into its context.  Sinks from far below to far above the scores; the gate's
    numbers lie behind the queries in rows of their own distance.  Pages before the window hold what is not a
    number and their table entries name no page.  ``mode``: which of the portions' kernels (0: chosen by
    the sizes)."""
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
    unit = lambda a: bf16(a * np.sqrt(D) / np.linalg.norm(a, axis=-1, keepdims=True))
    keys, vals = [], []
    for r in range(R):
        kk, vv = unit(rng.normal(size=(ctx[r], G, D))), bf16(rng.normal(size=(ctx[r], G, E)))
        keys.append(kk.astype(np.float64))
        vals.append(vv.astype(np.float64))
        for p in range(ctx[r]):
            pg = table[r, p // bs]
            kc[pg, :, p % bs] = kk[p]
            if tuned:
                vc[pg, :, :, p % bs] = vv[p]
            else:
                vc[pg, :, p % bs] = vv[p]
        first = ctx[r] - fresh[r] - window + 1 if window else 0       # the oldest key that a window of the step shows
        for j in range(blocks):
            gone = window and (j + 1) * bs - 1 < first
            if gone or j * bs >= ctx[r]:
                if gone:
                    kc[table[r, j]], vc[table[r, j]] = np.nan, np.nan
                table[r, j] = -1
    ld = H * D + (H + 15) // 8 * 8
    rows = np.zeros((T, ld), np.float32)
    q = unit(rng.normal(size=(T, H, D)))
    gate = bf16(rng.normal(0, 2, (T, H)))
    rows[:, :H * D], rows[:, H * D:H * D + H] = q.reshape(T, H * D), gate
    scale = 6.0 / D
    sinks = bf16(np.concatenate([[-30.0, 9.0, 2.0], rng.normal(1, 3, H)])[:H])
    use_s, use_g = use in ("both", "sinks"), use in ("both", "gate")
    q_start = np.concatenate([[0], np.cumsum(fresh)]).astype(np.int32)
    want = np.concatenate([plain_attention(q[q_start[r]:q_start[r + 1]].astype(np.float64), keys[r], vals[r], ctx[r] - fresh[r], scale, window,
                                           sinks.astype(np.float64) if use_s else None,
                                           gate[q_start[r]:q_start[r + 1]].astype(np.float64) if use_g else None) for r in range(R)])
    out = new(rt, (T, H * E), dtype)
    tab, d_rows = i32(rt, table), up(rt, rows, dtype)
    d_gate = d_rows.ptr + H * D * (2 if dtype == "bfloat16" else 4) if use_g else None
    d_sinks = up(rt, sinks).ptr if use_s else None
    if tuned:
        need = (int(k.zk_attention_bf16_workspace(R, H, E, max_ctx)) + 255) // 256 * 256
        need += int(k.zk_attention_bf16_portion_workspace(2 * (448 + 128), H, G, E))
        ws = new(rt, (need // 4 + 16,))
        for chunk in (64, 32) if mode == 0 else (64,):
            before = k.zk_attention_bf16_portion_kernel(mode)
            try:
                k.zk_attention_bf16_gated(d_rows.ptr, ld, up(rt, kc, dtype).ptr, up(rt, vc, dtype).ptr, tab.ptr, blocks,
                                          i32(rt, q_start).ptr, i32(rt, ctx).ptr, out.ptr, R, 2, 448, max_ctx, H, G, D, bs, scale, 0.0,
                                          window, chunk, ws.ptr, ws.nbytes, 0, 0, 1, 0, E, 0, d_sinks, d_gate, ld, rt.stream)
            finally:
                k.zk_attention_bf16_portion_kernel(before)
            err = np.abs(rt.download_f32(out).reshape(T, H, E) - want).max(axis=(1, 2))
            assert err.max() < 0.02, (chunk, int(np.argmax(err)), float(err.max()))
        return
    positions = np.concatenate([np.arange(ctx[r] - fresh[r], ctx[r]) for r in range(R)])
    owner = np.concatenate([np.full(fresh[r], r) for r in range(R)])
    k.zk_attention_plain_gated(d_rows.ptr, ld, up(rt, kc, dtype).ptr, up(rt, vc, dtype).ptr, tab.ptr, blocks, i32(rt, owner).ptr,
                               i32(rt, positions).ptr, out.ptr, T, H, G, D, E, bs, scale, 0.0, window, 0, None, 0, d_sinks, 0, 0, 0, 0,
                               d_gate, ld, rt.stream)
    err = np.abs(rt.download_f32(out).reshape(T, H, E) - want).max(axis=(1, 2))
    assert err.max() < (1e-5 if dtype == "float32" else 0.02), (int(np.argmax(err)), float(err.max()))


# ---------------------------------------------------------------- router and experts
@pytest.mark.parametrize("n,top,groups,keep", [(14, 3, 2, 1), (9, 3, 3, 2), (4, 4, 4, 4), (6, 2, 1, 1), (130, 16, 13, 4), (1024, 8, 128, 2),
                                               (64, 6, 64, 9), (3, 1, 3, 1)])
def test_groups_judged_by_their_best(n, top, groups, keep):
    rt, k = lib()
    rng = np.random.default_rng(n + top)
    T, ld = 40, n + 1
    z = rng.normal(0, 2, (T, ld)).astype(np.float32)
    z[3, :n] = 0.5                                     # equal scores
    corr = rng.normal(-0.2, 0.3, n).astype(np.float32)         # choice scores below zero among them
    ids, wts = i32(rt, np.zeros((T, top))), new(rt, (T, top))
    for c, best in ((corr, 1), (np.zeros(n, np.float32), 1), (corr, 2)):
        k.zk_moe_route_best(up(rt, z).ptr, ld, up(rt, c).ptr if c.any() else None, ids.ptr, wts.ptr, T, n, top, groups, keep, 1, 0, 1.7,
                            best, rt.stream)
        got_i, got_w = rt.download(ids), rt.download(wts)
        s = P.router_scores(z[:, :n].astype(np.float64), np.eye(n), np.float64)
        for t in range(T):
            assert len(set(got_i[t])) == top and got_i[t].min() >= 0 and got_i[t].max() < n
            assert np.abs(got_w[t] - 1.7 * s[t, got_i[t]]).max() < 1e-6
            if best != 1:
                continue
            want, gap = P.choose((s[t] + c).astype(np.float32), top, (groups, keep))
            order = np.sort((s[t] + c)[want])
            if (gap > 1e-6 and (np.diff(order) > 1e-6).all()) or (t == 3 and not c.any()):
                assert got_i[t].tolist() == want.tolist(), t


@pytest.mark.parametrize("T,E,I,top,W,F", [(3, 5, 2, 2, 48, 24), (40, 4, 3, 3, 36, 20), (1, 2, 1, 2, 64, 96), (90, 12, 4, 4, 64, 32),
                                           (70, 1, 3, 2, 40, 16), (200, 3, 0, 2, 128, 64), (300, 2, 1, 2, 72, 136), (33, 70, 3, 4, 136, 72),
                                           (150, 3, 1, 3, 1032, 200)])
@pytest.mark.parametrize("all_identity", [False, True])
def test_identity_experts_among_the_choices(T, E, I, top, W, F, all_identity):
    """Row by row in 32-bit; row by row and grouped on the matrix cores in bfloat16.  The scratch memory
    holds what is not a number: nothing of an identity expert's rows is read from there."""
    if all_identity and I < top:
        pytest.skip("more choices than identity experts")
    rt, k = lib()
    rng = np.random.default_rng(T + E)
    x = bf16(rng.normal(size=(T, W)))
    wg, wu = bf16(rng.normal(0, W ** -0.5, (E, F, W))), bf16(rng.normal(0, W ** -0.5, (E, F, W)))
    wd = bf16(rng.normal(0, F ** -0.5, (E, W, F)))
    lo = E if all_identity else 0
    ids = np.stack([lo + rng.permutation(E + I - lo)[:top] for _ in range(T)]).astype(np.int32)
    wts = rng.uniform(0.05, 1.5, (T, top)).astype(np.float32)
    want = np.zeros((T, W))
    xd = x.astype(np.float64)
    for t in range(T):
        for e, s in zip(ids[t], wts[t]):
            want[t] += s * (xd[t] if e >= E else (P.silu(xd[t] @ wg[e].T) * (xd[t] @ wu[e].T)) @ wd[e].T)
    gu = np.concatenate([wg, wu], axis=1)
    # a shared layer's rows on top: none, as they are, or times the sigmoid of the fourth of five numbers a row
    add, z = rng.normal(size=(T, W)).astype(np.float32), rng.normal(0, 2, (T, 5)).astype(np.float32)
    how = (T + E + all_identity) % 3
    want = want + (0.0 if how == 0 else add if how == 1 else add * P.sigmoid(z[:, 3:4].astype(np.float64)))
    more = lambda rt: (None if how == 0 else up(rt, add).ptr, up(rt, z).ptr + 12 if how == 2 else None, 5)
    scale = np.abs(want).max()
    nan = lambda shape, dtype: up(rt, np.full(shape, np.nan), dtype)
    out = new(rt, (T, W))
    k.zk_moe_experts_identity(up(rt, x).ptr, i32(rt, ids).ptr, up(rt, wts).ptr, up(rt, gu).ptr, up(rt, wd).ptr, nan((T * top, F), "float32").ptr,
                              out.ptr, T, top, W, F, 0.0, 1, 1, E, *more(rt), rt.stream)
    assert np.abs(rt.download(out) - want).max() < 1e-5 * scale
    rt, kb = lib("bfloat16")
    h16 = lambda a: up(rt, a, "bfloat16").ptr
    out = new(rt, (T, W))
    kb.zk_moe_experts_identity(h16(x), i32(rt, ids).ptr, up(rt, wts).ptr, h16(gu), h16(wd), nan((T * top, F), "bfloat16").ptr, out.ptr, T, top, W,
                               F, 0.0, 1, 1, E, *more(rt), rt.stream)
    assert np.abs(rt.download(out) - want).max() < 0.02 * scale
    if W % 8 or F % 8:
        return
    work = i32(rt, np.zeros(E + I + 1 + 2 * T * top))
    out = new(rt, (T, W))
    kb.zk_moe_experts_grouped_identity(h16(x), i32(rt, ids).ptr, up(rt, wts).ptr, h16(gu), h16(wd), work.ptr, None,
                                       nan((T * top, F), "bfloat16").ptr, nan((T * top, W), "float32").ptr, out.ptr, T, E, top, W, F, 0.0, 1, 1,
                                       I, *more(rt), rt.stream)
    assert np.abs(rt.download(out) - want).max() < 0.02 * scale


# ---------------------------------------------------------------- what joins the stream
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("T,W", [(5, 36), (3, 30), (9, 2048), (70, 2048), (4, 5000), (2, 8200), (6, 4097)])
@pytest.mark.parametrize("parts", [0, 3])
def test_a_normed_result_joins_and_the_stream_itself_is_handed_on(T, W, parts, dtype):
    """Every variant of the joining kernel: rows in whole groups of four or not, few and many of them."""
    rt, k = lib(dtype)
    rng = np.random.default_rng(T * W)
    h, gain = rng.normal(0, 30, (T, W)).astype(np.float32), rng.normal(0, 0.3, W).astype(np.float32)
    sub = bf16(rng.normal(0, 2, (max(parts, 1), T, W)))
    total = sub.astype(np.float64).sum(axis=0)
    total = bf16(total).astype(np.float64) if dtype == "bfloat16" else total
    dh, out = up(rt, h), new(rt, (T, W), dtype)
    src = up(rt, sub, "float32" if parts else dtype)
    k.zk_norm_add_norm(src.ptr, parts, up(rt, gain).ptr, 1e-5, 1, dh.ptr, None, 0.0, 0, out.ptr, T, W, rt.stream)
    want = h + P.model_norm(total, gain, 1e-5, np.float64)
    got = rt.download(dh)
    assert np.abs(got - want).max() < 2e-5 * np.abs(want).max()
    assert np.array_equal(rt.download_f32(out), got if dtype == "float32" else bf16(got))
    # without an output nothing is handed on
    dh = up(rt, h)
    k.zk_norm_add_norm(src.ptr, parts, up(rt, gain).ptr, 1e-5, 1, dh.ptr, None, 0.0, 0, None, T, W, rt.stream)
    assert np.array_equal(rt.download(dh), got)
    # the first sublayer's input, which nothing joins before
    first = new(rt, (T, W), dtype)
    k.zk_round_rows(up(rt, h).ptr, first.ptr, T * W, rt.stream)
    assert np.array_equal(rt.download_f32(first), h if dtype == "float32" else bf16(h))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("M,K,N,ldc", [(1, 64, 70, 72), (9, 320, 1158, 1160), (40, 64, 70, 80), (150, 128, 390, 392), (300, 72, 21, 24)])
def test_a_product_into_wider_rows(M, K, N, ldc, dtype):
    from types import SimpleNamespace
    from zse_amd.parts.ops import linear
    rt, k = lib(dtype)
    rng = np.random.default_rng(M + N)
    x, w = bf16(rng.normal(size=(M, K))), bf16(rng.normal(0, K ** -0.5, (N, K)))
    out = up(rt, np.full((M, ldc), 7.0), dtype)
    ws = new(rt, (1 << 20,))
    ctx = SimpleNamespace(dtype=dtype, tuned=True, k=k, stream=rt.stream, gemm_workspace=ws, sums_welcome=None)
    linear(ctx, up(rt, x, dtype), up(rt, w, dtype), out, ldc=ldc)
    got, want = rt.download_f32(out), x.astype(np.float64) @ w.T.astype(np.float64)
    assert np.abs(got[:, :N] - want).max() < (1e-5 if dtype == "float32" else 0.02) * np.abs(want).max()
    assert (got[:, N:] == 7.0).all()
    with pytest.raises(ValueError, match="apart"):
        linear(ctx, up(rt, x, dtype), up(rt, w, dtype), out, ldc=N - 1)


@pytest.mark.parametrize("unit", [True, False])
def test_a_factor_in_a_norms_gain(unit):
    from types import SimpleNamespace
    from zse_amd.config.plan import NormSpec
    from zse_amd.parts.norm import RMSNorm
    rt, k = lib()
    rng = np.random.default_rng(1)
    x, w = rng.normal(size=(3, 40)).astype(np.float32), rng.normal(0, 0.3, 40).astype(np.float32)
    n = RMSNorm(NormSpec(40, 1e-5, unit, "n", gain_scale=-0.3))
    source = SimpleNamespace(vector=lambda name: up(rt, w))
    ctx = SimpleNamespace(k=k, stream=rt.stream, alloc=lambda shape, *a: new(rt, shape))
    for _ in range(2):                       # loaded again, the factor is still there once
        n.load(source, rt, "float32")
        want = P.unit_rms(x, 1e-5, np.float64) * (w + (1.0 if unit else 0.0)) * -0.3
        assert np.abs(rt.download(n.forward(ctx, up(rt, x))) - want).max() < 1e-6
