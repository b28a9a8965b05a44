"""A plain, slow Bizepel forward pass over whole sequences (NumPy, no cache, no state carried
between calls).

Test-only oracle: one function per mechanism, written from the design's equations, sharing
nothing with the engine's product path.  It reads config.json keys itself and looks weights up
by their checkpoint names.  Every function takes ``dt`` (``np.float32`` or ``np.float64``) and
carries out all arithmetic in that type.

Notation: T tokens, W the model width, H query heads, G key/value heads, D the query/key size
of a head, E its value size, I the channels of a selective scan, N its state values a channel.
"""
from __future__ import annotations

import math

import numpy as np


# ---------------------------------------------------------------- small functions
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def softplus(z):
    return np.log1p(np.exp(-np.abs(z))) + np.maximum(z, 0)


_erf = np.vectorize(math.erf, otypes=[np.float64])


def gelu_exact(z):
    return 0.5 * z * (1.0 + _erf(z / math.sqrt(2.0))).astype(z.dtype)


def gelu_tanh(z):
    return 0.5 * z * (1.0 + np.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z * z * z)))


def relu_squared(z):
    return np.maximum(z, 0) ** 2


def unit_rms(x, eps, dt):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = x.astype(dt)
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + dt(eps))


def layer_norm(x, w, eps, dt):
    """(x - mean) / sqrt(var + eps) * w, var the mean of the squared deviations; no bias."""
    x = x.astype(dt)
    d = x - x.mean(axis=-1, keepdims=True)
    return d / np.sqrt((d * d).mean(axis=-1, keepdims=True) + dt(eps)) * w.astype(dt)


def causal_conv(u, w, dt):
    """y_t = sum_j w[:, j] u_(t - taps + 1 + j) channel by channel, rows before the start zero."""
    T, C = u.shape
    taps = w.shape[1]
    padded = np.concatenate([np.zeros((taps - 1, C), dt), u.astype(dt)])
    y = np.zeros((T, C), dt)
    for j in range(taps):
        y += w[:, j].astype(dt) * padded[j:j + T]
    return y


# ---------------------------------------------------------------- attention
def rotary_frequencies(dims, base):
    return np.array([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=np.float64)


def rotate_neighbours(x, positions, freqs, dt):
    """Rotate the first 2 n channels of the last axis, n = len(freqs): channel 2i with channel
    2i + 1 by the angle position * f_i; x: [T, heads, size]."""
    x = x.astype(dt).copy()
    n = 2 * len(freqs)
    ang = np.asarray(positions, dtype=np.float64)[:, None] * freqs[None, :]
    cs, sn = np.cos(ang).astype(dt)[:, None, :], np.sin(ang).astype(dt)[:, None, :]
    a, b = x[..., 0:n:2].copy(), x[..., 1:n:2].copy()
    x[..., 0:n:2] = a * cs - b * sn
    x[..., 1:n:2] = b * cs + a * sn
    return x


def visible(T, window, keep):
    """mask[i, j]: j <= i, and i - j < window or j < keep where there is a window."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    m = j <= i
    if window:
        m &= ((i - j) < window) | (j < keep)
    return m


def softmax_attention(q, k, v, scale, mask, dt):
    """q [T, H, D], k [T, G, D], v [T, G, E] -> [T, H, E]; query head h reads key/value head
    h // (H / G); softmax over the keys that ``mask`` shows."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = np.zeros((T, H, v.shape[2]), dtype=dt)
    for h in range(H):
        g = h // (H // G)
        s = (q[:, h] @ k[:, g].T) * dt(scale)
        s = np.where(mask, s, -np.inf)
        p = np.exp(s - s.max(axis=1, keepdims=True))
        out[:, h] = (p / p.sum(axis=1, keepdims=True)) @ v[:, g]
    return out


def attention_values(x, w, m, mx, dt):
    """The values of a layer after bias and convolution, before any mixing: [T, G * E]."""
    v = x @ w[m + "v"].T.astype(dt) + w[m + "v.b"].astype(dt)
    return causal_conv(v, w[m + "v.conv"], dt) if mx.get("conv") else v


def attention_mixer(x, positions, w, m, mx, eps, v_first, dt):
    """Returns (result [T, W], the layer's values before mixing)."""
    T = len(x)
    H, D, E = mx["heads"], mx["dim"], mx.get("vdim", mx["dim"])
    G = mx.get("kv_heads", H)
    rows = {}
    for r in ("q", "k"):
        u = x @ w[m + r].T.astype(dt) + w[f"{m}{r}.b"].astype(dt)
        if mx.get("conv"):
            u = causal_conv(u, w[f"{m}{r}.conv"], dt)
        rows[r] = u.reshape(T, -1, D)
        rows[r] = unit_rms(rows[r], eps, dt) * w[f"{m}{r}.norm"].astype(dt)
        if mx.get("rot"):
            rows[r] = rotate_neighbours(rows[r], positions, rotary_frequencies(mx["rot"].get("dims", D), mx["rot"]["base"]), dt)
    v = own = attention_values(x, w, m, mx, dt)
    if v_first is not None:
        lam = dt(w[m + "vmix"].reshape(()))
        v = (dt(1) - lam) * v + lam * v_first
    mask = mx.get("mask") or {}
    seen = visible(T, mask.get("size"), mask.get("keep_first", 0))
    o = softmax_attention(rows["q"], rows["k"], v.reshape(T, G, E), mx["scale"], seen, dt)
    return o.reshape(T, H * E) @ w[m + "o"].T.astype(dt), own


# ---------------------------------------------------------------- selective scan
def selective_scan(u, step, A, B, C, D, dt):
    """u, step [T, I], A [I, N], B, C [T, N], D [I] -> y [T, I]; the state starts at zero."""
    S = np.zeros(A.shape, dt)
    y = np.zeros(u.shape, dt)
    for t in range(len(u)):
        S = np.exp(step[t][:, None] * A) * S + (step[t] * u[t])[:, None] * B[t][None, :]
        y[t] = S @ C[t] + D * u[t]
    return y


def scan_mixer(x, w, m, mx, dt):
    I, N, R = mx["inner"], mx["state"], mx["dt_rank"]
    f = lambda name: w[m + name].astype(dt)
    uz = x @ f("in").T
    u, z = uz[:, :I], uz[:, I:]
    u = silu(causal_conv(u, w[m + "conv"], dt) + f("conv.b"))
    p = u @ f("x").T
    step = softplus(p[:, :R] @ f("dt").T + f("dt.b"))
    y = selective_scan(u, step, -np.exp(f("A_log")), p[:, R:R + N], p[:, R + N:], f("D"), dt)
    return (y * silu(z)) @ f("o").T


# ---------------------------------------------------------------- generalized delta rule
def general_delta_rule(r, k, v, w, a, dt, cancel=None):
    """One head: r, k, w, a [T, D], v [T, D] -> o [T, D].  S <- diag(w) S - (a u)(u^T S) + k v^T with
    the unit key u, both terms from the old S; o = S^T r.
    ``cancel``: an array [T] that receives the least size of o beside that of an o whose terms do not
    cancel: what is normalised next carries the rounding of r and S over this number."""
    D = r.shape[1]
    S = np.zeros((D, v.shape[1]), dt)
    o = np.zeros(v.shape, dt)
    for t in range(len(r)):
        u = k[t] / np.sqrt((k[t] * k[t]).sum() + dt(1e-6))
        S = w[t][:, None] * S - np.outer(a[t] * u, u @ S) + np.outer(k[t], v[t])
        o[t] = S.T @ r[t]
        if cancel is not None:
            whole = np.linalg.norm(r[t]) * np.linalg.norm(S) / math.sqrt(D)
            cancel[t] = min(cancel[t], np.linalg.norm(o[t]) / max(whole, 1e-30))
    return o


def general_delta_mixer(x, w, m, mx, eps, dt, cancel=None):
    T, H, D = len(x), mx["heads"], mx["dim"]
    f = lambda name: w[m + name].astype(dt)
    heads = lambda y: y.reshape(T, H, D)
    r, k, v = (heads(x @ f(n).T) for n in ("r", "k", "v"))
    decay = heads(np.exp(-math.exp(-0.5) * sigmoid(np.tanh(x @ f("w1").T) @ f("w2").T + f("w0"))))
    rate = heads(sigmoid(x @ f("a").T + f("a.b")))
    o = np.stack([general_delta_rule(r[:, h], k[:, h], v[:, h], decay[:, h], rate[:, h], dt, cancel) for h in range(H)], axis=1)
    o = unit_rms(o, eps, dt).reshape(T, H * D) * f("norm")
    return (o * sigmoid(x @ f("g").T)) @ f("o").T


# ---------------------------------------------------------------- feed-forward
def dense(x, w, f, dt):
    return gelu_exact(x @ w[f + "up"].T.astype(dt)) @ w[f + "down"].T.astype(dt)


def expert(x, w, f, dt):
    return relu_squared(x @ w[f + "up"].T.astype(dt)) @ w[f + "down"].T.astype(dt)


def choose(scores, correction, top, groups):
    """One token: the chosen experts (largest choice score first; the lower number among equals)."""
    c = scores + correction
    if groups:
        size = len(c) // groups["count"]
        value = [np.sort(c[g * size:(g + 1) * size])[::-1][:2].sum() for g in range(groups["count"])]
        kept = np.argsort(-np.array(value), kind="stable")[:groups["keep"]]
        c = np.array([c[e] if e // size in kept else -np.inf for e in range(len(c))])
    return np.argsort(-c, kind="stable")[:top]


def closeness(scores, correction, top, groups):
    """How close a token's choice was: the least distance between something chosen and something
    left out, of groups and of experts among the kept groups."""
    c = scores + correction
    near = np.inf
    if groups:
        size = len(c) // groups["count"]
        value = np.array([np.sort(c[g * size:(g + 1) * size])[::-1][:2].sum() for g in range(groups["count"])])
        order = np.sort(value)[::-1]
        if groups["keep"] < groups["count"]:
            near = min(near, order[groups["keep"] - 1] - order[groups["keep"]])
        kept = np.argsort(-value, kind="stable")[:groups["keep"]]
        c = np.array([c[e] for e in range(len(c)) if e // size in kept])
    order = np.sort(c)[::-1]
    if top < len(order):
        near = min(near, order[top - 1] - order[top])
    return near


def mixture(x, w, f, ml, dt, close=None):
    ro = ml["router"]
    scores = sigmoid(x @ w[f + "router"].T.astype(dt))
    corr = w[f + "correction"].astype(dt)
    y = np.zeros_like(x)
    share = np.zeros(scores.shape, dt)           # of every expert in every token; 0: not chosen
    for t in range(len(x)):
        ids = choose(scores[t], corr, ro["top"], ro.get("groups"))
        share[t, ids] = scores[t][ids] / (scores[t][ids].sum() + dt(1e-20)) * dt(ro.get("scale", 1.0))
        if close is not None:
            close[t] = min(close[t], closeness(scores[t], corr, ro["top"], ro.get("groups")))
    for e in range(ro["experts"]):
        at = np.nonzero(share[:, e])[0]
        if len(at):
            y[at] += share[at, e][:, None] * expert(x[at], w, f"{f}e{e}.", dt)
    if ml.get("shared"):
        y += expert(x, w, f + "shared.", dt)
    return y


# ---------------------------------------------------------------- the model
def side_input(h, tokens, i, w, cfg, dt):
    """The per-layer token input: what is added to the stream after the feed-forward."""
    p, d = f"l{i}.side.", cfg["token_side"]["dim"]
    e = w["side.embed"][np.asarray(tokens), i * d:(i + 1) * d].astype(dt)
    g = gelu_tanh(h @ w[p + "gate"].T.astype(dt)) * e
    return unit_rms(g @ w[p + "proj"].T.astype(dt), cfg["norm"]["eps"], dt) * w[p + "norm"].astype(dt)


def forward(cfg, w, tokens, dt=np.float64, layers_out=None, close=None, cancel=None):
    """Logits [T, vocab].  ``layers_out``: a list that receives the stream after every layer.
    ``close``: an array [T] that receives how close each token's nearest choice of experts was.
    ``cancel``: an array [T] that receives how far the worst read of a recurrence cancels."""
    eps = cfg["norm"]["eps"]
    tokens = np.asarray(tokens)
    pos = np.arange(len(tokens))
    h = layer_norm(w["embed"][tokens], w["embed.norm"], eps, dt)
    v_first = None
    if close is not None:
        close[:] = np.inf
    if cancel is not None:
        cancel[:] = np.inf

    def read(p, q):
        x = layer_norm(h, w[f"{p}norm{q}"], eps, dt)
        return x + causal_conv(x, w[f"{p}canon{q}"], dt) if cfg.get("canon") else x

    for i, l in enumerate(cfg["layers"]):
        p, mx = f"l{i}.", l["mixer"]
        x = read(p, 1)
        if l["type"] == "mamba1":
            y = scan_mixer(x, w, p + "mix.", mx, dt)
        elif l["type"] == "general_delta":
            y = general_delta_mixer(x, w, p + "mix.", mx, eps, dt, cancel)
        else:
            mixes = bool(mx.get("v_mix"))
            y, own = attention_mixer(x, pos, w, p + "mix.", mx, eps, v_first if mixes else None, dt)
            if mixes and v_first is None:
                v_first = own
        h = h + y * w[p + "ls1"].astype(dt)
        ml = l.get("mlp")
        if ml:
            x = read(p, 2)
            y = dense(x, w, p + "mlp.", dt) if ml["kind"] == "dense" else mixture(x, w, p + "mlp.", ml, dt, close)
            h = h + y * w[p + "ls2"].astype(dt)
        if cfg.get("token_side"):
            h = h + side_input(h, tokens, i, w, cfg, dt)
        if layers_out is not None:
            layers_out.append(h.copy())
    x = layer_norm(h, w["final.norm"], eps, dt)
    return x @ w["embed"].T.astype(dt) * dt(cfg.get("logit_scale", 1.0))
