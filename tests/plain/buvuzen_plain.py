"""A plain, slow Buvuzen forward pass over whole sequences (NumPy, no cache, no state carried
between calls).

Test-only oracle: one function per mechanism, written from the design's equations, sharing
nothing with the engine's product path.  It reads config.json keys itself and looks weights up
by their checkpoint names.  Every function takes ``dt`` (``np.float32`` or ``np.float64``) and
carries out all arithmetic in that type.

Notation: T tokens, W the model width, H query heads, G key/value heads, D the query/key size
of a head, E its value size.
"""
from __future__ import annotations

import numpy as np


# ---------------------------------------------------------------- small functions
def sigmoid(z):
    return 1.0 / (1.0 + np.exp(-z))


def silu(z):
    return z * sigmoid(z)


def unit_rms(x, eps, dt):
    """x / sqrt(mean(x^2) + eps) over the last axis."""
    x = x.astype(dt)
    return x / np.sqrt((x * x).mean(axis=-1, keepdims=True) + dt(eps))


def model_norm(x, w, eps, dt):
    """The norm of a sublayer's result and the model's last one: a gain stored around zero."""
    return unit_rms(x, eps, dt) * (dt(1.0) + w.astype(dt))


def head_norm(x, w, eps, dt):
    """The norm of a query or key head: a plain gain shared by the heads; x: [T, heads, D]."""
    return unit_rms(x, eps, dt) * w.astype(dt)


# ---------------------------------------------------------------- embedding and order
def embed(cfg, w, tokens, dt):
    scale = (cfg.get("embedding") or {}).get("scale", 1.0)
    return w["embed"][np.asarray(tokens)].astype(dt) * dt(scale)


def weights_layer(cfg, i):
    """The layer whose tensors layer i uses."""
    while cfg["layers"][i].get("weights_of") is not None:
        i = cfg["layers"][i]["weights_of"]
    return i


# ---------------------------------------------------------------- the mixer
def visible(T, window):
    """mask[i, j]: j <= i, and i - j < window where there is one."""
    i, j = np.arange(T)[:, None], np.arange(T)[None, :]
    m = j <= i
    if window:
        m &= (i - j) < window
    return m


def sink_softmax(s, mask, sink):
    """exp(s_j) / (exp(sink) + sum over visible keys of exp(s)), row by row."""
    s = np.where(mask, s, -np.inf)
    top = np.maximum(s.max(axis=1, keepdims=True), sink)
    p = np.exp(s - top)
    return p / (p.sum(axis=1, keepdims=True) + np.exp(sink - top))


def attention_mixer(mx, w, pre, x, eps, dt):
    T = x.shape[0]
    H, G, D = mx["heads"], mx.get("kv_heads", mx["heads"]), mx["dim"]
    E = mx.get("vdim", D)
    q = head_norm((x @ w[pre + "q"].astype(dt).T).reshape(T, H, D), w[pre + "q.norm"], eps, dt)
    k = head_norm((x @ w[pre + "k"].astype(dt).T).reshape(T, G, D), w[pre + "k.norm"], eps, dt)
    v = (x @ w[pre + "v"].astype(dt).T).reshape(T, G, E)
    gate = sigmoid(x @ w[pre + "g"].astype(dt).T)
    mask = visible(T, (mx.get("mask") or {}).get("size"))
    o = np.zeros((T, H, E), dtype=dt)
    for h in range(H):
        g = h // (H // G)
        p = sink_softmax((q[:, h] @ k[:, g].T) * dt(mx["scale"]), mask, dt(w[pre + "sink"][h]))
        o[:, h] = (p @ v[:, g]) * gate[:, h:h + 1]
    return o.reshape(T, H * E) @ w[pre + "o"].astype(dt).T


# ---------------------------------------------------------------- feed-forward
def gated(x, w, pre, dt):
    return (silu(x @ w[pre + "gate"].astype(dt).T) * (x @ w[pre + "up"].astype(dt).T)) @ w[pre + "down"].astype(dt).T


def router_scores(x, w_router, dt):
    z = x.astype(dt) @ w_router.astype(dt).T
    s = np.exp(z - z.max(axis=1, keepdims=True))
    return s / s.sum(axis=1, keepdims=True)


def choose(choice, top, groups):
    """One token's choice among the scores ``choice``: with (count, keep) only the experts of the
    ``keep`` groups with the largest single scores are in the race.  The lower number among equals,
    of groups as of experts.  Returns the ids in the order they were chosen and the smallest gap that
    decided anything (between the last kept and the first dropped group, the last chosen and the
    first left-out expert)."""
    n = len(choice)
    gap = np.inf
    allowed = np.ones(n, bool)
    if groups is not None and groups[1] < groups[0]:
        count, keep = groups
        best = choice.reshape(count, n // count).max(axis=1)
        order = np.argsort(-best, kind="stable")
        gap = best[order[keep - 1]] - best[order[keep]]
        for g in order[keep:]:
            allowed[g * (n // count):(g + 1) * (n // count)] = False
    c = np.where(allowed, choice, -np.inf)
    order = np.argsort(-c, kind="stable")
    if top < n:
        gap = min(gap, c[order[top - 1]] - c[order[top]])
    return order[:top], gap


def mixture(ml, w, pre, x, dt, close=None):
    """sum over the chosen of weight * expert(x), the last ``identity`` of the router's outputs being
    experts that give x back; plus the shared expert times sigmoid(W_sg x), one number a token."""
    r = ml["router"]
    gr = r.get("groups")
    s = router_scores(x, w[pre + "router"], dt)
    choice = s + w[pre + "correction"].astype(dt)
    out = np.zeros_like(x, dtype=dt)
    for t in range(x.shape[0]):
        ids, gap = choose(choice[t], r["top"], (gr["count"], gr["keep"]) if gr else None)
        if close is not None:
            close[t] = min(close[t], gap)
        for e in ids:
            y = x[t] if e >= r["experts"] else gated(x[t:t + 1], w, f"{pre}e{e}.", dt)[0]
            out[t] += s[t, e] * dt(r.get("scale", 1.0)) * y
    if ml.get("shared"):
        out += gated(x, w, pre + "shared.", dt) * sigmoid(x @ w[pre + "shared.sg"].astype(dt).T)
    return out


# ---------------------------------------------------------------- the model
def forward(cfg, w, tokens, dt=np.float64, layers_out=None, close=None):
    """Logits [T, vocab] of one sequence.  ``layers_out``: a list that receives the stream after
    every layer; ``close``: an array [T] that receives how close each token's nearest choice of
    experts was, as a gap between choice scores."""
    eps = cfg["norm"]["eps"]
    if close is not None:
        close[:] = np.inf
    x = embed(cfg, w, tokens, dt)
    for i in range(len(cfg["layers"])):
        j = weights_layer(cfg, i)
        l, p = cfg["layers"][j], f"l{j}."
        x = x + model_norm(attention_mixer(l["mixer"], w, p + "mix.", x, eps, dt), w[p + "norm1"], eps, dt)
        if l.get("mlp"):
            x = x + model_norm(mixture(l["mlp"], w, p + "mlp.", x, dt, close), w[p + "norm2"], eps, dt)
        if layers_out is not None:
            layers_out.append(x.copy())
    x = model_norm(x, w["final.norm"], eps, dt)
    return (x @ w["head"].astype(dt).T) * dt(cfg.get("logit_scale", 1.0))
