"""Buvuzen: a decoder-only model whose layers are listed one by one in its config.json; a layer may
use the weights of another one.

The embedded row of a token times a number is the stream.  A layer has norms on its sublayers'
results only (RMS norms with a gain stored around zero: 1 + w): h += norm1(mixer(h)), then
h += norm2(ff(h)); the sublayers read the stream itself.  The mixer is a grouped-query attention
without positions: an RMS norm per query and key head, a sliding window, a softmax whose denominator
also holds a learned sink per head, values of a size of their own, and a gate of one number a head on
the outputs.  The feed-forward is a mixture of silu-gated experts with softmax scores that weigh the
chosen experts' outputs: chosen by score plus a correction, among the groups of neighbouring experts
whose best choice score is largest, some of the numbers to choose from standing for identity experts;
and a shared expert times the sigmoid of a number a token.  The logits are those of a head of its own
behind the last norm, times a number.  A layer with the weights of another one keeps keys and values
of its own.

config.json: ``vocab``, ``width``, ``norm.eps``, optional ``embedding.scale``, ``logit_scale``, ``layers`` (a list of
``{type, mixer, mlp}``, optionally with ``weights_of``, the number of the layer whose weights it uses, whose
entry it equals otherwise).  ``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, optional ``mask.size``.
``mlp``: null or ``{kind: "moe", expert: {ff}, router: {experts, top, identity, scale, groups: {count, keep} or null},
shared: {ff} or null}``.  Tensor names: ``embed``, ``head``, ``final.norm`` and, for layer i, ``l<i>.norm1``, ``l<i>.norm2``,
``l<i>.mix.*``, ``l<i>.mlp.*``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from ..config.base import Architecture, Problems, need, register_architecture
from ..config.plan import (AttentionSpec, BlockSpec, EmbeddingSpec, GatedMLPSpec, HeadSpec, LayerCall, ModelPlan,
                           NoPositionSpec, NormSpec, RoutedMLPSpec)

NAME = "Buvuzen"
MAX_POSITION = 1 << 16        # the config names no longest sequence; tables and pools follow the runner's own limits
# the softmax's weights are 32-bit numbers of the design: where a matrix-core kernel multiplies them with
# the values they go in as two bfloat16 halves (16 bits of mantissa), not rounded to one
WIDE_WEIGHTS = True
EXPERT_ACTIVATION = "silu"
GROUP_BEST = 1                # a group of experts is judged by its largest choice score
TYPES = ("attention",)


@dataclass(frozen=True)
class BuvuzenMLP:
    ff: int                            # of one expert
    experts: int
    top: int
    identity: int = 0
    scale: float = 1.0
    groups: Optional[Tuple[int, int]] = None     # count, keep
    shared_ff: Optional[int] = None


@dataclass(frozen=True)
class BuvuzenAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    window: Optional[int] = None


@dataclass(frozen=True)
class BuvuzenLayer:
    type: str
    mixer: BuvuzenAttention
    mlp: Optional[BuvuzenMLP]
    weights: int                       # the layer whose tensors it uses (its own number: its own)


@dataclass(frozen=True)
class BuvuzenConfig:
    vocab: int
    width: int
    eps: float
    embedding_scale: float
    logit_scale: float
    layers: Tuple[BuvuzenLayer, ...]
    raw: dict

    @staticmethod
    def _mlp(mlp: dict, q: Problems) -> Optional[BuvuzenMLP]:
        kind = need(mlp, "kind", str, q, required=True)
        q.require(kind in (None, "moe"), f"mlp.kind must be 'moe', got {kind!r}")
        ex = need(mlp, "expert", dict, q, required=True) or {}
        ro = need(mlp, "router", dict, q, required=True) or {}
        sh = need(mlp, "shared", dict, q, default=None, allow_none=True)
        ff = need(ex, "ff", int, q, required=True)
        experts = need(ro, "experts", int, q, required=True)
        top = need(ro, "top", int, q, required=True)
        identity = need(ro, "identity", int, q, default=0)
        scale = need(ro, "scale", float, q, default=1.0)
        gr = need(ro, "groups", dict, q, default=None, allow_none=True)
        count = need(gr, "count", int, q, required=True) if gr is not None else None
        keep = need(gr, "keep", int, q, required=True) if gr is not None else None
        sff = need(sh, "ff", int, q, required=True) if sh is not None else None
        if q.items:
            return None
        n = experts + identity
        q.require(ff > 0, f"mlp.expert.ff must be positive, got {ff}")
        q.require(experts >= 1 and identity >= 0, f"mlp.router: experts must be positive and identity not negative, got {experts} and {identity}")
        q.require(1 <= top <= n, f"mlp.router: top must lie in 1..experts + identity, got {top} of {n}")
        q.require(top <= 16 and n <= 1024, f"mlp.router: up to 16 of up to 1024 experts, got {top} of {n}")
        q.require(gr is None or (count >= 1 and n % count == 0 and 1 <= keep <= count and keep * (n // count) >= top),
                  f"mlp.router.groups: count divides experts + identity and the kept ones hold 'top' of them, got {count} and {keep}")
        q.require(sh is None or sff > 0, f"mlp.shared.ff must be positive, got {sff}")
        return BuvuzenMLP(ff, experts, top, identity, scale, (count, keep) if gr is not None else None, sff)

    @staticmethod
    def _attention(mx: dict, q: Problems) -> Optional[BuvuzenAttention]:
        heads = need(mx, "heads", int, q, required=True)
        kvh = need(mx, "kv_heads", int, q, default=heads)
        dim = need(mx, "dim", int, q, required=True)
        vdim = need(mx, "vdim", int, q, default=dim)
        scale = need(mx, "scale", float, q, required=True)
        mask = need(mx, "mask", dict, q, default=None, allow_none=True)
        window = need(mask, "size", int, q, required=True) if mask is not None else None
        if q.items:
            return None
        q.require(heads > 0 and dim > 0 and vdim > 0, "heads, dim and vdim must be positive")
        q.require(kvh > 0 and heads % max(kvh, 1) == 0, f"heads ({heads}) must be a multiple of kv_heads ({kvh})")
        q.require(dim <= 256 and vdim <= 256, f"an attention takes dim and vdim up to 256, got {dim} and {vdim}")
        q.require(window is None or window >= 1, f"mask.size must be at least 1, got {window}")
        return BuvuzenAttention(heads, kvh, dim, vdim, scale, window)

    @staticmethod
    def _owner(layers: list, i: int, q: Problems) -> Optional[int]:
        """The layer whose tensors layer i uses, through ``weights_of`` of the layers it names."""
        at, seen = i, set()
        while True:
            of = need(layers[at], "weights_of", int, q, default=None, allow_none=True)
            if of is None or q.items:
                return at
            seen.add(at)
            if not (0 <= of < len(layers)) or of in seen or not isinstance(layers[of], dict):
                q.add(f"weights_of must name another layer that has weights, got {of}")
                return None
            at = of

    @staticmethod
    def from_dict(raw: dict) -> "BuvuzenConfig":
        p = Problems("Buvuzen config.json")
        V = need(raw, "vocab", int, p, required=True)
        W = need(raw, "width", int, p, required=True)
        norm = need(raw, "norm", dict, p, required=True) or {}
        eps = need(norm, "eps", float, p, required=True)
        emb = need(raw, "embedding", dict, p, default=None, allow_none=True) or {}
        scale = need(emb, "scale", float, p, default=1.0)
        logit_scale = need(raw, "logit_scale", float, p, default=1.0)
        layers_raw = need(raw, "layers", list, p, required=True) or []
        p.raise_if_any()
        p.require(V > 0 and W > 0, f"'vocab' and 'width' must be positive, got {V} and {W}")
        p.require(eps > 0, f"'norm.eps' must be positive, got {eps}")
        p.require(len(layers_raw) > 0, "'layers' is empty")
        layers = []
        for i, lr in enumerate(layers_raw):
            q = Problems(f"layer {i}")
            if not isinstance(lr, dict):
                p.add(f"layer {i} must be an object")
                continue
            typ = need(lr, "type", str, q, required=True)
            mx = need(lr, "mixer", dict, q, required=True) or {}
            mlp_raw = need(lr, "mlp", dict, q, default=None, allow_none=True)
            mlp = BuvuzenConfig._mlp(mlp_raw, q) if mlp_raw is not None else None
            mixer = None
            if typ not in TYPES:
                q.add(f"unknown type {typ!r} {TYPES}")
            elif not q.items:
                mixer = BuvuzenConfig._attention(mx, q)
            owner = BuvuzenConfig._owner(layers_raw, i, q)
            layers.append(BuvuzenLayer(typ, mixer, mlp, owner if owner is not None else i))
            if q.items:
                p.add(f"layer {i}: " + "; ".join(q.items))
        p.raise_if_any()
        for i, l in enumerate(layers):
            o = layers[l.weights]
            p.require((l.type, l.mixer, l.mlp) == (o.type, o.mixer, o.mlp),
                      f"layer {i}: it uses the weights of layer {l.weights}, so its entry must equal that layer's")
        p.raise_if_any()
        return BuvuzenConfig(V, W, eps, scale, logit_scale, tuple(layers), dict(raw))

    def to_dict(self) -> dict:
        return dict(self.raw)


def _layer(c: BuvuzenConfig, i: int) -> BlockSpec:
    l, pre = c.layers[i], f"l{i}."
    a, mix = l.mixer, pre + "mix."
    mixer = AttentionSpec(
        hidden_size=c.width, num_heads=a.heads, num_kv_heads=a.kv_heads, head_dim=a.dim, scale=a.scale, softcap=None,
        window=a.window, position=NoPositionSpec(), names={r: mix + r for r in ("q", "k", "v", "o")}, value_dim=a.vdim,
        q_norm=mix + "q.norm", k_norm=mix + "k.norm", norm_eps=c.eps, sinks=mix + "sink", head_gate=mix + "g",
        wide_weights=WIDE_WEIGHTS)
    norms = {"post_mixer": NormSpec(c.width, c.eps, True, pre + "norm1")}
    ffn = None
    if l.mlp is not None:
        m, mlp = l.mlp, pre + "mlp."
        norms["post_ffn"] = NormSpec(c.width, c.eps, True, pre + "norm2")
        shared = None
        if m.shared_ff is not None:
            shared = GatedMLPSpec(hidden_size=c.width, intermediate_size=m.shared_ff, activation=EXPERT_ACTIVATION,
                                  names={r: f"{mlp}shared.{r}" for r in ("gate", "up", "down")})
        ffn = RoutedMLPSpec(
            hidden_size=c.width, intermediate_size=m.ff, num_experts=m.experts, top_k=m.top, activation=EXPERT_ACTIVATION,
            limit=None, router=mlp + "router", expert_names=mlp + "e{e}.{role}", shared=shared, scale_input=False,
            scoring="softmax", correction=mlp + "correction", groups=m.groups, group_best=GROUP_BEST, identity=m.identity,
            weight_scale=m.scale, shared_gate=(mlp + "shared.sg") if shared is not None else None)
    return BlockSpec(arrangement="postnorm", mixer=mixer, ffn=ffn, norms=norms)


def buvuzen_plan(c: BuvuzenConfig) -> ModelPlan:
    owners = sorted({l.weights for l in c.layers})        # the layers that have weights
    place = {o: n for n, o in enumerate(owners)}
    # a layer without a feed-forward has no second norm; a checkpoint may hold one
    unused = tuple(f"l{o}.norm2" for o in owners if c.layers[o].mlp is None)
    return ModelPlan(
        architecture=NAME, hidden_size=c.width, vocab_size=c.vocab, max_position=MAX_POSITION,
        embedding=EmbeddingSpec(c.vocab, c.width, c.embedding_scale, "embed", exact_scale=True),
        layers=tuple(_layer(c, o) for o in owners), order=tuple(LayerCall(place[l.weights]) for l in c.layers),
        # the logits are linear in the last norm's result: their factor rides in its gain, in floats
        final_norm=NormSpec(c.width, c.eps, True, "final.norm", gain_scale=c.logit_scale),
        head=HeadSpec(c.vocab, c.width, None, "head"),
        ignored_tensors=unused, optional_prefixes=())


BUVUZEN = register_architecture(Architecture(
    name=NAME, config_from_dict=BuvuzenConfig.from_dict, plan=buvuzen_plan, model_types=("buvuzen",)))
