"""Bizepel: a decoder-only model whose layers are listed one by one in its config.json.

The embedded row of a token passes a layer norm before it becomes the stream.  A layer is a
pre-norm layer (layer norms with a gain and no bias); each sublayer reads h + conv(h), a short
causal convolution over time of its normed input, and its result is multiplied by a gain per
channel before it joins the stream.  After the feed-forward every layer adds an input that
follows from the token itself, rms(W_proj (gelu_tanh(W_gate x) * e)) * gain with e the layer's part of
the token's row of a second table.  The mixer is
  - ``attention``: grouped-query attention with biases on q, k and v, a short convolution over time on
    all three, an RMS norm per query and key head, rotary positions (pairs (2i, 2i + 1)) on part of a
    head, a sliding window that keeps the sequence's first tokens in sight, values of a size of
    their own; in every ``v_mix`` layer but the first the values are mixed with the first one's;
  - ``mamba1``: a selective scan behind a causal convolution with bias and silu;
  - ``general_delta``: a recurrence over a matrix state per head, the generalized delta rule.
The feed-forward is W_down gelu(W_up x) (the gelu with the error function) or a mixture of
W_down relu(W_up x)^2 experts: sigmoid scores, chosen by score plus a correction among the best groups of
neighbouring experts, weights brought to a sum and scaled, and a shared expert.  The logits come
from the embedding table behind a layer norm, times a number.

config.json: ``vocab``, ``width``, ``norm.eps``, optional ``canon.taps``, ``token_side.dim``, ``logit_scale``,
``layers`` (a list of ``{type, mixer, mlp}``).  ``attention``: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``,
optional ``conv``, ``rot`` (``base``, ``dims``), ``mask`` (``size``, ``keep_first``), ``v_mix``.  ``mamba1``: ``inner``,
``state``, ``dt_rank``, ``conv``.  ``general_delta``: ``heads``, ``dim`` (the rank of the decays' projection is read off
the tensors).  ``mlp``: null, ``{kind: "dense", ff}`` or ``{kind: "moe", expert: {ff}, router: {experts, top,
groups: {count, keep} or null, scale}, shared: {ff} or null}``.  Tensor names: ``embed``, ``embed.norm``,
``side.embed``, ``final.norm`` and, for layer i, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.canon1``, ``l<i>.canon2``,
``l<i>.ls1``, ``l<i>.ls2``, ``l<i>.mix.*``, ``l<i>.mlp.*``, ``l<i>.side.*``.
"""
from __future__ import annotations

from dataclasses import dataclass
from typing import Optional, Tuple

from ..config.base import Architecture, Problems, need, register_architecture
from ..config.plan import (AttentionSpec, EmbeddingSpec, FilteredBlockSpec, GeneralDeltaSpec, HeadSpec, LayerCall,
                           LayerNormSpec, MLPSpec, ModelPlan, NoPositionSpec, RotarySpec, RoutedMLPSpec, SelectiveScanSpec,
                           ShortConvSpec, TokenSideSpec)

NAME = "Bizepel"
MAX_POSITION = 1 << 16        # the config names no longest sequence; tables and pools follow the runner's own limits
# the softmax's weights are 32-bit numbers of the design: where a matrix-core kernel multiplies them with
# the values they go in as two bfloat16 halves (16 bits of mantissa), not rounded to one
WIDE_WEIGHTS = True
DENSE_ACTIVATION = "gelu"
EXPERT_ACTIVATION = "relu2"
TYPES = ("attention", "mamba1", "general_delta")


@dataclass(frozen=True)
class BizepelMLP:
    kind: str                          # "dense" | "moe"
    ff: int                            # of the dense layer, or of one expert
    experts: int = 0
    top: int = 0
    groups: Optional[Tuple[int, int]] = None     # count, keep
    scale: float = 1.0
    shared_ff: Optional[int] = None


@dataclass(frozen=True)
class BizepelAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    taps: Optional[int] = None
    window: Optional[int] = None
    keep: int = 0
    rot_base: Optional[float] = None
    rot_dims: int = 0
    v_mix: bool = False


@dataclass(frozen=True)
class BizepelScan:
    inner: int
    state: int
    dt_rank: int
    taps: int


@dataclass(frozen=True)
class BizepelDelta:
    heads: int
    dim: int
    rank: int                          # of the decays' projection (0: the tensors say it)


@dataclass(frozen=True)
class BizepelLayer:
    type: str
    mixer: object
    mlp: Optional[BizepelMLP]


@dataclass(frozen=True)
class BizepelConfig:
    vocab: int
    width: int
    eps: float
    taps: Optional[int]                # of the sublayers' input convolution
    side_dim: Optional[int]
    logit_scale: float
    layers: Tuple[BizepelLayer, ...]
    raw: dict

    @staticmethod
    def _mlp(mlp: dict, q: Problems) -> Optional[BizepelMLP]:
        kind = need(mlp, "kind", str, q, required=True)
        if kind == "dense":
            ff = need(mlp, "ff", int, q, required=True)
            q.require(ff is None or ff > 0, f"mlp.ff must be positive, got {ff}")
            return BizepelMLP("dense", ff or 0)
        if kind != "moe":
            q.add(f"mlp.kind must be 'dense' or 'moe', got {kind!r}")
            return None
        ex = need(mlp, "expert", dict, q, required=True) or {}
        ro = need(mlp, "router", dict, q, required=True) or {}
        sh = need(mlp, "shared", dict, q, default=None, allow_none=True)
        ff = need(ex, "ff", int, q, required=True)
        experts = need(ro, "experts", int, q, required=True)
        top = need(ro, "top", int, q, required=True)
        scale = need(ro, "scale", float, q, default=1.0)
        gr = need(ro, "groups", dict, q, default=None, allow_none=True)
        count = need(gr, "count", int, q, required=True) if gr is not None else None
        keep = need(gr, "keep", int, q, required=True) if gr is not None else None
        sff = need(sh, "ff", int, q, required=True) if sh is not None else None
        if q.items:
            return None
        q.require(ff > 0, f"mlp.expert.ff must be positive, got {ff}")
        q.require(1 <= top <= experts, f"mlp.router: top must lie in 1..experts, got {top} of {experts}")
        q.require(top <= 16 and experts <= 1024, f"mlp.router: up to 16 of up to 1024 experts, got {top} of {experts}")
        q.require(gr is None or (count >= 1 and experts % count == 0 and 1 <= keep <= count and keep * (experts // count) >= top),
                  f"mlp.router.groups: count divides the experts and the kept ones hold 'top' of them, got {count} and {keep}")
        q.require(sh is None or sff > 0, f"mlp.shared.ff must be positive, got {sff}")
        return BizepelMLP("moe", ff, experts, top, (count, keep) if gr is not None else None, scale, sff)

    @staticmethod
    def _attention(mx: dict, q: Problems) -> Optional[BizepelAttention]:
        heads = need(mx, "heads", int, q, required=True)
        kvh = need(mx, "kv_heads", int, q, default=heads)
        dim = need(mx, "dim", int, q, required=True)
        vdim = need(mx, "vdim", int, q, default=dim)
        scale = need(mx, "scale", float, q, required=True)
        taps = need(mx, "conv", int, q, default=None, allow_none=True)
        v_mix = need(mx, "v_mix", bool, q, default=False)
        mask = need(mx, "mask", dict, q, default=None, allow_none=True)
        window = need(mask, "size", int, q, required=True) if mask is not None else None
        keep = need(mask, "keep_first", int, q, default=0) if mask is not None else 0
        rot = need(mx, "rot", dict, q, default=None, allow_none=True)
        base = need(rot, "base", float, q, required=True) if rot is not None else None
        dims = need(rot, "dims", int, q, default=dim) if rot is not None else 0
        if q.items:
            return None
        q.require(heads > 0 and dim > 0 and vdim > 0, "heads, dim and vdim must be positive")
        q.require(kvh > 0 and heads % max(kvh, 1) == 0, f"heads ({heads}) must be a multiple of kv_heads ({kvh})")
        q.require(dim <= 256 and vdim <= 256, f"an attention takes dim and vdim up to 256, got {dim} and {vdim}")
        q.require(taps is None or 1 <= taps <= 9, f"conv must lie in 1..9, got {taps}")
        q.require(window is None or window >= 1, f"mask.size must be at least 1, got {window}")
        q.require(keep is None or keep >= 0, f"mask.keep_first must not be negative, got {keep}")
        q.require(rot is None or (base > 0 and base != 1 and dims % 2 == 0 and 0 < dims <= dim),
                  f"rot.base must be positive and rot.dims even and in (0, dim], got {base} and {dims}")
        return BizepelAttention(heads, kvh, dim, vdim, scale, taps, window, keep or 0, base, dims or 0, v_mix)

    @staticmethod
    def _scan(mx: dict, q: Problems) -> Optional[BizepelScan]:
        vals = [need(mx, key, int, q, required=True) for key in ("inner", "state", "dt_rank", "conv")]
        if q.items:
            return None
        q.require(vals[0] > 0 and vals[2] > 0 and vals[3] >= 1, f"inner, dt_rank and conv must be positive, got {vals}")
        q.require(0 < vals[1] <= 128, f"state must lie in 1..128, got {vals[1]}")
        return BizepelScan(*vals)

    @staticmethod
    def _delta(mx: dict, q: Problems) -> Optional[BizepelDelta]:
        heads = need(mx, "heads", int, q, required=True)
        dim = need(mx, "dim", int, q, required=True)
        rank = need(mx, "rank", int, q, default=0)        # not a key of the format: the tensors' shapes say it
        if q.items:
            return None
        q.require(heads > 0 and 0 < dim <= 256, f"heads must be positive and dim in 1..256, got {heads} and {dim}")
        return BizepelDelta(heads, dim, rank)

    @staticmethod
    def from_dict(raw: dict) -> "BizepelConfig":
        p = Problems("Bizepel config.json")
        V = need(raw, "vocab", int, p, required=True)
        W = need(raw, "width", int, p, required=True)
        norm = need(raw, "norm", dict, p, required=True) or {}
        eps = need(norm, "eps", float, p, required=True)
        canon = need(raw, "canon", dict, p, default=None, allow_none=True)
        taps = need(canon, "taps", int, p, required=True) if canon is not None else None
        side = need(raw, "token_side", dict, p, default=None, allow_none=True)
        side_dim = need(side, "dim", int, p, required=True) if side is not None else None
        logit_scale = need(raw, "logit_scale", float, p, default=1.0)
        layers_raw = need(raw, "layers", list, p, required=True) or []
        p.raise_if_any()
        p.require(V > 0 and W > 0, f"'vocab' and 'width' must be positive, got {V} and {W}")
        p.require(eps > 0, f"'norm.eps' must be positive, got {eps}")
        p.require(taps is None or 1 <= taps <= 9, f"'canon.taps' must lie in 1..9, got {taps}")
        p.require(side_dim is None or side_dim > 0, f"'token_side.dim' must be positive, got {side_dim}")
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
            mlp = BizepelConfig._mlp(mlp_raw, q) if mlp_raw is not None else None
            read = {"attention": BizepelConfig._attention, "mamba1": BizepelConfig._scan,
                    "general_delta": BizepelConfig._delta}.get(typ)
            mixer = None
            if read is None:
                q.add(f"unknown type {typ!r} {TYPES}")
            elif not q.items:
                mixer = read(mx, q)
            layers.append(BizepelLayer(typ, mixer, mlp))
            if q.items:
                p.add(f"layer {i}: " + "; ".join(q.items))
        mixing = [(l.mixer.kv_heads, l.mixer.vdim) for l in layers if isinstance(l.mixer, BizepelAttention) and l.mixer.v_mix]
        p.require(len({g * e for g, e in mixing}) <= 1, f"layers that mix values have the same number of value channels, got {mixing}")
        p.raise_if_any()
        return BizepelConfig(V, W, eps, taps, side_dim, logit_scale, tuple(layers), dict(raw))

    def to_dict(self) -> dict:
        return dict(self.raw)


def _mixer(c: BizepelConfig, l: BizepelLayer, mix: str, lends: bool, takes: bool):
    m = l.mixer
    if l.type == "mamba1":
        return SelectiveScanSpec(
            hidden_size=c.width, inner=m.inner, state=m.state, dt_rank=m.dt_rank, conv_taps=m.taps,
            names={"in": mix + "in", "conv": mix + "conv", "conv_bias": mix + "conv.b", "x": mix + "x", "dt": mix + "dt",
                   "dt_bias": mix + "dt.b", "A_log": mix + "A_log", "D": mix + "D", "o": mix + "o"})
    if l.type == "general_delta":
        return GeneralDeltaSpec(
            hidden_size=c.width, num_heads=m.heads, dim=m.dim, decay_rank=m.rank, eps=c.eps,
            names={"r": mix + "r", "k": mix + "k", "v": mix + "v", "gate": mix + "g", "a": mix + "a", "a_bias": mix + "a.b",
                   "w1": mix + "w1", "w2": mix + "w2", "w0": mix + "w0", "norm": mix + "norm", "o": mix + "o"})
    rotary = (RotarySpec(head_dim=m.dim, rotary_dim=m.rot_dims, theta=m.rot_base, interleaved=True)
              if m.rot_base is not None else NoPositionSpec())
    return AttentionSpec(
        hidden_size=c.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, scale=m.scale, softcap=None,
        window=m.window, position=rotary, names={r: mix + r for r in ("q", "k", "v", "o")}, value_dim=m.vdim,
        q_norm=mix + "q.norm", k_norm=mix + "k.norm", norm_eps=c.eps, biases={r: f"{mix}{r}.b" for r in ("q", "k", "v")},
        keep_first=m.keep if m.window is not None else 0,
        convs={r: f"{mix}{r}.conv" for r in ("q", "k", "v")} if m.taps is not None else None, conv_taps=m.taps or 1,
        lend_values=lends, value_share=(mix + "vmix") if takes else None, wide_weights=WIDE_WEIGHTS)


def _ffn(c: BizepelConfig, m: Optional[BizepelMLP], mlp: str):
    if m is None:
        return None
    if m.kind == "dense":
        return MLPSpec(hidden_size=c.width, intermediate_size=m.ff, activation=DENSE_ACTIVATION,
                       names={"up": mlp + "up", "down": mlp + "down"})
    shared = None
    if m.shared_ff is not None:
        shared = MLPSpec(hidden_size=c.width, intermediate_size=m.shared_ff, activation=EXPERT_ACTIVATION,
                         names={"up": mlp + "shared.up", "down": mlp + "shared.down"})
    return RoutedMLPSpec(
        hidden_size=c.width, intermediate_size=m.ff, num_experts=m.experts, top_k=m.top, activation=EXPERT_ACTIVATION,
        limit=None, router=mlp + "router", expert_names=mlp + "e{e}.{role}", shared=shared, scale_input=False,
        scoring="sigmoid", gated=False, correction=mlp + "correction", groups=m.groups, normalise=True, weight_scale=m.scale)


def bizepel_plan(c: BizepelConfig) -> ModelPlan:
    layers, unused = [], []
    first_mix = None
    for i, l in enumerate(c.layers):
        pre = f"l{i}."
        mix = pre + "mix."
        lends = takes = False
        if l.type == "attention" and l.mixer.v_mix:
            lends, takes = first_mix is None, first_mix is not None
            if lends:
                first_mix = i
                unused.append(mix + "vmix")          # a checkpoint may hold the first layer's share
        ffn = _ffn(c, l.mlp, pre + "mlp.")
        norms = {"pre_mixer": LayerNormSpec(c.width, c.eps, pre + "norm1", None)}
        filters, scales = {}, {"mixer": pre + "ls1"}
        if c.taps is not None:
            filters["pre_mixer"] = ShortConvSpec(c.width, c.taps, pre + "canon1")
        if ffn is not None:
            norms["pre_ffn"] = LayerNormSpec(c.width, c.eps, pre + "norm2", None)
            scales["ffn"] = pre + "ls2"
            if c.taps is not None:
                filters["pre_ffn"] = ShortConvSpec(c.width, c.taps, pre + "canon2")
        else:
            unused += [pre + "norm2", pre + "ls2", pre + "canon2"]
        side = None
        if c.side_dim is not None:
            side = TokenSideSpec(dim=c.side_dim, column=i * c.side_dim, vocab_size=c.vocab,
                                 table_columns=len(c.layers) * c.side_dim, eps=c.eps,
                                 names={"table": "side.embed", "gate": pre + "side.gate", "proj": pre + "side.proj",
                                        "norm": pre + "side.norm"})
        layers.append(FilteredBlockSpec(mixer=_mixer(c, l, mix, lends, takes), ffn=ffn, norms=norms, filters=filters,
                                        scales=scales, side=side))
    return ModelPlan(
        architecture=NAME, hidden_size=c.width, vocab_size=c.vocab, max_position=MAX_POSITION,
        embedding=EmbeddingSpec(c.vocab, c.width, 1.0, "embed", norm=LayerNormSpec(c.width, c.eps, "embed.norm", None)),
        layers=tuple(layers), order=tuple(LayerCall(i) for i in range(len(layers))),
        # the logits are linear in the last norm's result: their factor rides in its gain, in floats
        final_norm=LayerNormSpec(c.width, c.eps, "final.norm", None, gain_scale=c.logit_scale),
        head=HeadSpec(c.vocab, c.width, None, "embed"),
        ignored_tensors=tuple(unused), optional_prefixes=())


BIZEPEL = register_architecture(Architecture(
    name=NAME, config_from_dict=BizepelConfig.from_dict, plan=bizepel_plan, model_types=("bizepel",)))
