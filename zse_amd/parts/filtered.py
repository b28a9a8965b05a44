"""A pre-norm layer whose sublayers read their norm through a short convolution over time:

    h += s1 * mixer(f1(norm1(h)));   h += s2 * ffn(f2(norm2(h)))          f(n)_t = n_t + conv(n)_t
    h += rms(W_proj (gelu_tanh(W_gate h) * e)) * gain                    e: the layer's part of the token's row of a table

Each of the filters, the scales (a gain per channel), the feed-forward and the token's input may be
absent.  One kernel adds a sublayer's result to the float stream and makes the next sublayer's
input, also across the boundary to the next layer; in steps of single tokens the convolution
and the renewal of its state ride in the same launch, otherwise the convolution's own kernel
follows.  What the filters keep per request lies in the layer's part of the state slot.
"""
from __future__ import annotations

from typing import List

from ..runtime.device import F32, Tensor
from .base import ROLE_GAIN, Part, TensorReq, build_part, register_part
from .norm import LayerNorm
from .ops import linear


class TokenSide(Part):
    """The products and the gate of a layer's token input; the block adds the result to the stream
    (unit root mean square and gain are the joining kernel's)."""
    graph_safe = True      # tokens are read by the kernels from device memory

    def __init__(self, spec):
        if not (spec.dim >= 1 and 0 <= spec.column <= spec.table_columns - spec.dim):
            raise ValueError(f"columns [{spec.column}, {spec.column + spec.dim}) of a table of {spec.table_columns}")
        self.spec = spec
        self.size = None             # the stream's width, set by the block
        self.table = self.w_gate = self.w_proj = self.gain = None

    def tensor_reqs(self) -> List[TensorReq]:
        s, n = self.spec, self.spec.names
        return [TensorReq(n["table"], (s.vocab_size, s.table_columns)), TensorReq(n["gate"], (s.dim, self.size)),
                TensorReq(n["proj"], (self.size, s.dim)), TensorReq(n["norm"], (self.size,), ROLE_GAIN)]

    def load(self, weights, rt, dtype):
        s, n = self.spec, self.spec.names
        strip = getattr(weights, "wants_strip", None)
        self.table = weights.matrix([n["table"]])                       # row-major: rows are gathered; shared by the layers
        self.w_gate = weights.matrix([n["gate"]], strip=bool(strip and strip(self.size)))
        self.w_proj = weights.matrix([n["proj"]], strip=bool(strip and strip(s.dim)))
        self.gain = weights.vector(n["norm"])

    def flops_per_token(self) -> float:
        return 4.0 * self.spec.dim * self.size      # gate and projection; the table's row is gathered

    def forward(self, ctx, x: Tensor) -> Tensor:
        """``x``: the stream in the activation type; what comes back is W_proj(...) before its norm."""
        s = self.spec
        T = x.shape[0]
        z = linear(ctx, x, self.w_gate, ctx.alloc((T, s.dim), F32))
        g = ctx.alloc((T, s.dim))
        ctx.k.zk_token_gate(z.ptr, self.table.ptr, ctx.tokens, s.table_columns, s.column, g.ptr, T, s.dim, ctx.stream)
        return linear(ctx, g, self.w_proj, ctx.alloc((T, self.size)), sums_ok=True)


class FilteredBlock(Part):
    graph_safe = True      # its launches take what changes from step to step from device memory alone
    SUBLAYERS = ("pre_mixer", "pre_ffn")

    def __init__(self, spec):
        self.spec = spec
        self.norms = {"pre_mixer": build_part("norm", spec.norms["pre_mixer"])}
        self.mixer = build_part("mixer", spec.mixer)
        self.ffn = build_part("ffn", spec.ffn) if spec.ffn is not None else None
        if self.ffn is not None:
            self.norms["pre_ffn"] = build_part("norm", spec.norms["pre_ffn"])
        for n in self.norms.values():
            if not isinstance(n, LayerNorm) or n.spec.streams != 1:
                raise ValueError("a filtered block reads one stream through layer norms")
        self.size = self.norms["pre_mixer"].spec.size
        self.filters = {}
        for role in self.norms:
            f = spec.filters.get(role)
            if f is None:
                continue
            if f.size != self.size or not f.residual or f.activation or f.bias or f.in_bias:
                raise ValueError("a block's filter adds a plain convolution of all its channels to its input")
            self.filters[role] = build_part("filter", f)
        self.scale_names = {r: n for r, n in (spec.scales or {}).items() if r == "mixer" or self.ffn is not None}
        self.scales = {}
        self.side = None
        if spec.side is not None:
            self.side = TokenSide(spec.side)
            self.side.size = self.size

    def children(self):
        out = list(self.norms.values()) + [self.mixer] + ([self.ffn] if self.ffn is not None else [])
        return out + list(self.filters.values()) + ([self.side] if self.side is not None else [])

    def tensor_reqs(self) -> List[TensorReq]:
        return [TensorReq(n, (self.size,), ROLE_GAIN) for n in self.scale_names.values()]

    def load(self, weights, rt, dtype):
        self.scales = {r: weights.vector(n) for r, n in self.scale_names.items()}

    def state_needs(self):
        return [(role, f.state_bytes()) for role, f in self.filters.items() if f.state_bytes()]

    def entry_norm(self):
        """What the layer before needs to make this one's first input in the kernel that ends its own
        work: this block (its first norm and filter); the place of the filter's state comes with
        the call (``model.forward`` hands the next entry's cache along in ``ctx.next_cache``)."""
        return self

    def _join(self, ctx, h: Tensor, y, gain, unit, reader, role, cache, raw=None, out=None):
        """h += y (times ``gain``; ``unit``: (eps) y is brought to unit root mean square first), then the
        input of ``reader``'s sublayer ``role`` (None: no read), whose filter's state lies in ``cache``."""
        T, W = h.shape
        ptr = lambda t: t.ptr if t is not None else None
        norm = reader.norms[role] if reader is not None else None
        filt = reader.filters.get(role) if reader is not None else None
        if norm is not None:
            out = ctx.alloc((T, W)) if out is None else Tensor(out.ptr, (T, W), ctx.dtype, out.owner)
        parts = y.shape[0] if (y is not None and y.layout == "parts") else 0
        offset = cache.extra[role][0] if (filt is not None and role in cache.extra) else 0
        single = ctx.max_q_len == 1 and T == ctx.R       # every request brings one token
        fused = filt is not None and single
        made = out
        if norm is not None and filt is not None and not fused:
            made = ctx.alloc((T, W))                     # the norm alone; the convolution follows
        state = ctx.state.ptr if (fused and ctx.state is not None) else None
        ctx.k.zk_sublayer_step(
            h.ptr, ptr(y), parts, ptr(gain), 0 if unit is None else 1, float(unit or 0.0), ptr(raw),
            ptr(norm.weight) if norm is not None else None, ptr(norm.bias) if norm is not None else None,
            float(norm.spec.eps) if norm is not None else 0.0, ptr(made) if norm is not None else None,
            ptr(filt.weight) if fused else None, filt.spec.taps if fused else 0, state,
            ctx.state.shape[1] if state else 0, offset // 4, ctx.positions, ctx.req_of_token, ctx.slot_of_req, T, W, ctx.stream)
        if norm is None:
            return None
        if filt is not None and not fused:
            out = filt.forward(ctx, made, offset, out=out)
        return out

    def forward(self, ctx, h: Tensor, cache, x_in: Tensor = None, next_norm=None, x_out: Tensor = None):
        """Update the stream ``h`` in place.  ``x_in``: this block's first input, if the caller has it.
        ``next_norm``: the block that runs next (its ``entry_norm()``); its first input is returned,
        made by the kernel that joins this block's last result."""
        x = x_in if x_in is not None else self._join(ctx, h, None, None, None, self, "pre_mixer", cache)
        nxt = next_norm if (isinstance(next_norm, FilteredBlock) and next_norm.size == self.size) else None
        ctx.sums_welcome = self.mixer          # the joining kernel adds partial sums up itself
        y, gain = self.mixer.forward(ctx, x, cache), self.scales.get("mixer")
        if self.ffn is not None:
            x = self._join(ctx, h, y, gain, None, self, "pre_ffn", cache)
            ctx.sums_welcome = self.ffn
            y, gain = self.ffn.forward(ctx, x), self.scales.get("ffn")
        ctx.sums_welcome = None
        unit = None
        if self.side is not None:
            raw = ctx.alloc(h.shape)
            self._join(ctx, h, y, gain, None, None, None, cache, raw=raw)
            y, gain, unit = self.side.forward(ctx, raw), self.side.gain, self.side.spec.eps
        return self._join(ctx, h, y, gain, unit, nxt, "pre_mixer", ctx.next_cache, out=x_out)


register_part("block", "filtered", FilteredBlock)
