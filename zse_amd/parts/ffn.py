"""Gated feed-forward: act(x Wg^T) * (x Wu^T), then Wd^T.

act is one of gelu_tanh, silu and relu (max(z, 0)).
gelu_tanh(z) = 0.5 z (1 + tanh(sqrt(2/pi) (z + 0.044715 z^3))) is the
reference's GeGLU kernel (orchestrator/kernels.py:1678-1697, wiring
model_runner.py:518-530); silu is its Llama activation (kernels.py:228-244).
Gate and up are two products there (model_runner.py:1270-1275), one here.
"""
from __future__ import annotations

from typing import List

from ..runtime.device import BF16, F32, I32, Tensor
from .base import ROLE_GAIN, Part, TensorReq, build_part, register_part
from .ops import linear, tuned_gemm

ACTIVATION_CODES = {"gelu_tanh": 0, "silu": 1, "relu": 2}
CLAMPED = "clamped_swiglu"     # g = min(gate, limit), u = clamp(up, +-limit): g sigmoid(1.702 g) (u + 1)


class GatedMLP(Part):
    graph_safe = True      # its launches take what changes from step to step from device memory alone

    def __init__(self, spec):
        if spec.activation not in ACTIVATION_CODES and spec.activation != CLAMPED:
            raise ValueError(f"activation must be one of {sorted(ACTIVATION_CODES) + [CLAMPED]}, got {spec.activation!r}")
        if spec.activation == CLAMPED and not (getattr(spec, "limit", None) or 0) > 0:
            raise ValueError(f"{CLAMPED} needs a positive limit, got {getattr(spec, 'limit', None)!r}")
        self.spec = spec
        self.w_gu = self.w_down = None

    def tensor_reqs(self) -> List[TensorReq]:
        s = self.spec
        return [TensorReq(s.names["gate"], (s.intermediate_size, s.hidden_size)),
                TensorReq(s.names["up"], (s.intermediate_size, s.hidden_size)),
                TensorReq(s.names["down"], (s.hidden_size, s.intermediate_size))]

    def load(self, weights, rt, dtype):
        s = self.spec
        strip = getattr(weights, "wants_strip", None)
        gu = [s.names["gate"], s.names["up"]]
        self.w_gu = (weights.matrix(gu, strip=True) if strip and strip(s.hidden_size, s.intermediate_size)
                     else weights.matrix(gu))
        self.w_down = (weights.matrix([s.names["down"]], strip=True) if strip and strip(s.intermediate_size)
                       else weights.matrix([s.names["down"]]))

    def forward(self, ctx, x: Tensor, out: Tensor = None) -> Tensor:
        """``out``: where the result goes (activations or float32 [T, hidden]); the product that
        ends the layer then never hands partial sums back."""
        s = self.spec
        T, I = x.shape[0], s.intermediate_size
        last = None if out is not None else self
        if s.activation == CLAMPED and tuned_gemm(ctx, s.hidden_size):
            # the activation in the product's epilogue, on the float sums
            a = linear(ctx, x, self.w_gu, ctx.alloc((T, I)), epilogue=CLAMPED, cap=float(s.limit))
            return linear(ctx, a, self.w_down, out if out is not None else ctx.alloc((T, s.hidden_size)), last_of=last)
        if s.activation == CLAMPED:
            gu = linear(ctx, x, self.w_gu, ctx.alloc((T, 2 * I)))
            a = ctx.alloc((T, I))
            ctx.k.zk_clamped_glu(gu.ptr, a.ptr, T, I, float(s.limit), ctx.stream)
            return linear(ctx, a, self.w_down, out if out is not None else ctx.alloc((T, s.hidden_size)), last_of=last)
        if tuned_gemm(ctx, s.hidden_size):
            a = linear(ctx, x, self.w_gu, ctx.alloc((T, I)), epilogue=s.activation)
            return linear(ctx, a, self.w_down, out if out is not None else ctx.alloc((T, s.hidden_size)), last_of=last)
        gu = linear(ctx, x, self.w_gu, ctx.alloc((T, 2 * I)))
        a = ctx.alloc((T, I))
        ctx.k.zk_gated_act(gu.ptr, a.ptr, T, I, ACTIVATION_CODES[s.activation], ctx.stream)
        return linear(ctx, a, self.w_down, out if out is not None else ctx.alloc((T, s.hidden_size)), last_of=last)


UNARY_CODES = {"relu2": 0, "gelu": 1}     # max(z, 0)^2;  z (1 + erf(z / sqrt(2))) / 2


class MLP(Part):
    """act(x Wu^T) Wd^T without a gate; the activation rides in the first product's epilogue where
    the matrix-core product serves the step."""
    graph_safe = True      # its launches take what changes from step to step from device memory alone

    def __init__(self, spec):
        if spec.activation not in UNARY_CODES:
            raise ValueError(f"activation must be one of {sorted(UNARY_CODES)}, got {spec.activation!r}")
        self.spec = spec
        self.w_up = self.w_down = None

    def tensor_reqs(self) -> List[TensorReq]:
        s = self.spec
        return [TensorReq(s.names["up"], (s.intermediate_size, s.hidden_size)),
                TensorReq(s.names["down"], (s.hidden_size, s.intermediate_size))]

    def load(self, weights, rt, dtype):
        s = self.spec
        strip = getattr(weights, "wants_strip", None)
        self.w_up = weights.matrix([s.names["up"]], strip=bool(strip and strip(s.hidden_size)))
        self.w_down = weights.matrix([s.names["down"]], strip=bool(strip and strip(s.intermediate_size)))

    def forward(self, ctx, x: Tensor, out: Tensor = None) -> Tensor:
        """``out``: where the result goes (activations or float32 [T, hidden]); the product that
        ends the layer then never hands partial sums back."""
        s = self.spec
        T, I = x.shape[0], s.intermediate_size
        if tuned_gemm(ctx, s.hidden_size) and x.ptr % 16 == 0:
            a = linear(ctx, x, self.w_up, ctx.alloc((T, I)), epilogue=s.activation)
        else:
            up = linear(ctx, x, self.w_up, ctx.alloc((T, I)))
            a = ctx.alloc((T, I))
            ctx.k.zk_unary_act(up.ptr, a.ptr, T * I, UNARY_CODES[s.activation], ctx.stream)
        return linear(ctx, a, self.w_down, out if out is not None else ctx.alloc((T, s.hidden_size)),
                      last_of=None if out is not None else self)


class RoutedMLP(Part):
    """A mixture of small layers (gated, or without a gate): scores from a float router product (sigmoids, or a softmax
    over all experts), the ``top_k`` largest chosen on the device (the lower index among equals;
    optionally by score plus a correction, among the experts of the best groups only; some of the numbers
    to choose from may stand for identity experts, which have no weights and give their input back),
    the chosen scores as weights on the experts' inputs or on their outputs, the experts' results
    added in the order they were chosen, a shared layer on top (optionally times the sigmoid of a
    number a token, whose row rides below the router's in one product).  In bfloat16 the (token, choice) pairs are sorted by
    expert on the device and a grouped matrix-core product runs over each expert's rows, whatever their number; in
    32-bit, and where a width is no multiple of eight, each chosen expert's rows are read once per pair.
    Nothing comes back to the host, so steps are captured and written down like any other."""
    graph_safe = True

    def __init__(self, spec):
        s = self.spec = spec
        self.gated = bool(getattr(s, "gated", True))
        if not self.gated and (s.activation != "relu2" or s.scale_input):
            raise ValueError(f"experts without a gate are relu2 layers with weights on their results, got {s.activation!r}")
        self.correction_name = getattr(s, "correction", None)
        self.groups = tuple(getattr(s, "groups", None) or (1, 1))
        self.group_best = int(getattr(s, "group_best", 2))
        self.identity = int(getattr(s, "identity", 0) or 0)
        n = self.choices = s.num_experts + self.identity          # what the router chooses from
        if self.identity < 0 or s.num_experts < 1:
            raise ValueError(f"at least one expert and no fewer than 0 identity experts, got {s.num_experts} and {self.identity}")
        if n % self.groups[0] or not (1 <= self.groups[1] <= self.groups[0]) or \
                self.groups[1] * (n // self.groups[0]) < s.top_k:
            raise ValueError(f"equal groups of experts of which enough stay for {s.top_k} choices, got {n} "
                             f"experts in {self.groups[0]} groups, {self.groups[1]} kept")
        if self.group_best not in (1, 2):
            raise ValueError(f"a group is judged by its one or two best scores, got {self.group_best}")
        # a choice by anything but the scores alone, or weights that are not the scores: the wider router kernel
        self.wide_route = bool(self.correction_name or self.groups != (1, 1) or getattr(s, "normalise", False)
                               or getattr(s, "weight_scale", 1.0) != 1.0)
        self.correction = None
        if self.gated and s.activation not in (CLAMPED, "silu"):
            raise ValueError(f"routed experts are {CLAMPED} or silu layers, got {s.activation!r}")
        if not (1 <= s.top_k <= min(n, 16)) or n > 1024:
            raise ValueError(f"1 to 16 of up to 1024 experts a token, got {s.top_k} of {n}")
        if s.activation == CLAMPED and not (s.limit or 0) > 0:
            raise ValueError(f"{CLAMPED} needs a positive limit, got {s.limit!r}")
        self.scoring = getattr(s, "scoring", "sigmoid")
        if self.scoring not in ("sigmoid", "softmax"):
            raise ValueError(f"scores are sigmoid or softmax, got {self.scoring!r}")
        self.shared = build_part("ffn", s.shared) if s.shared is not None else None
        self.shared_gate = getattr(s, "shared_gate", None)
        if self.shared_gate and self.shared is None:
            raise ValueError("a gate on the shared layer needs a shared layer")
        self.w_router = self.w_gu = self.w_down = None

    def children(self):
        return [self.shared] if self.shared is not None else []

    def _name(self, e: int, role: str) -> str:
        return self.spec.expert_names.format(e=e, role=role)

    def tensor_reqs(self) -> List[TensorReq]:
        s = self.spec
        out = [TensorReq(s.router, (self.choices, s.hidden_size))]
        if self.shared_gate:
            out.append(TensorReq(self.shared_gate, (1, s.hidden_size)))
        if self.correction_name:
            out.append(TensorReq(self.correction_name, (self.choices,), ROLE_GAIN))
        for e in range(s.num_experts):
            if self.gated:
                out.append(TensorReq(self._name(e, "gate"), (s.intermediate_size, s.hidden_size)))
            out += [TensorReq(self._name(e, "up"), (s.intermediate_size, s.hidden_size)),
                    TensorReq(self._name(e, "down"), (s.hidden_size, s.intermediate_size))]
        return out

    def load(self, weights, rt, dtype):
        s = self.spec
        self.w_router = weights.matrix([s.router] + ([self.shared_gate] if self.shared_gate else []))
        # expert e: rows [e 2F, e 2F + F) its gate, the next F its up (without a gate: F rows an expert); down: rows
        # [e W, (e + 1) W)
        roles = ("gate", "up") if self.gated else ("up",)
        self.w_gu = weights.matrix([self._name(e, r) for e in range(s.num_experts) for r in roles])
        self.correction = weights.vector(self.correction_name) if self.correction_name else None
        self.w_down = weights.matrix([self._name(e, "down") for e in range(s.num_experts)])

    def flops_per_token(self) -> float:
        # (with identity experts: as many experts at work as an even choice gives)
        s = self.spec
        at_work = s.top_k * s.num_experts / self.choices
        return 2.0 * self.choices * s.hidden_size + at_work * (6.0 if self.gated else 4.0) * s.intermediate_size * s.hidden_size

    def forward(self, ctx, x: Tensor) -> Tensor:
        s, k = self.spec, ctx.k
        T, W, F, E, top = x.shape[0], s.hidden_size, s.intermediate_size, s.num_experts, s.top_k
        n = self.choices
        ld = n + (1 if self.shared_gate else 0)
        logits = linear(ctx, x, self.w_router, ctx.alloc((T, ld), F32))
        ids, wts = ctx.alloc((T, top), I32), ctx.alloc((T, top), F32)
        softmax = 1 if self.scoring == "softmax" else 0
        if self.wide_route:
            k.zk_moe_route_best(logits.ptr, ld, self.correction.ptr if self.correction is not None else None, ids.ptr, wts.ptr,
                                T, n, top, self.groups[0], self.groups[1], softmax, 1 if getattr(s, "normalise", False) else 0,
                                float(getattr(s, "weight_scale", 1.0)), self.group_best, ctx.stream)
        else:
            k.zk_moe_route_ext(logits.ptr, ld, ids.ptr, wts.ptr, T, n, top, softmax, ctx.stream)
        act, on_out, limit = (2 if not self.gated else 1 if s.activation == "silu" else 0), (0 if s.scale_input else 1), float(s.limit or 0.0)
        # the shared layer's rows first: what adds up the chosen experts' results takes them in, with their gate
        add = gate = None
        if self.shared is not None:
            add = self.shared.forward(ctx, x, out=ctx.alloc((T, W), F32)).ptr
            gate = logits.ptr + n * 4 if self.shared_gate else None
        plane = ctx.alloc((1, T, W), F32)
        y = ctx.alloc((T * top, F))
        # (measured with six layers of 8 experts, 2 a token: 0.87 -> 0.66 ms a decode step of one request at
        # 2048 x 2048, 0.51 -> 0.46 at 1024 x 1024, and more with more requests)
        grouped = (ctx.dtype == BF16 and ctx.tuned and W % 8 == 0 and F % 8 == 0 and x.ptr % 16 == 0
                   and k.has("zk_moe_experts_grouped_identity"))
        if grouped:
            work = ctx.alloc((n + 1 + 2 * T * top,), I32)
            xg = ctx.alloc((T * top, W)).ptr if s.scale_input else None
            rows = ctx.alloc((T * top, W), F32)
            k.zk_moe_experts_grouped_identity(x.ptr, ids.ptr, wts.ptr, self.w_gu.ptr, self.w_down.ptr, work.ptr, xg, y.ptr,
                                              rows.ptr, plane.ptr, T, E, top, W, F, limit, act, on_out, self.identity, add, gate, ld,
                                              ctx.stream)
        else:
            k.zk_moe_experts_identity(x.ptr, ids.ptr, wts.ptr, self.w_gu.ptr, self.w_down.ptr, y.ptr, plane.ptr, T, top, W, F,
                                      limit, act, on_out, E, add, gate, ld, ctx.stream)
        if getattr(ctx, "sums_welcome", None) is self:
            # the block's joining kernel takes the float rows as they are
            return Tensor(plane.ptr, (1, T, W), F32, plane.owner, layout="parts")
        out = ctx.alloc((T, W))
        k.zk_planes_sum(plane.ptr, 1, out.ptr, T, W, ctx.stream)
        return out


register_part("ffn", "gated_mlp", GatedMLP)
register_part("ffn", "mlp", MLP)
register_part("ffn", "routed_mlp", RoutedMLP)
