"""A recurrent mixer with a matrix state per head, written by the generalized delta rule.

Per head, D channels of keys and of values; the state S [D, D] starts at zero and is carried as
floats in the request's state slot:

    r = W_r x,   k = W_k x,   v = W_v x,   u = k / sqrt(sum k^2 + 1e-6)            (per head)
    w = exp(-exp(-1/2) sigmoid(W_w2 tanh(W_w1 x) + w0)),   a = sigmoid(W_a x + b)  (per key channel, float)
    S <- diag(w) S - (a u)(u^T S) + k v^T;   o = S^T r                             (both terms from the old S)
    out = W_o ( o / sqrt(mean(o^2) + eps) * gain * sigmoid(W_g x) )                (the mean per head)

r, k, v and the gate are one product; a and the narrow W_w1 a second one whose results stay floats.
One small kernel makes w and a of the step's tokens (tanh, W_w2, sigmoids and the exponential in
floats).  Portions of prompts run in chunks of 32 tokens on the 32-bit matrix cores, short ones token by
token, single tokens in a kernel of their own; the 32-bit library has the walk token by token alone,
so a request's values there are the same bits however its tokens are cut.
"""
from __future__ import annotations

from typing import List

from ..runtime.device import BF16, F32, ITEMSIZE, Tensor
from .base import ROLE_GAIN, Part, StateNeed, TensorReq, register_part
from .ops import linear


class GeneralDelta(Part):
    graph_safe = True      # rows, requests and slots are read by the kernels from device memory
    CHUNKED_FROM = 16      # tokens of a step's longest portion from which the chunks are used (bfloat16)
    WORK_BYTES = 96 << 20  # of operands at a time: what the last-level cache keeps until they are read

    def __init__(self, spec):
        s = self.spec = spec
        if s.dim > 256 or s.dim < 1 or s.num_heads < 1:
            raise ValueError(f"heads of 1 to 256 channels, got {s.num_heads} of {s.dim}")
        if s.decay_rank < 0:
            raise ValueError(f"the decays' rank must not be negative, got {s.decay_rank}")
        self.rank = int(s.decay_rank)          # 0: the checkpoint's tensors say it, at load
        self.width = s.num_heads * s.dim
        self.w_in = self.w_aw = self.w_w2 = self.w_o = self.a_bias = self.w0 = self.gain = None

    def tensor_reqs(self) -> List[TensorReq]:
        s, n, W, C = self.spec, self.spec.names, self.spec.hidden_size, self.width
        rank = s.decay_rank or -1
        return [TensorReq(n["r"], (C, W)), TensorReq(n["k"], (C, W)), TensorReq(n["v"], (C, W)), TensorReq(n["gate"], (C, W)),
                TensorReq(n["a"], (C, W)), TensorReq(n["a_bias"], (C,), ROLE_GAIN), TensorReq(n["w1"], (rank, W)),
                TensorReq(n["w2"], (C, rank)), TensorReq(n["w0"], (C,), ROLE_GAIN), TensorReq(n["norm"], (C,), ROLE_GAIN),
                TensorReq(n["o"], (W, C))]

    def load(self, weights, rt, dtype):
        s, n = self.spec, self.spec.names
        self.rank = weights.shape_of(n["w1"])[0]
        if weights.shape_of(n["w2"])[1] != self.rank:
            raise ValueError(f"{n['w2']} has {weights.shape_of(n['w2'])[1]} columns, {n['w1']} {self.rank} rows")
        if self.rank > 1024:
            raise ValueError(f"the decays' rank up to 1024, got {self.rank}")
        strip = getattr(weights, "wants_strip", None)
        wide = bool(strip and strip(s.hidden_size))
        self.w_in = weights.matrix([n["r"], n["k"], n["v"], n["gate"]], strip=wide)
        self.w_aw = weights.matrix([n["a"], n["w1"]], strip=wide)
        self.w_w2 = weights.matrix([n["w2"]])
        self.w_o = weights.matrix([n["o"]], strip=bool(strip and strip(self.width)))
        self.a_bias, self.w0, self.gain = weights.vector(n["a_bias"]), weights.vector(n["w0"]), weights.vector(n["norm"])

    def state_words(self) -> int:
        return self.width * self.spec.dim

    def cache_need(self):
        return StateNeed(self.state_words() * 4)

    def flops_per_token(self) -> float:
        s, W, C = self.spec, self.spec.hidden_size, self.width
        return 2.0 * (W * (5 * C + self.rank) + self.rank * C + C * W) + 8.0 * s.num_heads * s.dim * s.dim

    def forward(self, ctx, x: Tensor, cache) -> Tensor:
        s, k = self.spec, ctx.k
        T, C, H, D = x.shape[0], self.width, s.num_heads, s.dim
        ld, lda = 4 * C, C + self.rank
        rows = linear(ctx, x, self.w_in, ctx.alloc((T, ld)))
        low = linear(ctx, x, self.w_aw, ctx.alloc((T, lda), F32))
        decay, rate = ctx.alloc((T, C), F32), ctx.alloc((T, C), F32)
        k.zk_gdelta_gates(low.ptr, lda, C, self.rank, self.w_w2.ptr, self.w0.ptr, self.a_bias.ptr, decay.ptr, rate.ptr, T, C,
                          ctx.stream)
        out = ctx.alloc((T, C))
        gate = rows.ptr + 3 * C * ITEMSIZE[ctx.dtype]
        place = (ctx.state.ptr, ctx.state.shape[1], cache.state_offset // 4)
        if ctx.dtype == BF16 and ctx.tuned and ctx.max_q_len == 1 and T == ctx.R and k.zk_gdelta_token_supports(D):
            k.zk_gdelta_token(rows.ptr, ld, C, 2 * C, gate, ld, decay.ptr, rate.ptr, self.gain.ptr, *place, ctx.positions,
                              ctx.req_of_token, ctx.slot_of_req, out.ptr, T, H, D, float(s.eps), ctx.stream)
        elif ctx.dtype == BF16 and ctx.tuned and ctx.max_q_len >= self.CHUNKED_FROM and k.zk_gdelta_chunk_floats(D):
            raw = ctx.alloc((T, C), F32)
            # the operands of as many chunks of every request as WORK_BYTES hold (one at least)
            chunk = ctx.R * H * k.zk_gdelta_chunk_floats(D)
            count = max(1, min(-(-int(ctx.max_q_len) // 32), self.WORK_BYTES // (4 * chunk)))
            work = ctx.alloc((count * chunk,), F32)
            k.zk_gdelta_chunked(rows.ptr, ld, C, 2 * C, gate, ld, decay.ptr, rate.ptr, self.gain.ptr, *place, ctx.q_start,
                                ctx.slot_of_req, ctx.positions, out.ptr, raw.ptr, work.ptr, count * chunk, T, ctx.R,
                                int(ctx.max_q_len), H, D, float(s.eps), ctx.stream)
        else:
            raw = ctx.alloc((T, C), F32)
            k.zk_gdelta(rows.ptr, ld, C, 2 * C, gate, ld, decay.ptr, rate.ptr, self.gain.ptr, *place, ctx.q_start,
                        ctx.slot_of_req, ctx.positions, out.ptr, raw.ptr, T, ctx.R, int(ctx.max_q_len), H, D, float(s.eps),
                        ctx.stream)
        return linear(ctx, out, self.w_o, ctx.alloc((T, s.hidden_size)), last_of=self)


register_part("mixer", "general_delta", GeneralDelta)
