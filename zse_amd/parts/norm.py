"""Root-mean-square norm, gain (1 + w) or w; layer norm with gain and bias; no norm.

Statistics and the product are float; rsqrt(mean(x^2) + eps) as in the
reference's kernel (orchestrator/kernels.py:1435-1465); the reference multiplies
by plain w and names the (1 + w) form of Gemma 2 in a comment (:1476-1478).
"""
from __future__ import annotations

from dataclasses import replace
from typing import List, Optional

import numpy as np

from ..runtime.device import F32, Tensor
from .base import ROLE_GAIN, Part, TensorReq, register_part


class RMSNorm(Part):
    graph_safe = True      # its launches take what changes from step to step from device memory alone

    def __init__(self, spec):
        self.spec = self.given = spec
        self.weight: Optional[Tensor] = None

    def tensor_reqs(self) -> List[TensorReq]:
        return [TensorReq(self.spec.weight, (self.spec.size,), ROLE_GAIN)]

    def load(self, weights, rt, dtype):
        s = self.given
        self.weight = weights.vector(s.weight)
        scale = float(getattr(s, "gain_scale", 1.0))
        if scale != 1.0:
            # the whole gain, as the kernels see it from now on
            gain = rt.download(self.weight) + np.float32(1.0 if s.unit_offset else 0.0)
            self.weight = rt.upload((gain * np.float32(scale)).astype(np.float32))
            self.spec = replace(s, unit_offset=False, gain_scale=1.0)

    def forward(self, ctx, x: Tensor, out_rows=None) -> Tensor:
        """Norm of every row of ``x`` (float stream or activations), or of the rows
        ``out_rows = (device int32 pointer, count)``."""
        s = self.spec
        rows_ptr, n = (out_rows if out_rows is not None else (0, x.shape[0]))
        out = ctx.alloc((n, s.size))
        ctx.k.zk_rmsnorm(x.ptr, 1 if x.dtype == F32 else 0,
                         rows_ptr or None, self.weight.ptr, out.ptr, s.eps,
                         1 if s.unit_offset else 0, n, s.size, ctx.stream)
        return out


class LayerNorm(Part):
    """(x - mean) / sqrt(var + eps) * gain + bias over the float residual; with several residual
    streams a token the norm reads their plain sum."""
    graph_safe = True      # its launches take what changes from step to step from device memory alone

    def __init__(self, spec):
        if not (1 <= spec.streams <= 8):
            raise ValueError(f"a layer norm reads 1 to 8 streams, got {spec.streams}")
        self.spec = spec
        self.weight: Optional[Tensor] = None
        self.bias: Optional[Tensor] = None

    def tensor_reqs(self) -> List[TensorReq]:
        s = self.spec
        out = [TensorReq(s.weight, (s.size,), ROLE_GAIN)]
        if s.bias:
            out.append(TensorReq(s.bias, (s.size,), ROLE_GAIN))
        return out

    def load(self, weights, rt, dtype):
        self.weight = weights.vector(self.spec.weight)
        self.bias = weights.vector(self.spec.bias) if self.spec.bias else None
        scale = float(getattr(self.spec, "gain_scale", 1.0))
        if scale != 1.0:
            self.weight = rt.upload((rt.download(self.weight) * np.float32(scale)).astype(np.float32))
            if self.bias is not None:
                self.bias = rt.upload((rt.download(self.bias) * np.float32(scale)).astype(np.float32))

    def in_place(self, ctx, x: Tensor) -> None:
        """The float rows ``x`` replaced by their norm, not rounded."""
        s = self.spec
        if x.dtype != F32 or s.streams != 1 or x.shape[1] != s.size:
            raise ValueError(f"a layer norm in place over float rows of {s.size}: got {x.dtype} {x.shape}")
        ctx.k.zk_norm_stream(x.ptr, self.weight.ptr, self.bias.ptr if self.bias is not None else None, float(s.eps),
                             x.shape[0], s.size, ctx.stream)

    def forward(self, ctx, x: Tensor, out_rows=None) -> Tensor:
        s = self.spec
        if x.dtype != F32 or x.shape[1] != s.streams * s.size:
            raise ValueError(f"layer norm over {s.streams} float streams of {s.size}: got {x.dtype} {x.shape}")
        rows_ptr, n = (out_rows if out_rows is not None else (0, x.shape[0]))
        out = ctx.alloc((n, s.size))
        ctx.k.zk_streams_step(x.ptr, s.streams, None, 0, None, None, None, self.weight.ptr,
                              self.bias.ptr if self.bias is not None else None, s.eps, rows_ptr or None, out.ptr, n,
                              x.shape[0], s.size, ctx.stream)
        return out


class NoNorm(Part):
    """Stands where a sublayer reads the stream itself: its rows in the activation type."""
    graph_safe = True      # its launches take what changes from step to step from device memory alone

    def __init__(self, spec):
        self.spec = spec

    def forward(self, ctx, x: Tensor, out_rows=None) -> Tensor:
        if x.dtype != F32 or out_rows is not None:
            raise ValueError(f"all rows of the float stream, got {x.dtype} {x.shape}")
        out = ctx.alloc(x.shape)
        ctx.k.zk_round_rows(x.ptr, out.ptr, x.numel, ctx.stream)
        return out


register_part("norm", "rmsnorm", RMSNorm)
register_part("norm", "none", NoNorm)
register_part("norm", "layernorm", LayerNorm)
