"""RMS norm, fused with the pending add into the float32 residual stream.

y = v / sqrt(mean(v^2) + eps) * w with v = x + delta (+ delta_bias); the sum of
squares and the product are float32 and the result is rounded once. The
reference calls its norm before attention, before the feed-forward and on the
gathered output rows (models/llama/common/src/compute.rs:206-207,
:274-275, :358-363) and keeps x for the residual (:169, x1 is a separate buffer).
"""
from __future__ import annotations

from typing import Optional

import torch

from .. import kernels
from ..weights.loader import Param
from .base import Part, register_part


class RMSNorm(Part):
    graph_safe = True
    takes_shift = True      # ``run(..., shift=)``: a single-token step's token shift in the norm's kernel

    def __init__(self, spec, dtype, device):
        self.size, self.eps, self.dtype = spec.size, float(spec.eps), dtype

    def params(self):
        return {"weight": Param((self.size,), "vector", init="around_one")}

    def run(self, x: torch.Tensor, out: torch.Tensor, delta: Optional[torch.Tensor] = None,
            delta_bias: Optional[torch.Tensor] = None, rows: Optional[torch.Tensor] = None, shift=None):
        """x: float32 [nt, size], updated in place by the pending delta unless
        ``rows`` selects the rows to normalise. out: engine dtype. ``delta`` may be a
        ``kernels.GatedDelta`` (what a gated sublayer leaves to be added)."""
        if shift is not None:
            # a single-token step's token shift rides on the norm (``kernels.gated_add_rmsnorm``)
            if delta is not None and not isinstance(delta, kernels.GatedDelta):
                delta = kernels.GatedDelta(delta, delta_bias)
            return kernels.gated_add_rmsnorm(x, self.gain(), self.eps, out, delta, rows, shift)
        if isinstance(delta, kernels.GatedDelta):
            return kernels.gated_add_rmsnorm(x, self.gain(), self.eps, out, delta, rows)
        return kernels.add_rmsnorm(x, self.gain(), self.eps, out, delta, delta_bias, rows)

    def gain(self) -> torch.Tensor:
        """The weight per coordinate, float32 [size]."""
        return self.w["weight"]

    def fold(self, x: torch.Tensor, out: torch.Tensor, ctx) -> "kernels.NormFold":
        """For the few-rows product in front of this norm, which then does the add and the
        sums of squares itself; ``.scale()`` of the result goes to the product behind it."""
        parts = ctx.ws.take("norm.parts", kernels.NormFold.parts_shape(self.size), torch.float32)
        return kernels.NormFold(x, self.gain(), self.eps, out, parts)


class ScalarRMSNorm(RMSNorm):
    """The same norm with one gain for all coordinates: the parameter is a 0-d tensor, and the
    kernels get it spread over a row once, when the weights are bound."""

    def params(self):
        return {"weight": Param((), "vector", init="around_one")}

    def bind(self, tensors):
        super().bind(tensors)
        self._gain = tensors["weight"].to(torch.float32).reshape(1).expand(self.size).contiguous()

    def gain(self):
        return self._gain


class OffsetRMSNorm(RMSNorm):
    """The same norm with a weight stored around zero: the gain is 1 + w, formed in float32 once, when
    the weights are bound."""

    def params(self):
        return {"weight": Param((self.size,), "vector")}

    def bind(self, tensors):
        super().bind(tensors)
        self._gain = (tensors["weight"].to(torch.float32) + 1.0).contiguous()

    def gain(self):
        return self._gain


register_part("rmsnorm_offset", OffsetRMSNorm)
register_part("rmsnorm", RMSNorm)
register_part("rmsnorm_scalar", ScalarRMSNorm)
