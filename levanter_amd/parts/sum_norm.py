"""How a sublayer's result enters a residual stream that is normed behind every sum: ``x <- N(alpha * x + f(x))``.

The sublayer reads the stream itself. Sum and norm are 32-bit and one row kernel, which is not launched by itself but left pending and
done by the pass that reads the stream next (the next sublayer's rounding of its input, or the norm before the head), so a sublayer
costs one row kernel; that kernel also adds up what the sublayer's last products have left unsummed (a product's K ranges, the outputs of
routed experts).
"""
from __future__ import annotations

from typing import Dict, Optional

import torch

from levanter_amd.kernels.library import PendingSumNorm
from .base import BuildEnv, Part, StepContext
from .registry import STREAM_MIXES
from .spec import PartSpec


@STREAM_MIXES.register("norm_after_sum")
class NormAfterSum(Part):
    """params: ``dim``, ``alpha`` (1), ``eps``, ``rms`` (False: a layer norm; True: an RMS norm). Tensors: ``weight`` ``[dim]``, optional
    ``bias``. Stands in a ``post_norm`` block's ``connect1`` and ``connect2``."""

    graph_safe = True
    takes_unsummed = True

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], env: BuildEnv):
        super().__init__(spec, tensors, env)
        p = spec.params
        self.dim, self.alpha, self.eps, self.rms = int(p["dim"]), float(p.get("alpha", 1.0)), float(p["eps"]), bool(p.get("rms", False))
        self.weight = tensors["weight"].to(env.device, torch.float32).contiguous()
        bias = tensors.get("bias")
        self.bias = None if bias is None else bias.to(env.device, torch.float32).contiguous()
        if self.weight.numel() != self.dim or (self.bias is not None and self.bias.numel() != self.dim):
            raise ValueError(f"norm_after_sum: the norm must have {self.dim} weights")

    def gate_of(self, h: torch.Tensor, ctx: StepContext) -> None:
        return None

    def read(self, x: torch.Tensor, ctx: StepContext) -> torch.Tensor:
        """The stream, rounded to the compute dtype by a pass that also does the write that is pending."""
        pending = ctx.take_pending(x)
        if pending is not None and not isinstance(pending, PendingSumNorm):
            ctx.kernels.finish(pending)
            pending = None
        if ctx.dtype == x.dtype:  # nothing to round: the stream itself (no part changes its input)
            if pending is not None:
                ctx.kernels.finish(pending)
            return x
        h = ctx.empty(x.shape[0], x.shape[1])
        ctx.kernels.sum_norm_step(x, pending=pending, h_out=h)
        return h

    def write(self, y: Optional[torch.Tensor], gate, x: torch.Tensor, ctx: StepContext, product=None, experts=None) -> None:
        """``y`` None: nothing but ``experts``; ``product``: ``y`` is its output and holds nothing yet."""
        if product is not None:
            y = None
        pending = ctx.kernels.sum_norm_step(x, alpha=self.alpha, y=y, product=product, experts=experts,
                                            write_norm=(self.weight, self.bias, self.eps, self.rms), defer=True)
        if ctx.may_defer:
            ctx.pending = pending
        else:
            ctx.kernels.finish(pending)
