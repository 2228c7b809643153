"""A token's row of a second table as an input of its own to every layer.

With x the residual stream at the layer's end and e the layer's part of the token's row:

    y = W_proj (gelu_tanh(W_gate x) * e),        x <- x + y / sqrt(mean(y^2) + eps) * w

The stream itself is the first product's input (rounded to the compute dtype by the pass that does what is unfinished about it); the
activation runs in 32-bit on the product's 32-bit sums; the normed write is left pending for the pass that reads the stream next.
"""
from __future__ import annotations

from typing import Dict

import torch

from .base import BuildEnv, Part, StepContext
from .gated_block import read_stream
from .linear import Linear
from .registry import STREAM_MIXES
from .spec import PartSpec


@STREAM_MIXES.register("gated_token_input")
class GatedTokenInput(Part):
    """params: ``dim``, ``token_dim`` (numbers of the table a layer reads), ``offset`` (the first of them in a row), ``eps``. Tensors: ``table``
    ``[vocab, >= offset + token_dim]``, ``gate.weight`` ``[token_dim, dim]``, ``proj.weight`` ``[dim, token_dim]``, ``norm.weight`` ``[dim]``. Sizes that
    are no multiple of 8 carry zeros behind them."""

    graph_safe = True

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], env: BuildEnv):
        super().__init__(spec, tensors, env)
        p = spec.params
        D, n, off = int(p["dim"]), int(p["token_dim"]), int(p["offset"])
        self.dim, self.token_dim, self.eps = D, n, float(p["eps"])
        self.padded = (n + 7) // 8 * 8

        def f32(name, shape):
            t = tensors[name].to(torch.float32).cpu()
            if tuple(t.shape) != tuple(shape):
                raise ValueError(f"gated_token_input: {name} must be {list(shape)}, got {list(t.shape)}")
            return t

        table = tensors["table"]
        if table.dim() != 2 or table.shape[1] < off + n:
            raise ValueError(f"gated_token_input: a table of rows {list(table.shape)} has no columns {off} .. {off + n - 1}")
        self.table = torch.zeros(table.shape[0], self.padded, dtype=env.dtype, device=env.device)
        self.table[:, :n] = table[:, off:off + n].to(env.device, env.dtype)
        fill = self.padded - n
        self.gate = Linear(torch.cat([f32("gate.weight", (n, D)), torch.zeros(fill, D)], 0), None, "out_in", env)
        self.proj = Linear(torch.cat([f32("proj.weight", (D, n)), torch.zeros(D, fill)], 1), None, "out_in", env)
        self.norm_weight = f32("norm.weight", (D,)).to(env.device).contiguous()

    def add(self, x: torch.Tensor, ctx: StepContext) -> None:
        K = ctx.kernels
        h = read_stream(x, ctx, 1, self.eps)
        g = ctx.empty(x.shape[0], self.padded)
        if not K.token_gate_linear(h, self.gate.weight, ctx.tokens, self.table, g):
            K.token_gate(self.gate(h, ctx, out_dtype=torch.float32), ctx.tokens, self.table, g)
        y = self.proj(g, ctx, out_dtype=torch.float32)
        pending = K.group_norm_step(x, groups=1, eps=self.eps, y=y, post_weight=self.norm_weight, defer=True)
        if ctx.may_defer:
            ctx.pending = pending
        else:
            K.finish(pending)
