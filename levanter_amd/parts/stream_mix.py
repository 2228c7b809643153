"""Stream mixes: what the next layer reads as a function of the results of all layers so far, and what a loop over layers does to
the stream where a pass begins.

Depth-weighted average: with X_0 the embedding's output and X_(i+1) the result of the i-th layer run (its input plus what
its branches add), the stream that goes on is sum_j w[j] X_j over j = 0 .. i+1, with a weight vector of the layer's own.
The results are kept for the step in one float32 tensor ``[runs + 1, T, dim]``; the sum runs in 32-bit, in the order of j.
"""
from __future__ import annotations

from typing import Dict

import torch

from .base import BuildEnv, StepContext, StreamEntry, StreamMix
from .gated_block import read_stream
from .registry import STREAM_MIXES
from .spec import PartSpec


@STREAM_MIXES.register("depth_weighted_average")
class DepthWeightedAverage(StreamMix):
    """params: ``index`` (how many layer runs come before this one), ``n_runs`` (layer runs of the model); tensor
    ``weights`` ``[index + 2]``."""

    graph_safe = True
    KEY = "depth_weighted_average.streams"

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], env: BuildEnv):
        super().__init__(spec, tensors, env)
        self.index = int(spec.params["index"])
        self.n_runs = int(spec.params["n_runs"])
        if not 0 <= self.index < self.n_runs:
            raise ValueError(f"depth_weighted_average: run {self.index} of {self.n_runs}")
        self.weights = tensors["weights"].to(env.device, torch.float32).contiguous()
        if self.weights.numel() != self.index + 2:
            raise ValueError(f"depth_weighted_average: run {self.index} needs {self.index + 2} weights, got {self.weights.numel()}")

    def enter(self, x: torch.Tensor, ctx: StepContext) -> None:
        if self.index == 0:  # the embedding's output is the first of the results
            ctx.settle()
            streams = torch.empty((self.n_runs + 1,) + tuple(x.shape), dtype=torch.float32, device=x.device)
            streams[0].copy_(x)
            ctx.shared[self.KEY] = streams

    def leave(self, x: torch.Tensor, ctx: StepContext) -> None:
        streams = ctx.shared.get(self.KEY)
        if streams is None or streams.shape[1:] != x.shape:
            raise RuntimeError("depth_weighted_average: the run with index 0 has not been through this step")
        ctx.settle()
        # where the block allows it the sum is left to the norm that reads x next (the next layer's, or the one before the head)
        ctx.pending = ctx.kernels.stream_average(streams, x, self.weights, self.index + 2, defer=bool(ctx.may_defer))


@STREAM_MIXES.register("loop_input")
class LoopInput(StreamEntry):
    """Where pass t of a loop over layers begins: ``x <- W [x; x0] + step[t]`` with ``x0`` the embedding's output. The half of the product that
    reads ``x0`` is the same in every pass and computed once a step. Products run in the compute dtype with 32-bit sums. params: ``dim``,
    ``eps`` (of the layers' norms: a write of such a norm that is unfinished is then done in the pass that reads the stream); tensors ``weight`` ``[dim, 2 dim]`` (the columns of x first), ``step`` ``[passes, dim]``."""

    graph_safe = True
    KEY = "loop_input.start"

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], env: BuildEnv):
        super().__init__(spec, tensors, env)
        self.dim = int(spec.params["dim"])
        self.eps = float(spec.params.get("eps", 1e-6))
        w, steps = tensors["weight"], tensors["step"].to(env.device, torch.float32)
        if tuple(w.shape) != (self.dim, 2 * self.dim) or steps.dim() != 2 or steps.shape[1] != self.dim:
            raise ValueError(f"loop_input: the weight must be [{self.dim}, {2 * self.dim}] and the steps [passes, {self.dim}]")
        self.weight = w[:, :self.dim].to(env.device, env.dtype).contiguous()
        self.start_weight = w[:, self.dim:].to(env.device, env.dtype).contiguous()
        self.steps = [row.contiguous() for row in steps]

    def begin(self, x: torch.Tensor, ctx: StepContext) -> None:
        start = torch.empty_like(x)
        ctx.kernels.linear(read_stream(x, ctx, 1, self.eps), self.start_weight, None, start)
        ctx.shared[self.KEY] = start

    def enter_run(self, x: torch.Tensor, run: int, ctx: StepContext) -> None:
        h = read_stream(x, ctx, 1, self.eps)
        ctx.settle()
        ctx.kernels.linear(h, self.weight, self.steps[run], x, residual=ctx.shared[self.KEY])
