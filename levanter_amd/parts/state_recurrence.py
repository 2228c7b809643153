"""Recurrent mixers with a matrix state per head, one decay per head and token, and a short convolution ahead of the recurrence.

State-space duality (Mamba-2; Dao and Gu, "Transformers are SSMs: Generalized Models and Efficient Algorithms Through Structured State
Space Duality"): one projection gives [z | x | B | C | dt]; x, B and C pass a causal convolution per channel and silu; with
dt <- softplus(dt + bias) the state of head h, whose B and C are those of its group, goes

    S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T,        y_t = S_t^T C_t + D x_t,

and y * silu(z) is normed in equal parts of its row, multiplied by a weight, and goes through W_o.

Gated delta rule (Yang, Kautz and Hatamizadeh, "Gated Delta Networks: Improving Mamba2 with Delta Rule"): q, k and v pass the same kind of
convolution; q and k become unit vectors per head; with beta = sigmoid(W_b h) and g = exp(-exp(A_log) softplus(W_a h + bias))

    S <- g S,        S <- S + k (beta (v - S^T k))^T,        o = S^T q,

each head's o is normed, multiplied by a weight and by silu(W_g h), and goes through W_o.

What a request carries from step to step is one float32 vector in its state slot: the convolution's last inputs (those of position p in row
p mod taps) and S. The projections and the convolution's output are in the compute dtype, everything else is 32-bit.
"""
from __future__ import annotations

from typing import Dict

import torch

from levanter_amd.cache.requirements import SlotState
from .base import BuildEnv, CacheUnitView, Mixer, StepContext
from .linear import Linear
from .registry import MIXERS
from .spec import PartSpec


def _pad8(n: int) -> int:
    return (n + 7) // 8 * 8


class StateRecurrence(Mixer):
    """What the two mixers share: ``proj`` / ``attend`` / ``out`` around ``kernels.state_recurrence``. A subclass sets the sizes, ``columns`` (name ->
    first column of ``proj``'s output: ``x`` the convolution's channels, ``a`` the decay's sums, ``b`` the write rate's or None, ``gate``)
    and ``rule_args`` (the offsets of queries, keys and values among the channels, the norm's parts, constants)."""

    graph_safe = True
    rule = ""

    def _tensor(self, tensors: Dict[str, torch.Tensor], name: str, shape) -> torch.Tensor:
        t = tensors[name].to(torch.float32).cpu()
        if tuple(t.shape) != tuple(shape):
            raise ValueError(f"{self.kind}: {name} must be {list(shape)}, got {list(t.shape)}")
        return t

    def _check_sizes(self) -> None:
        if self.n_heads % self.n_groups:
            raise ValueError(f"{self.kind}: {self.n_heads} heads are no multiple of {self.n_groups} groups")
        if max(self.key_dim, self.value_dim) > 256:
            raise ValueError(f"{self.kind}: heads of {self.key_dim} / {self.value_dim} key / value channels (at most 256)")
        if self.taps < 1:
            raise ValueError(f"{self.kind}: a convolution of {self.taps} taps")

    def cache_requirement(self):
        return SlotState((self.taps * self.channels + self.n_heads * self.key_dim * self.value_dim,), "float32")

    def forward(self, h: torch.Tensor, x: torch.Tensor, ctx: StepContext, unit: CacheUnitView, writes_cache: bool) -> None:
        a = ctx.empty(h.shape[0], self.n_heads * self.value_dim)
        self.attend(self.proj(h, ctx), ctx, unit, writes_cache, a)
        self.out(a, ctx, residual=x, final=True)

    def compute(self, h: torch.Tensor, y: torch.Tensor, ctx: StepContext, unit: CacheUnitView, writes_cache: bool) -> None:
        a = ctx.empty(h.shape[0], self.n_heads * self.value_dim)
        self.attend(self.proj(h, ctx), ctx, unit, writes_cache, a)
        self.out(a, ctx, out=y, may_leave=True)

    def attend(self, p: torch.Tensor, ctx: StepContext, unit: CacheUnitView, writes_cache: bool, a: torch.Tensor) -> None:
        """Everything between the two products: ``p`` is what ``proj`` gives, ``a`` ``[T, H*dv]`` takes what ``out`` reads. The request's state is
        read and advanced."""
        if not writes_cache:
            raise ValueError(f"{self.kind}: a recurrence cannot read another entry's state without advancing it")
        c, H, inner = self.columns, self.n_heads, self.n_heads * self.value_dim
        # a step with prompt portions has fewer runs than tokens (at most one per request of the step): the path for runs
        max_runs = int(ctx.seq_slots.numel()) if ctx.attention.n_prefill_tiles else None
        ctx.kernels.state_recurrence(
            self.rule, p[:, c["x"]:c["x"] + self.channels], self.conv_taps, self.conv_bias, p[:, c["a"]:c["a"] + H],
            None if c["b"] is None else p[:, c["b"]:c["b"] + H], self.a_bias, self.rate, self.skip, p[:, c["gate"]:c["gate"] + inner], self.norm_weight,
            unit.state, ctx.token_slots, ctx.attention.positions, a, n_heads=H, n_groups=self.n_groups, key_dim=self.key_dim, value_dim=self.value_dim,
            norm_eps=self.norm_eps, max_runs=max_runs, **self.rule_args)


@MIXERS.register("state_space_dual")
class StateSpaceDual(StateRecurrence):
    """params: ``dim``, ``n_heads``, ``value_dim``, ``key_dim`` (the state's size), ``n_groups``, ``taps``, ``norm_groups``, ``norm_eps``, ``out_scale`` (1).
    Tensors (``[out, in]``): ``in.weight`` ``[inner + C + heads, dim]`` with inner = heads * value_dim and C = inner + 2 * n_groups * key_dim,
    ``conv.weight`` ``[C, taps]`` (the last column is the current token's), ``conv.bias`` ``[C]`` (optional), ``dt.bias``, ``decay`` (A_log),
    ``skip`` (D) ``[heads]``, ``norm.weight`` ``[inner]``, ``out.weight`` ``[dim, inner]``."""

    rule = "ssd"

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], env: BuildEnv):
        super().__init__(spec, tensors, env)
        p = spec.params
        self.dim, self.n_heads, self.value_dim, self.key_dim = int(p["dim"]), int(p["n_heads"]), int(p["value_dim"]), int(p["key_dim"])
        self.n_groups, self.taps, self.norm_eps = int(p["n_groups"]), int(p["taps"]), float(p["norm_eps"])
        self._check_sizes()
        H, inner, gn = self.n_heads, self.n_heads * self.value_dim, self.n_groups * self.key_dim
        if inner % int(p["norm_groups"]):
            raise ValueError(f"state_space_dual: {inner} numbers do not split into {p['norm_groups']} equal parts")
        C = self.channels = inner + 2 * gn
        w = self._tensor(tensors, "in.weight", (inner + C + H, self.dim))
        self.proj = Linear(torch.cat([w, torch.zeros((-w.shape[0]) % 8, self.dim)], 0), None, "out_in", env)
        self.columns = {"gate": 0, "x": inner, "a": inner + C, "b": None}
        self.rule_args = {"q_offset": inner + gn, "k_offset": inner, "v_offset": 0, "norm_groups": int(p["norm_groups"])}

        def vector(name, n):
            return self._tensor(tensors, name, (n,)).to(env.device).contiguous()

        self.conv_taps = self._tensor(tensors, "conv.weight", (C, self.taps)).to(env.device).contiguous()
        self.conv_bias = vector("conv.bias", C) if "conv.bias" in tensors else None
        self.a_bias, self.skip = vector("dt.bias", H), vector("skip", H)
        self.rate = torch.exp(vector("decay", H)).contiguous()
        self.norm_weight = (vector("norm.weight", inner) * float(p.get("out_scale", 1.0))).contiguous()
        self.out = Linear(self._tensor(tensors, "out.weight", (self.dim, inner)), tensors.get("out.bias"), "out_in", env)


@MIXERS.register("gated_delta_rule")
class GatedDeltaRule(StateRecurrence):
    """params: ``dim``, ``n_heads``, ``n_kv_heads`` (heads of queries and keys), ``key_dim``, ``value_dim``, ``taps``, ``key_eps``, ``q_scale``
    (``key_dim^(-1/2)`` by default), ``norm_eps``, ``out_scale`` (1). Tensors (``[out, in]``): ``q.weight``, ``k.weight`` ``[kv_heads*dk, dim]``, ``v.weight``,
    ``gate.weight`` ``[heads*dv, dim]``, their convolutions ``q.conv``, ``k.conv``, ``v.conv`` ``[channels, taps]`` (the last column is the current
    token's), ``decay_rate.weight`` (W_a), ``write_rate.weight`` (W_b) ``[heads, dim]``, ``dt.bias``, ``decay`` (A_log) ``[heads]``, ``norm.weight`` ``[dv]``
    (shared by the heads), ``out.weight`` ``[dim, heads*dv]``."""

    rule = "delta"

    def __init__(self, spec: PartSpec, tensors: Dict[str, torch.Tensor], env: BuildEnv):
        super().__init__(spec, tensors, env)
        p = spec.params
        self.dim, self.n_heads, self.n_groups = int(p["dim"]), int(p["n_heads"]), int(p["n_kv_heads"])
        self.key_dim, self.value_dim, self.taps, self.norm_eps = int(p["key_dim"]), int(p["value_dim"]), int(p["taps"]), float(p["norm_eps"])
        self._check_sizes()
        H, dk, dv, D = self.n_heads, self.key_dim, self.value_dim, self.dim
        nk, nv = self.n_groups * dk, H * dv
        C = self.channels = 2 * nk + nv
        # one product for everything that reads h: [q | k | v | gate | decay rate | write rate], parts behind v at multiples of 8 columns
        rows, at, self.columns = [], 0, {"x": 0}

        def part(name, weight):
            nonlocal at
            self.columns[name] = at
            width = _pad8(weight.shape[0])
            rows.extend([weight, torch.zeros(width - weight.shape[0], D)])
            at += width

        part("x", torch.cat([self._tensor(tensors, f"{n}.weight", (c, D)) for n, c in (("q", nk), ("k", nk), ("v", nv))], 0))
        part("gate", self._tensor(tensors, "gate.weight", (nv, D)))
        part("a", self._tensor(tensors, "decay_rate.weight", (H, D)))
        part("b", self._tensor(tensors, "write_rate.weight", (H, D)))
        self.proj = Linear(torch.cat(rows, 0), None, "out_in", env)
        self.conv_taps = torch.cat([self._tensor(tensors, f"{n}.conv", (c, self.taps)) for n, c in (("q", nk), ("k", nk), ("v", nv))], 0).to(env.device).contiguous()
        self.conv_bias = self.skip = None
        self.a_bias = self._tensor(tensors, "dt.bias", (H,)).to(env.device).contiguous()
        self.rate = torch.exp(self._tensor(tensors, "decay", (H,))).to(env.device).contiguous()
        self.norm_weight = (self._tensor(tensors, "norm.weight", (dv,)).repeat(H) * float(p.get("out_scale", 1.0))).to(env.device).contiguous()
        self.rule_args = {"q_offset": 0, "k_offset": nk, "v_offset": 2 * nk, "norm_groups": H, "key_eps": float(p["key_eps"]),
                          "q_scale": float(p["q_scale"]) if p.get("q_scale") is not None else dk ** -0.5}
        self.out = Linear(self._tensor(tensors, "out.weight", (D, nv)), tensors.get("out.bias"), "out_in", env)
