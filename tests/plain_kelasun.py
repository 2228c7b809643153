"""Kelasun, stated plainly: whole sequences in float64, one function per mechanism, no cache, no kernels, nothing shared with the
package. ``weights`` maps checkpoint tensor names to float64 tensors, ``cfg`` is the raw config.json dict.

Notation: x the residual stream ``[T, D]``, which is also every sublayer's input h; positions count from 0.
"""
from __future__ import annotations

import contextlib
import math
from typing import Callable, Dict, List, Optional, Tuple

import torch

F64 = torch.float64

_ROUND: Callable[[torch.Tensor], torch.Tensor] = lambda t: t


@contextlib.contextmanager
def rounded_products():
    """Inside it every linear map's input and result are rounded to bfloat16: how far rounding alone moves a model's logits."""
    global _ROUND
    was, _ROUND = _ROUND, lambda t: t.float().to(torch.bfloat16).double()
    try:
        yield
    finally:
        _ROUND = was


_MARGINS: Optional[List[torch.Tensor]] = None


@contextlib.contextmanager
def close_calls():
    """Collects, router by router, how far apart the last chosen and the first left-out logit of every token are (infinitely far where
    every expert is chosen): where they nearly tie, another rounding chooses another expert and gets another result."""
    global _MARGINS
    was, _MARGINS = _MARGINS, []
    try:
        yield _MARGINS
    finally:
        _MARGINS = was


def lin(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """w x for every row of x (weights are stored [out, in])."""
    return _ROUND(_ROUND(x) @ w.T)


# ---- norms ----------------------------------------------------------------------------------------------------------
def layer_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """(x - mean) / sqrt(mean squared deviation + eps) * w."""
    d = x - x.mean(-1, keepdim=True)
    return d / torch.sqrt((d * d).mean(-1, keepdim=True) + eps) * w


def rms_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * w."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


def norm_after_sum(x: torch.Tensor, y: torch.Tensor, alpha: float, w: torch.Tensor, eps: float) -> torch.Tensor:
    """How a sublayer's result y enters the stream: the stream becomes the norm of alpha x + y."""
    return layer_norm(alpha * x + y, w, eps)


# ---- rotation ---------------------------------------------------------------------------------------------------------
def stretched_frequencies(dims: int, base: float, scaling: Optional[dict]) -> List[float]:
    """Radians a position for each of the dims / 2 pairs. With ``scaling``: fast pairs keep theirs, slow pairs turn ``factor`` times
    slower, and along a ramp over the pairs' indices in between the two are mixed."""
    plain = [base ** (-2.0 * i / dims) for i in range(dims // 2)]
    if not scaling:
        return plain
    where = lambda turns: dims * math.log(scaling["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))
    lo, hi = max(math.floor(where(scaling["fast"])), 0), min(math.ceil(where(scaling["slow"])), dims - 1)
    out = []
    for i, f in enumerate(plain):
        r = min(max((i - lo) / max(hi - lo, 0.001), 0.0), 1.0)
        out.append(r * f / scaling["factor"] + (1.0 - r) * f)
    return out


def rotation_magnitude(scaling: Optional[dict]) -> float:
    """What cosine and sine are multiplied by."""
    return 1.0 if not scaling else 0.1 * math.log(scaling["factor"]) + 1.0


def rotate_pairs(v: torch.Tensor, positions: torch.Tensor, freqs: List[float], magnitude: float = 1.0) -> torch.Tensor:
    """v ``[T, heads, d]``: dimensions (2i, 2i + 1) turn by p * freqs[i] and grow by ``magnitude``; dimensions behind the pairs pass."""
    out = v.clone()
    n = len(freqs)
    if n == 0:
        return out
    a = positions.to(F64)[:, None] * torch.tensor(freqs, dtype=F64)[None, :]
    cos, sin = magnitude * torch.cos(a)[:, None, :], magnitude * torch.sin(a)[:, None, :]
    u, w = v[..., 0:2 * n:2], v[..., 1:2 * n:2]
    out[..., 0:2 * n:2] = u * cos - w * sin
    out[..., 1:2 * n:2] = w * cos + u * sin
    return out


# ---- attention from a cached latent -------------------------------------------------------------------------------------
def latent_attention(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """Keys and values of every head made from one latent per token; a rotated key part that all heads share; queries through a latent of
    their own; every element of the heads gated by a sigmoid of the input. Written without absorbing any matrix into another."""
    T = h.shape[0]
    H, dk, dr, dv, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    q = lin(rms_norm(lin(h, W[f"{p}.dq"]), W[f"{p}.dq.norm"], eps), W[f"{p}.uq"]).view(T, H, dk + dr)
    down = lin(h, W[f"{p}.dkv"])
    c = rms_norm(down[:, :R], W[f"{p}.dkv.norm"], eps)
    k, v = lin(c, W[f"{p}.uk"]).view(T, H, dk), lin(c, W[f"{p}.uv"]).view(T, H, dv)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    freqs, mag = stretched_frequencies(rot["dims"], rot["base"], rot.get("scaling")), rotation_magnitude(rot.get("scaling"))
    pos = torch.arange(T)
    q_rot, k_rot = rotate_pairs(q[..., dk:], pos, freqs, mag), rotate_pairs(down[:, None, R:], pos, freqs, mag)[:, 0]
    future = torch.ones(T, T, dtype=torch.bool).triu(1)
    o = torch.zeros(T, H, dv, dtype=F64)
    for i in range(H):
        s = (q[:, i, :dk] @ k[:, i].T + q_rot[:, i] @ k_rot.T) * m["scale"]
        o[:, i] = torch.softmax(s.masked_fill(future, -math.inf), -1) @ v[:, i]
    return lin(o.reshape(T, H * dv) * torch.sigmoid(lin(h, W[f"{p}.g"])), W[f"{p}.o"])


# ---- attention with a distance term and a sink ----------------------------------------------------------------------------
def temperature(positions: torch.Tensor, q_temp: Optional[dict]) -> torch.Tensor:
    """What the queries at these positions are multiplied by: one plus coef times the logarithm of one plus the number of whole stretches
    of ``every`` positions up to and including each."""
    if not q_temp:
        return torch.ones(positions.numel(), dtype=F64)
    return 1.0 + q_temp["coef"] * torch.log(torch.floor((positions.to(F64) + 1.0) / q_temp["every"]) + 1.0)


def distance_slopes(H: int) -> List[float]:
    return [2.0 ** (-8.0 * (h + 1) / H) for h in range(H)]


def sink_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, slopes: List[float], sinks: torch.Tensor) -> torch.Tensor:
    """q ``[T, H, d]``, k ``[T, G, d]``, v ``[T, G, dv]`` -> ``[T, H, dv]``: causal softmax attention; head h reads key/value head
    h // (H / G), a score is scale q.k - slopes[h] (i - j), and head h's denominator also holds exp(sinks[h])."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    distance = (torch.arange(T)[:, None] - torch.arange(T)[None, :]).to(F64)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale - slopes[h] * distance).masked_fill(distance < 0, -math.inf)
        top = torch.maximum(s.max(-1).values, sinks[h])[:, None]
        w = torch.exp(s - top)
        out[:, h] = (w @ v[:, g]) / (w.sum(-1, keepdim=True) + torch.exp(sinks[h] - top))
    return out


def biased_attention(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(lin(h, W[f"{p}.q"]), W[f"{p}.q.norm"], eps) * temperature(torch.arange(T), m.get("q_temp"))[:, None]
    k = rms_norm(lin(h, W[f"{p}.k"]), W[f"{p}.k.norm"], eps)
    v = lin(h, W[f"{p}.v"])
    o = sink_attention(q.view(T, H, d), k.view(T, G, d), v.view(T, G, dv), m["scale"], distance_slopes(H), W[f"{p}.sink"])
    o = o * torch.sigmoid(lin(h, W[f"{p}.g"]))[:, :, None]
    return lin(o.reshape(T, H * dv), W[f"{p}.o"])


# ---- feed-forward -------------------------------------------------------------------------------------------------------
def squared_relu(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) ** 2


def expert(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return lin(squared_relu(lin(h, W[f"{p}.up"])), W[f"{p}.down"])


def route(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Router logits ``[T, E]`` -> the ``top`` experts of each token and their weights, the softmax of the chosen logits alone."""
    if _MARGINS is not None:
        order = z.sort(-1, descending=True).values
        _MARGINS.append(order[:, top - 1] - order[:, top] if top < z.shape[1] else torch.full((z.shape[0],), math.inf, dtype=F64))
    best = z.topk(top, dim=-1)
    return best.indices, torch.softmax(best.values, -1)


def experts(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, mlp: dict) -> torch.Tensor:
    chosen, weights = route(h @ W[f"{p}.router"].T, mlp["router"]["top"])
    y = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        share = (weights * (chosen == e)).sum(-1)
        rows = share > 0
        if bool(rows.any()):
            y[rows] += share[rows][:, None] * expert(h[rows], W, f"{p}.e{e}")
    if mlp.get("shared"):
        y = y + expert(h, W, f"{p}.shared")
    return y


# ---- the model ----------------------------------------------------------------------------------------------------------
def forward(tokens: List[int], weights: Dict[str, torch.Tensor], cfg: dict) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """Logits ``[T, vocab]`` and the residual stream after every layer."""
    eps, alpha = float(cfg["norm"]["eps"]), float(cfg["postln_alpha"])
    x = weights["embed"][torch.tensor(tokens)]
    streams = []
    for i, layer in enumerate(cfg["layers"]):
        p = f"l{i}"
        mixer = {"latent_attention": latent_attention, "attention": biased_attention}[layer["type"]]
        x = norm_after_sum(x, mixer(x, weights, f"{p}.mix", layer["mixer"], eps), alpha, weights[f"{p}.norm1"], eps)
        if layer.get("mlp") is not None:
            x = norm_after_sum(x, experts(x, weights, f"{p}.mlp", layer["mlp"]), alpha, weights[f"{p}.norm2"], eps)
        streams.append(x.clone())
    return lin(layer_norm(x, weights["final.norm"], eps), weights["head"]) * cfg["logit_scale"], streams


def plain_logits(W: Dict[str, torch.Tensor], cfg: dict, tokens) -> torch.Tensor:
    return forward([int(t) for t in tokens], W, cfg)[0]


# ---- configurations and weights for tests ---------------------------------------------------------------------------------
def experts_mlp(ff=24, experts=8, top=2, shared=16) -> dict:
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, **({"shared": {"ff": shared}} if shared else {})}


def latent_layer(heads=4, dim=16, rot_dim=8, vdim=8, kv_rank=24, q_rank=40, base=100.0, scaling=(4.0, 64, 8.0, 1.0), scale=None, mlp=None) -> dict:
    rot = {"dims": rot_dim, "base": base}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "scale": (dim + rot_dim) ** -0.5 if scale is None else scale, "rot": rot}}


def biased_layer(heads=4, kv_heads=2, dim=16, vdim=8, q_temp=(0.3, 16), scale=None, mlp=None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale}
    if q_temp is not None:
        m["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return {"type": "attention", "mixer": m, "mlp": mlp}


def make_config(vocab=97, width=64, layers=None, eps=1e-5, alpha=1.5, logit_scale=0.5) -> dict:
    return {"architecture": "Kelasun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "logit_scale": logit_scale,
            "layers": layers if layers is not None else [biased_layer(), latent_layer()]}


def random_weights(cfg: dict, seed: int, dtype=F64) -> Dict[str, torch.Tensor]:
    """Weights drawn so that every mechanism matters: scores of order one to three, sinks that take a share, gates on both sides of one
    half, norm weights away from one. Values are bfloat16 numbers (a file stores them exactly)."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]

    def rn(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).to(dtype)

    def mat(rows, cols, gain=1.0):
        return rn(rows, cols, std=gain / math.sqrt(cols))

    W = {"embed": rn(V, D), "final.norm": rn(D, mean=1.0, std=0.2), "head": mat(V, D, 2.0)}
    for i, L in enumerate(cfg["layers"]):
        m, p, q = L["mixer"], f"l{i}.", f"l{i}.mix."
        W[p + "norm1"] = rn(D, mean=1.0, std=0.2)
        H = m["heads"]
        if L["type"] == "latent_attention":
            dk, dr, dv, R, Q = m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
            W[q + "dq"], W[q + "dq.norm"], W[q + "uq"] = mat(Q, D), rn(Q, mean=1.5, std=0.3), mat(H * (dk + dr), Q)
            W[q + "dkv"], W[q + "dkv.norm"] = mat(R + dr, D), rn(R, mean=1.2, std=0.3)
            W[q + "uk"], W[q + "uv"], W[q + "g"] = mat(H * dk, R), mat(H * dv, R), mat(H * dv, D, 1.5)
        else:
            G, dk, dv = m["kv_heads"], m["dim"], m["vdim"]
            W[q + "q"], W[q + "k"], W[q + "v"] = mat(H * dk, D), mat(G * dk, D), mat(G * dv, D)
            W[q + "q.norm"], W[q + "k.norm"] = rn(H * dk, mean=1.5, std=0.3), rn(G * dk, mean=1.5, std=0.3)
            W[q + "sink"], W[q + "g"] = rn(H, mean=1.0), mat(H, D, 1.5)
        W[q + "o"] = mat(D, H * dv, 2.0)
        mlp = L.get("mlp")
        if mlp is not None:
            W[p + "norm2"] = rn(D, mean=1.0, std=0.2)
            W[p + "mlp.router"] = mat(mlp["router"]["experts"], D, 1.5)
            inner = {f"e{e}": mlp["expert"]["ff"] for e in range(mlp["router"]["experts"])}
            if mlp.get("shared"):
                inner["shared"] = mlp["shared"]["ff"]
            for name, F in inner.items():
                W[f"{p}mlp.{name}.up"], W[f"{p}mlp.{name}.down"] = mat(F, D), mat(D, F)
    return W


def write_folder(cfg: dict, W: Dict[str, torch.Tensor], path: str, dtype=torch.bfloat16) -> str:
    """config.json and model.safetensors of these weights, through the safetensors package."""
    import json
    import os

    from safetensors.torch import save_file

    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.to(dtype).contiguous() for k, v in W.items()}, os.path.join(path, "model.safetensors"))
    return path
