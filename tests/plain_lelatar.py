"""Lelatar, stated plainly: whole sequences in float64, one function per mechanism, no cache, no kernels, nothing shared with the
package. ``weights`` maps checkpoint tensor names to float64 tensors, ``cfg`` is the raw config.json dict.

Notation: x the residual stream ``[T, D]``, h a sublayer's input, positions count from 0.
"""
from __future__ import annotations

import contextlib
import math
from typing import Callable, Dict, List, Optional, Tuple

import torch

F64 = torch.float64

KEY_EPS = 1e-6  # inside the root of the unit norms of the delta rule's queries and keys

_ROUND: Callable[[torch.Tensor], torch.Tensor] = lambda t: t


@contextlib.contextmanager
def rounded_products():
    """Inside it every linear map's input and result (and the convolutions' results) are rounded to bfloat16: how far rounding alone moves
    a model's logits."""
    global _ROUND
    was, _ROUND = _ROUND, lambda t: t.float().to(torch.bfloat16).double()
    try:
        yield
    finally:
        _ROUND = was


def lin(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """w x for every row of x (weights are stored [out, in])."""
    return _ROUND(_ROUND(x) @ w.T)


# ---- norms and activations ----------------------------------------------------------------------------------------
def rms_norm(x: torch.Tensor, w: Optional[torch.Tensor], eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension, times w."""
    y = x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)
    return y if w is None else y * w


def one_plus_norm(x: torch.Tensor, w: torch.Tensor, eps: float) -> torch.Tensor:
    """The norms of the residual stream: their weight is stored as the distance from one."""
    return rms_norm(x, 1.0 + w, eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z / (1.0 + torch.exp(-z))


def softplus(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) + torch.log1p(torch.exp(-z.abs()))


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- short convolution ----------------------------------------------------------------------------------------------
def causal_conv(x: torch.Tensor, taps: torch.Tensor, bias: Optional[torch.Tensor] = None) -> torch.Tensor:
    """x ``[T, C]``, taps ``[C, K]``: out[t, c] = sum_k taps[c, K - 1 - k] x[t - k, c] (+ bias), zeros before the start."""
    T, K = x.shape[0], taps.shape[1]
    out = torch.zeros_like(x)
    for k in range(min(K, T)):
        out[k:] += x[:T - k] * taps[:, K - 1 - k]
    return out if bias is None else out + bias


# ---- a state per head with a scalar decay (Mamba-2) -------------------------------------------------------------------
def ssd_scan(x: torch.Tensor, B: torch.Tensor, C: torch.Tensor, dt: torch.Tensor, A: torch.Tensor, D: torch.Tensor,
             state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """x ``[T, H, P]``, B and C ``[T, G, N]``, dt ``[T, H]`` (positive), A ``[H]`` (positive rate), D ``[H]``. Per head h, reading group
    h // (H / G): S <- exp(-A dt) S + dt B x^T, y = S^T C + D x. Returns y ``[T, H, P]`` and the last state ``[H, N, P]``."""
    T, H, P = x.shape
    G, N = B.shape[1:]
    own = torch.arange(H) // (H // G)
    S = torch.zeros(H, N, P, dtype=F64) if state is None else state.clone()
    y = torch.zeros_like(x)
    for t in range(T):
        S = torch.exp(-A * dt[t])[:, None, None] * S + (dt[t][:, None] * B[t, own])[:, :, None] * x[t][:, None, :]
        y[t] = (S * C[t, own][:, :, None]).sum(1) + D[:, None] * x[t]
    return y, S


def mamba2(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * P
    z, xbc, dt = torch.split(lin(h, W[f"{p}.in"]), [inner, inner + 2 * G * N, H], dim=1)
    xbc = _ROUND(silu(causal_conv(xbc, W[f"{p}.conv"], W[f"{p}.conv.b"])))
    x, B, C = torch.split(xbc, [inner, G * N, G * N], dim=1)
    dt = softplus(dt + W[f"{p}.dt_bias"])
    y, _ = ssd_scan(x.view(T, H, P), B.view(T, G, N), C.view(T, G, N), dt, torch.exp(W[f"{p}.A_log"]), W[f"{p}.D"])
    y = y.reshape(T, inner) * silu(z)
    y = rms_norm(y.view(T, m["norm_groups"], -1), None, eps).reshape(T, inner) * W[f"{p}.norm"]
    return lin(y, W[f"{p}.o"])


# ---- attention ------------------------------------------------------------------------------------------------------
def rotate_half(v: torch.Tensor, positions: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """v ``[T, heads, d]``: dimension i < dims/2 is paired with i + dims/2, the pair turns by p * base^(-2i/dims); dimensions from
    ``dims`` on pass unchanged."""
    out = v.clone()
    n = dims // 2
    if n == 0:
        return out
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(n)], dtype=F64)
    a = positions.to(F64)[:, None] * f[None, :]
    cos, sin = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    u, w = v[..., :n], v[..., n:2 * n]
    out[..., :n] = u * cos - w * sin
    out[..., n:2 * n] = w * cos + u * sin
    return out


def sink_attention(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, scale: float, sinks: torch.Tensor) -> torch.Tensor:
    """q ``[T, H, d]``, k ``[T, G, d]``, v ``[T, G, dv]`` -> ``[T, H, dv]``: causal softmax attention; head h reads key/value head
    h // (H / G), and its denominator also holds exp(sinks[h])."""
    T, H, _ = q.shape
    G = k.shape[1]
    out = torch.zeros(T, H, v.shape[2], dtype=F64)
    future = torch.ones(T, T, dtype=torch.bool).triu(1)
    for h in range(H):
        g = h // (H // G)
        s = ((q[:, h] @ k[:, g].T) * scale).masked_fill(future, -math.inf)
        top = torch.maximum(s.max(-1).values, sinks[h])[:, None]
        w = torch.exp(s - top)
        out[:, h] = (w @ v[:, g]) / (w.sum(-1, keepdim=True) + torch.exp(sinks[h] - top))
    return out


def rotary_sink_attention(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(lin(h, W[f"{p}.q"]), W[f"{p}.q.norm"], eps).view(T, H, d)
    k = rms_norm(lin(h, W[f"{p}.k"]), W[f"{p}.k.norm"], eps).view(T, G, d)
    v = lin(h, W[f"{p}.v"]).view(T, G, dv)
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    pos = torch.arange(T)
    q, k = rotate_half(q, pos, rot["dims"], rot["base"]), rotate_half(k, pos, rot["dims"], rot["base"])
    o = sink_attention(q, k, v, m["scale"], W[f"{p}.sink"])
    return lin(o.reshape(T, H * dv), W[f"{p}.o"])


# ---- gated delta rule -----------------------------------------------------------------------------------------------
def delta_scan(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, g: torch.Tensor, beta: torch.Tensor,
               state: Optional[torch.Tensor] = None) -> Tuple[torch.Tensor, torch.Tensor]:
    """q, k ``[T, G, d]``, v ``[T, H, dv]``, g and beta ``[T, H]``. Per head h, reading query/key head h // (H / G): S <- g S;
    S <- S + k (beta (v - S^T k))^T; o = S^T q. Returns o ``[T, H, dv]`` and the last state ``[H, d, dv]``."""
    T, H, dv = v.shape
    G, d = q.shape[1:]
    own = torch.arange(H) // (H // G)
    S = torch.zeros(H, d, dv, dtype=F64) if state is None else state.clone()
    o = torch.zeros_like(v)
    for t in range(T):
        kt, qt = k[t, own][:, :, None], q[t, own][:, :, None]
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * kt).sum(1))
        S = S + kt * u[:, None, :]
        o[t] = (S * qt).sum(1)
    return o, S


def unit(x: torch.Tensor) -> torch.Tensor:
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + KEY_EPS)


def gated_delta_rule(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (_ROUND(silu(causal_conv(lin(h, W[f"{p}.{n}"]), W[f"{p}.{n}.conv"]))) for n in ("q", "k", "v"))
    q, k = unit(q.view(T, G, d)) * d ** -0.5, unit(k.view(T, G, d))
    beta = torch.sigmoid(lin(h, W[f"{p}.b"]))
    g = torch.exp(-torch.exp(W[f"{p}.A_log"]) * softplus(lin(h, W[f"{p}.a"]) + W[f"{p}.dt_bias"]))
    o, _ = delta_scan(q, k, v.view(T, H, dv), g, beta)
    o = rms_norm(o, W[f"{p}.norm"], eps).reshape(T, H * dv) * silu(lin(h, W[f"{p}.g"]))
    return lin(o, W[f"{p}.o"])


def parallel_mixer(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """Half the sum of the two branches, each through an RMS norm of the model's width with a weight of its own."""
    left = rotary_sink_attention(h, W, f"{p}.left", m["left"], eps)
    right = gated_delta_rule(h, W, f"{p}.right", m["right"], eps)
    return 0.5 * (rms_norm(left, W[f"{p}.left.out"], eps) + rms_norm(right, W[f"{p}.right.out"], eps))


# ---- feed-forward, token input, loop ----------------------------------------------------------------------------------
def dense_feed_forward(h: torch.Tensor, W: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return lin(silu(lin(h, W[f"{p}.gate"])) * lin(h, W[f"{p}.up"]), W[f"{p}.down"])


def token_input(x: torch.Tensor, tokens: List[int], W: Dict[str, torch.Tensor], layer: int, dim: int, eps: float) -> torch.Tensor:
    """What layer ``layer`` adds to the stream for each token: the layer's part of the token's row of a second table, gated by
    the stream, projected to the width and normed."""
    e = W["side.embed"][torch.tensor(tokens)][:, layer * dim:(layer + 1) * dim]
    y = lin(gelu_tanh(lin(x, W[f"l{layer}.side.gate"])) * e, W[f"l{layer}.side.proj"])
    return rms_norm(y, W[f"l{layer}.side.norm"], eps)


def loop_entry(x: torch.Tensor, x0: torch.Tensor, W: Dict[str, torch.Tensor], run: int) -> torch.Tensor:
    """The stream as the loop's pass number ``run`` starts on it: a product of [x; x0] plus the pass's vector."""
    return lin(torch.cat([x, x0], 1), W["loop.in"]) + W["loop.step"][run]


def layer_order(cfg: dict) -> List[Tuple[int, Optional[int]]]:
    """The layers in the order they run, each with the number of the loop's pass that begins right before it (None: none does)."""
    n = len(cfg["layers"])
    loop = cfg.get("loop")
    if not loop:
        return [(i, None) for i in range(n)]
    a, b = loop["start"], loop["stop"]
    order = [(i, None) for i in range(a)]
    for t in range(loop["times"]):
        order += [(i, t if i == a else None) for i in range(a, b)]
    return order + [(i, None) for i in range(b, n)]


# ---- the model --------------------------------------------------------------------------------------------------------
def forward(tokens: List[int], weights: Dict[str, torch.Tensor], cfg: dict) -> Tuple[torch.Tensor, List[torch.Tensor]]:
    """Logits ``[T, vocab]`` and the residual stream after every layer run."""
    eps = float(cfg["norm"]["eps"])
    side = cfg.get("token_side")
    x = x0 = weights["embed"][torch.tensor(tokens)]
    streams = []
    for i, run in layer_order(cfg):
        if run is not None:
            x = loop_entry(x, x0, weights, run)
        layer, p = cfg["layers"][i], f"l{i}"
        h = one_plus_norm(x, weights[f"{p}.norm1"], eps)
        mixer = {"mamba2": mamba2, "parallel": parallel_mixer}[layer["type"]]
        x = x + mixer(h, weights, f"{p}.mix", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            x = x + dense_feed_forward(one_plus_norm(x, weights[f"{p}.norm2"], eps), weights, f"{p}.mlp")
        if side:
            x = x + token_input(x, tokens, weights, i, side["dim"], eps)
        streams.append(x.clone())
    return lin(one_plus_norm(x, weights["final.norm"], eps), weights["head"]), streams


def plain_logits(W: Dict[str, torch.Tensor], cfg: dict, tokens) -> torch.Tensor:
    return forward([int(t) for t in tokens], W, cfg)[0]


# ---- configurations and weights for tests -------------------------------------------------------------------------------
def left_sizes(heads=4, kv_heads=2, dim=16, vdim=8, rot_dims=8, base=10000.0, scale=None) -> dict:
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale}
    if rot_dims is not None:
        m["rot"] = {"dims": rot_dims, "base": base}
    return m


def right_sizes(heads=4, kv_heads=2, dim=16, vdim=8, conv=4) -> dict:
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def parallel_layer(left=None, right=None, ff=48) -> dict:
    return {"type": "parallel", "mixer": {"left": left or left_sizes(), "right": right or right_sizes()}, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def mamba_layer(heads=4, vdim=16, state=12, groups=2, norm_groups=2, conv=3, ff=None) -> dict:
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def make_config(vocab=97, width=64, layers=None, eps=1e-5, loop=(1, 2, 2), side=8) -> dict:
    cfg = {"architecture": "Lelatar", "vocab": vocab, "width": width, "norm": {"eps": eps},
           "layers": layers if layers is not None else [parallel_layer(), mamba_layer()]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        cfg["token_side"] = {"dim": side}
    return cfg


def random_weights(cfg: dict, seed: int, dtype=F64) -> Dict[str, torch.Tensor]:
    """Weights drawn so that every mechanism matters: scores of order one to three, sinks that take a share, decays from fast to
    slow, step sizes around one half. Values are bfloat16 numbers (a file stores them exactly)."""
    g = torch.Generator().manual_seed(seed)
    D, V = cfg["width"], cfg["vocab"]

    def rn(*shape, std=1.0, mean=0.0):
        return (torch.randn(*shape, generator=g) * std + mean).to(torch.bfloat16).to(dtype)

    W = {"embed": rn(V, D), "final.norm": rn(D, std=0.2), "head": rn(V, D, std=1 / math.sqrt(D))}
    lin = 1 / math.sqrt(D)
    side, loop = cfg.get("token_side"), cfg.get("loop")
    if side:
        W["side.embed"] = rn(V, len(cfg["layers"]) * side["dim"])
    if loop:
        W["loop.in"] = rn(D, 2 * D, std=1 / math.sqrt(2 * D))
        W["loop.step"] = rn(loop["times"], D, std=0.3)
    for i, L in enumerate(cfg["layers"]):
        m, p = L["mixer"], f"l{i}."
        W[p + "norm1"] = rn(D, std=0.2)
        if L["type"] == "mamba2":
            H, P, N, G, K = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
            inner, C = H * P, H * P + 2 * G * N
            q = p + "mix."
            W[q + "in"] = rn(inner + C + H, D, std=lin)
            W[q + "conv"], W[q + "conv.b"] = rn(C, K, std=0.7), rn(C, std=0.2)
            W[q + "dt_bias"], W[q + "A_log"], W[q + "D"] = rn(H, std=1.0, mean=-2.0), rn(H, std=1.0), rn(H, mean=0.5, std=0.5)
            W[q + "norm"], W[q + "o"] = rn(inner, mean=1.0, std=0.2), rn(D, inner, std=1 / math.sqrt(inner))
        else:
            le, ri = m["left"], m["right"]
            H, G, dk, dv = le["heads"], le["kv_heads"], le["dim"], le["vdim"]
            q = p + "mix.left."
            W[q + "q"], W[q + "k"], W[q + "v"] = rn(H * dk, D, std=lin), rn(G * dk, D, std=lin), rn(G * dv, D, std=lin)
            W[q + "q.norm"], W[q + "k.norm"] = rn(H * dk, mean=1.5, std=0.3), rn(G * dk, mean=1.5, std=0.3)
            W[q + "sink"] = rn(H, mean=1.0)
            W[q + "o"] = rn(D, H * dv, std=1 / math.sqrt(H * dv))
            W[p + "mix.left.out"], W[p + "mix.right.out"] = rn(D, mean=1.0, std=0.2), rn(D, mean=1.0, std=0.2)
            H, G, dk, dv, K = ri["heads"], ri["kv_heads"], ri["dim"], ri["vdim"], ri["conv"]
            q = p + "mix.right."
            for n, c in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
                W[q + n], W[q + n + ".conv"] = rn(c, D, std=lin), rn(c, K, std=0.7)
            W[q + "a"], W[q + "b"] = rn(H, D, std=lin), rn(H, D, std=lin)
            W[q + "dt_bias"], W[q + "A_log"] = rn(H, mean=-2.0), rn(H)
            W[q + "norm"], W[q + "g"] = rn(dv, mean=1.0, std=0.2), rn(H * dv, D, std=1.5 * lin)
            W[q + "o"] = rn(D, H * dv, std=1 / math.sqrt(H * dv))
        mlp = L.get("mlp")
        if mlp is not None:
            F = mlp["ff"]
            W[p + "norm2"] = rn(D, std=0.2)
            W[p + "mlp.gate"], W[p + "mlp.up"], W[p + "mlp.down"] = rn(F, D, std=lin), rn(F, D, std=lin), rn(D, F, std=1 / math.sqrt(F))
        if side:
            d = side["dim"]
            W[p + "side.gate"], W[p + "side.proj"], W[p + "side.norm"] = rn(d, D, std=lin), rn(D, d, std=1 / math.sqrt(d)), rn(D, mean=0.5, std=0.2)
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
