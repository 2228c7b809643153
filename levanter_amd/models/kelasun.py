"""Kelasun as a model description: which parts each layer has and where their tensors come from.

The residual stream starts as the token's row of ``embed``. A layer's sublayers read the stream itself, which is normed behind every
sum: x <- N(alpha x + mixer(x)) with ``norm1``, then the same with the feed-forward and ``norm2``; N is a layer norm with a weight, alpha
is ``postln_alpha``. The mixer (``l<i>.mix.*``) is one of two:

* ``attention``: softmax attention with queries and keys normed over the whole projection (``q.norm``, ``k.norm``), queries scaled by a
  temperature of their position, a distance term per head instead of a rotation, a sink per head (``sink``), an output gate per head
  (``g``), ``o``;
* ``latent_attention``: queries through a latent (``dq``, its RMS norm ``dq.norm``, ``uq``), keys and values from a cached latent (``dkv`` with
  ``dkv.norm``, ``uk``, ``uv``) plus one rotated key part that all heads share (the last ``rot_dim`` rows of ``dkv``), neighbouring pairs
  rotated with frequencies stretched along a ramp, an output gate per element (``g``), ``o``.

The feed-forward is a mixture of experts (``l<i>.mlp.router``, ``.e<j>.{up,down}``) without gates, weighted by the softmax over the chosen
logits, beside a shared expert (``.shared.{up,down}``); a layer may have none. ``final.norm`` comes before the head ``head``, whose logits are
multiplied by ``logit_scale``. Linear weights are stored ``[out, in]``.
"""
from __future__ import annotations

import math

from levanter_amd.config.kelasun import KelasunConfig
from levanter_amd.parts.spec import LayerSpec, ModelSpec, PartSpec, PlanEntry, TensorSpec

ROTATION_MAGNITUDE_SLOPE = 0.1  # cosine and sine are multiplied by ROTATION_MAGNITUDE_SLOPE * ln(factor) + 1 where frequencies are stretched
DISTANCE_SLOPE_RANGE = 8.0  # head h of H takes 2^(-DISTANCE_SLOPE_RANGE (h + 1) / H) a position off its scores
EXPERT_ACTIVATION = "relu_squared"


def kelasun_model_spec(cfg: KelasunConfig) -> ModelSpec:
    d, eps = cfg.width, float(cfg.norm_eps)
    lin = 1.0 / math.sqrt(d)

    def connection(name: str) -> PartSpec:
        return PartSpec("norm_after_sum", {"dim": d, "alpha": float(cfg.postln_alpha), "eps": eps},
                        {"weight": TensorSpec(name, (d,), init="one_plus_normal", std=0.1)}, family="stream_mix")

    def attention(p: str, m: dict) -> PartSpec:
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        temp = m.get("q_temp")
        return PartSpec("talking_heads_attention",
                        {"dim": d, "n_heads": H, "n_kv_heads": G, "head_dim": dk, "value_dim": dv, "scale": float(m["scale"]), "qk_norm": "projection",
                         "qk_norm_eps": eps, "q_temperature": None if temp is None else {"coef": temp["coef"], "every": temp["every"]},
                         "distance_slopes": [2.0 ** (-DISTANCE_SLOPE_RANGE * (h + 1) / H) for h in range(H)]},
                        {"q.weight": TensorSpec(f"{p}.q", (H * dk, d), std=lin), "k.weight": TensorSpec(f"{p}.k", (G * dk, d), std=lin),
                         "v.weight": TensorSpec(f"{p}.v", (G * dv, d), std=lin),
                         "q_norm.weight": TensorSpec(f"{p}.q.norm", (H * dk,), init="one_plus_normal", std=0.1),
                         "k_norm.weight": TensorSpec(f"{p}.k.norm", (G * dk,), init="one_plus_normal", std=0.1),
                         "sinks": TensorSpec(f"{p}.sink", (H,), std=1.0), "gate.weight": TensorSpec(f"{p}.g", (H, d), std=lin),
                         "out.weight": TensorSpec(f"{p}.o", (d, H * dv), std=1.0 / math.sqrt(H * dv))}, family="mixer")

    def latent(p: str, m: dict) -> PartSpec:
        H, dk, dr, dv, R, Q = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["q_rank"]
        rot, rotary = m.get("rot"), None
        if rot is not None and rot["dims"]:
            sc = rot.get("scaling")
            rotary = {"dims": rot["dims"], "base": float(rot["base"]), "layout": "pairs", "scaling": dict(sc) if sc else None,
                      "magnitude": ROTATION_MAGNITUDE_SLOPE * math.log(float(sc["factor"])) + 1.0 if sc else 1.0}
        return PartSpec("latent_attention",
                        {"dim": d, "n_heads": H, "head_dim": dk, "value_dim": dv, "latent_dim": R, "query_latent_dim": Q, "rope_dim": dr, "rotary": rotary,
                         "scale": float(m["scale"]), "norm_eps": eps, "gate": True, "gate_kind": "element"},
                        {"q_down.weight": TensorSpec(f"{p}.dq", (Q, d), std=lin),
                         "q_norm.weight": TensorSpec(f"{p}.dq.norm", (Q,), init="one_plus_normal", std=0.1),
                         "q.weight": TensorSpec(f"{p}.uq", (H * (dk + dr), Q), std=1.0 / math.sqrt(Q)),
                         "down.weight": TensorSpec(f"{p}.dkv", (R + dr, d), std=lin),
                         "latent_norm.weight": TensorSpec(f"{p}.dkv.norm", (R,), init="one_plus_normal", std=0.1),
                         "up_k.weight": TensorSpec(f"{p}.uk", (H * dk, R), std=1.0 / math.sqrt(R)),
                         "up_v.weight": TensorSpec(f"{p}.uv", (H * dv, R), std=1.0 / math.sqrt(R)),
                         "gate.weight": TensorSpec(f"{p}.g", (H * dv, d), std=lin),
                         "out.weight": TensorSpec(f"{p}.o", (d, H * dv), std=1.0 / math.sqrt(H * dv))}, family="mixer")

    def expert_tensors(p: str, f: int) -> dict:
        return {"up.weight": TensorSpec(f"{p}.up", (f, d), std=lin), "down.weight": TensorSpec(f"{p}.down", (d, f), std=1.0 / math.sqrt(f))}

    def experts(p: str, mlp: dict) -> PartSpec:
        E, f, shared = mlp["router"]["experts"], mlp["expert"]["ff"], mlp.get("shared")
        tensors = {"router.weight": TensorSpec(f"{p}.router", (E, d), std=lin)}
        for e in range(E):
            tensors.update({f"experts.{e}.{k}": t for k, t in expert_tensors(f"{p}.e{e}", f).items()})
        if shared is not None:
            shared = PartSpec("dense_mlp", {"dim": d, "inner_dim": shared["ff"], "activation": EXPERT_ACTIVATION}, expert_tensors(f"{p}.shared", shared["ff"]),
                              family="feed_forward")
        return PartSpec("routed_experts", {"dim": d, "inner_dim": f, "n_experts": E, "top": mlp["router"]["top"], "score": "softmax_chosen", "gated": False,
                                           "activation": EXPERT_ACTIVATION, "correction": False, "shared": shared}, tensors, family="feed_forward")

    layers, plan, ignored = [], [], []
    for i, layer in enumerate(cfg.layers):
        p, m = f"l{i}", layer["mixer"]
        parts = {"mixer": (attention if layer["type"] == "attention" else latent)(f"{p}.mix", m), "connect1": connection(f"{p}.norm1")}
        if layer.get("mlp") is not None:
            parts["feed_forward"] = experts(f"{p}.mlp", layer["mlp"])
            parts["connect2"] = connection(f"{p}.norm2")
        else:  # a file may still hold the second sublayer's norm of a layer that has none
            ignored.append(rf"l{i}\.norm2")
        layers.append(LayerSpec("post_norm", parts))
        plan.append(PlanEntry(layer=i, cache=i, writes_cache=True))

    return ModelSpec(
        architecture="kelasun",
        vocab_size=cfg.vocab,
        dim=d,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "dim": d, "position": None}, {"table": TensorSpec("embed", (cfg.vocab, d), std=1.0)},
                           family="embedding"),
        layers=layers,
        plan=plan,
        # logit_scale * (head h) = head (logit_scale * h): the factor rides on the norm's 32-bit weight
        final_norm=PartSpec("layernorm", {"dim": d, "eps": eps, "bias": False, "out_scale": float(cfg.logit_scale)},
                            {"weight": TensorSpec("final.norm", (d,), init="one_plus_normal", std=0.1)}, family="norm"),
        head=PartSpec("linear_head", {"vocab_size": cfg.vocab, "dim": d}, {"weight": TensorSpec("head", (cfg.vocab, d), std=lin)}, family="head"),
        max_positions=None,
        ignored_tensors=tuple(ignored),
        init_std=cfg.initializer_range,
    )
