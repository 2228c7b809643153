"""Lelatar as a model description: which parts each layer has and where their tensors come from.

A layer is pre-norm (``norm1``, ``norm2``: RMS norms whose weight is stored as its distance from one): the mixer (``l<i>.mix.*``), then a
gated feed-forward (``l<i>.mlp.{gate,up,down}``, silu) or none, then, where the model has a second token table (``side.embed``), an input of
the layer's own from its part of the token's row (``l<i>.side.{gate,proj,norm}``). The mixer is one of two:

* ``mamba2``: state-space duality (``in`` gives [z | x | B | C | dt]; ``conv`` with ``conv.b``, ``dt_bias``, ``A_log``, ``D``, ``norm``, ``o``);
* ``parallel``: half the sum of two branches, each through an RMS norm over the width with a weight of its own (``left.out``,
  ``right.out``). ``left``: causal softmax attention with queries and keys normed over the whole projection (``q.norm``, ``k.norm``), a
  rotation in the rotate-half layout, a sink per head (``sink``), ``o``. ``right``: a gated delta rule (``q``, ``k``, ``v`` with a convolution each,
  ``a``, ``b``, ``A_log``, ``dt_bias``, the head norm's weight ``norm``, the silu gate ``g``, ``o``).

The layers of ``loop`` run several times in a row with the same weights, every pass with cache units of its own; where a pass begins the
stream becomes ``loop.in`` [x; the embedding's output] plus the pass's row of ``loop.step``. ``final.norm`` comes before the head ``head``.
Linear weights are stored ``[out, in]``.
"""
from __future__ import annotations

import math

from levanter_amd.config.lelatar import LelatarConfig
from levanter_amd.parts.spec import LayerSpec, ModelSpec, PartSpec, PlanEntry, TensorSpec

BRANCH_WEIGHT = 0.5  # the mixer 'parallel' is half the sum of its branches
UNIT_KEY_EPS = 1e-6  # inside the root of the delta rule's unit norms of queries and keys


def lelatar_model_spec(cfg: LelatarConfig) -> ModelSpec:
    d, eps = cfg.width, float(cfg.norm_eps)
    lin = 1.0 / math.sqrt(d)

    def norm(name: str) -> PartSpec:
        return PartSpec("group_rmsnorm", {"dim": d, "groups": 1, "eps": eps, "weight_offset": 1.0}, {"weight": TensorSpec(name, (d,), std=0.1)}, family="norm")

    def weight(name: str, *shape: int) -> TensorSpec:
        return TensorSpec(name, shape, std=1.0 / math.sqrt(shape[-1]))

    def near_one(name: str, n: int) -> TensorSpec:
        return TensorSpec(name, (n,), init="one_plus_normal", std=0.1)

    def mamba(p: str, m: dict) -> PartSpec:
        H, P, N, G, K = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
        inner, C = H * P, H * P + 2 * G * N
        return PartSpec("state_space_dual",
                        {"dim": d, "n_heads": H, "value_dim": P, "key_dim": N, "n_groups": G, "taps": K, "norm_groups": m["norm_groups"], "norm_eps": eps},
                        {"in.weight": weight(f"{p}.in", inner + C + H, d), "conv.weight": TensorSpec(f"{p}.conv", (C, K), std=0.5),
                         "conv.bias": TensorSpec(f"{p}.conv.b", (C,), std=0.2), "dt.bias": TensorSpec(f"{p}.dt_bias", (H,), std=1.0),
                         "decay": TensorSpec(f"{p}.A_log", (H,), std=1.0), "skip": near_one(f"{p}.D", H), "norm.weight": near_one(f"{p}.norm", inner),
                         "out.weight": weight(f"{p}.o", d, inner)}, family="mixer")

    def attention(p: str, m: dict) -> PartSpec:
        H, G, dk, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        rot = m.get("rot")
        rotary = PartSpec("rotary_half", {"dims": rot["dims"], "base": float(rot["base"])}, family="position") if rot is not None and rot["dims"] else None
        return PartSpec("talking_heads_attention",
                        {"dim": d, "n_heads": H, "n_kv_heads": G, "head_dim": dk, "value_dim": dv, "scale": float(m["scale"]), "window": None,
                         "qk_norm": "projection", "qk_norm_eps": eps, "rotary": rotary},
                        {"q.weight": weight(f"{p}.q", H * dk, d), "k.weight": weight(f"{p}.k", G * dk, d), "v.weight": weight(f"{p}.v", G * dv, d),
                         "q_norm.weight": near_one(f"{p}.q.norm", H * dk), "k_norm.weight": near_one(f"{p}.k.norm", G * dk),
                         "sinks": TensorSpec(f"{p}.sink", (H,), std=1.0), "out.weight": weight(f"{p}.o", d, H * dv)}, family="mixer")

    def delta(p: str, m: dict) -> PartSpec:
        H, G, dk, dv, K = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"]
        tensors = {"gate.weight": weight(f"{p}.g", H * dv, d), "decay_rate.weight": weight(f"{p}.a", H, d), "write_rate.weight": weight(f"{p}.b", H, d),
                   "dt.bias": TensorSpec(f"{p}.dt_bias", (H,), std=1.0), "decay": TensorSpec(f"{p}.A_log", (H,), std=1.0),
                   "norm.weight": near_one(f"{p}.norm", dv), "out.weight": weight(f"{p}.o", d, H * dv)}
        for n, c in (("q", G * dk), ("k", G * dk), ("v", H * dv)):
            tensors[f"{n}.weight"], tensors[f"{n}.conv"] = weight(f"{p}.{n}", c, d), TensorSpec(f"{p}.{n}.conv", (c, K), std=0.5)
        return PartSpec("gated_delta_rule", {"dim": d, "n_heads": H, "n_kv_heads": G, "key_dim": dk, "value_dim": dv, "taps": K, "key_eps": UNIT_KEY_EPS, "norm_eps": eps},
                        tensors, family="mixer")

    def parallel(p: str, m: dict) -> PartSpec:
        return PartSpec("parallel_mixers", {"left": attention(f"{p}.left", m["left"]), "right": delta(f"{p}.right", m["right"]),
                                            "left_scale": BRANCH_WEIGHT, "right_scale": BRANCH_WEIGHT, "branch_norm_eps": eps},
                        {"left_norm.weight": near_one(f"{p}.left.out", d), "right_norm.weight": near_one(f"{p}.right.out", d)}, family="mixer")

    layers = []
    for i, layer in enumerate(cfg.layers):
        p, m, mlp = f"l{i}", layer["mixer"], layer.get("mlp")
        parts = {"norm1": norm(f"{p}.norm1"), "mixer": mamba(f"{p}.mix", m) if layer["type"] == "mamba2" else parallel(f"{p}.mix", m)}
        if mlp is not None:
            f = mlp["ff"]
            parts["norm2"] = norm(f"{p}.norm2")
            parts["feed_forward"] = PartSpec("gated_mlp", {"dim": d, "inner_dim": f, "activation": "silu"},
                                             {"gate.weight": weight(f"{p}.mlp.gate", f, d), "up.weight": weight(f"{p}.mlp.up", f, d),
                                              "down.weight": weight(f"{p}.mlp.down", d, f)}, family="feed_forward")
        if cfg.token_side is not None:
            n = cfg.token_side["dim"]
            parts["token_input"] = PartSpec("gated_token_input", {"dim": d, "token_dim": n, "offset": i * n, "eps": eps},
                                            {"table": TensorSpec("side.embed", (cfg.vocab, cfg.n_layers * n), std=1.0),
                                             "gate.weight": weight(f"{p}.side.gate", n, d), "proj.weight": weight(f"{p}.side.proj", d, n),
                                             "norm.weight": near_one(f"{p}.side.norm", d)}, family="stream_mix")
        layers.append(LayerSpec("pre_norm", parts))

    entries = []
    if cfg.loop is not None:
        entries.append(PartSpec("loop_input", {"dim": d, "eps": eps}, {"weight": weight("loop.in", d, 2 * d), "step": TensorSpec("loop.step", (cfg.loop["times"], d), std=0.1)},
                                family="stream_mix"))
    embedding = PartSpec("token_embedding", {"vocab_size": cfg.vocab, "dim": d, "position": None}, {"table": TensorSpec("embed", (cfg.vocab, d), std=1.0)},
                         family="embedding")
    head = PartSpec("linear_head", {"vocab_size": cfg.vocab, "dim": d}, {"weight": TensorSpec("head", (cfg.vocab, d), std=lin)}, family="head")
    return ModelSpec(
        architecture="lelatar",
        vocab_size=cfg.vocab,
        dim=d,
        embedding=embedding,
        layers=layers,
        # every run of a layer has its own cache unit, also the runs of one layer in the loop
        plan=[PlanEntry(layer=layer, cache=run, writes_cache=True, enters=None if t is None else (0, t)) for run, (layer, t) in enumerate(cfg.layer_order())],
        final_norm=norm("final.norm"),
        head=head,
        max_positions=None,
        init_std=cfg.initializer_range,
        stream_entries=entries,
    )
