"""KelasunConfig: the configuration of the Kelasun architecture under its config.json keys.

config.json: ``architecture`` ("Kelasun"), ``vocab``, ``width``, ``norm.eps``, ``postln_alpha`` (the stream's factor in every sum with a
sublayer's result, 1 by default), ``logit_scale`` (1 by default) and ``layers``, a list with one entry per layer: ``type`` (the mixer:
"attention" or "latent_attention"), ``mixer`` (its sizes and constants) and ``mlp`` (null: the layer has no feed-forward). Layers may
differ in all of it.

* attention: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, optional ``q_temp`` (``coef``, ``every``: queries are multiplied by a factor
  that grows with the number of whole stretches of ``every`` positions).
* latent_attention: ``heads``, ``dim`` and ``rot_dim`` (unrotated and rotated dimensions of a query head), ``vdim``, ``kv_rank``, ``q_rank`` (sizes of
  the latents), ``scale``, ``rot`` with ``dims`` (``rot_dim``, or fewer), ``base`` and optional ``scaling`` (``factor``, ``original``, ``fast``, ``slow``).
* mlp: ``kind`` "moe" with ``expert.ff``, ``router`` (``experts``, ``top``) and optional ``shared.ff``.
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, Tuple

from .lm_config import ConfigError, LmConfig

MIXER_TYPES = ("attention", "latent_attention")


def _positive_int(v) -> bool:
    return isinstance(v, int) and not isinstance(v, bool) and v > 0


def _number(v) -> bool:
    return isinstance(v, (int, float)) and not isinstance(v, bool)


def _need_ints(where: str, d: Any, keys) -> None:
    if not isinstance(d, dict):
        raise ConfigError(f"kelasun: {where} must be an object, got {d!r}")
    for key in keys:
        if not _positive_int(d.get(key)):
            raise ConfigError(f"kelasun: {where}.{key} must be a positive integer, got {d.get(key)!r}")


def _need_numbers(where: str, d: Any, keys, positive: bool = True) -> None:
    if not isinstance(d, dict):
        raise ConfigError(f"kelasun: {where} must be an object, got {d!r}")
    for key in keys:
        if not _number(d.get(key)) or (positive and d[key] <= 0):
            raise ConfigError(f"kelasun: {where}.{key} must be a {'positive ' if positive else ''}number, got {d.get(key)!r}")


def _check_attention(where: str, m: dict) -> None:
    m.setdefault("kv_heads", m.get("heads"))
    m.setdefault("vdim", m.get("dim"))
    _need_ints(where, m, ("heads", "kv_heads", "dim", "vdim"))
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"kelasun: {where}: {m['heads']} heads are no multiple of {m['kv_heads']} key/value heads")
    if m.get("q_temp") is not None:
        _need_numbers(f"{where}.q_temp", m["q_temp"], ("coef",), positive=False)
        _need_numbers(f"{where}.q_temp", m["q_temp"], ("every",))


def _check_latent(where: str, m: dict) -> None:
    m.setdefault("rot_dim", 0)
    _need_ints(where, m, ("heads", "dim", "vdim", "kv_rank", "q_rank"))
    dr = m["rot_dim"]
    if not isinstance(dr, int) or isinstance(dr, bool) or dr < 0:
        raise ConfigError(f"kelasun: {where}.rot_dim must be a non-negative integer, got {dr!r}")
    rot = m.get("rot")
    if rot is None:
        return
    dims = rot.get("dims") if isinstance(rot, dict) else None
    if not isinstance(dims, int) or isinstance(dims, bool) or dims < 0 or dims % 2 or dims > dr:
        raise ConfigError(f"kelasun: {where}.rot.dims must be an even number of at most rot_dim={dr}, got {rot!r}")
    if not (_number(rot.get("base")) and rot["base"] > 1):
        raise ConfigError(f"kelasun: {where}.rot.base must be a number above 1, got {rot.get('base')!r}")
    if rot.get("scaling") is not None:
        _need_numbers(f"{where}.rot.scaling", rot["scaling"], ("factor", "original", "fast", "slow"))


def _check_layer(i: int, layer) -> None:
    if not isinstance(layer, dict) or layer.get("type") not in MIXER_TYPES:
        raise ConfigError(f"kelasun: layer {i} has type {layer.get('type') if isinstance(layer, dict) else layer!r}; known: {', '.join(MIXER_TYPES)}")
    m, where = layer.get("mixer"), f"layer {i}: mixer"
    if not isinstance(m, dict):
        raise ConfigError(f"kelasun: layer {i} has no 'mixer' sizes")
    (_check_attention if layer["type"] == "attention" else _check_latent)(where, m)
    _need_numbers(where, m, ("scale",), positive=False)
    mlp, where = layer.get("mlp"), f"layer {i}: mlp"
    if mlp is None:
        return
    if not isinstance(mlp, dict) or mlp.get("kind") != "moe":
        raise ConfigError(f"kelasun: {where}.kind must be 'moe', got {mlp!r}")
    _need_ints(f"{where}.expert", mlp.get("expert"), ("ff",))
    _need_ints(f"{where}.router", mlp.get("router"), ("experts", "top"))
    if mlp["router"]["top"] > mlp["router"]["experts"]:
        raise ConfigError(f"kelasun: {where}.router: {mlp['router']['top']} experts a token out of {mlp['router']['experts']}")
    if mlp.get("shared") is not None:
        _need_ints(f"{where}.shared", mlp["shared"], ("ff",))


@LmConfig.register_subclass("kelasun")
@dataclass(frozen=True)
class KelasunConfig(LmConfig):
    vocab: int = 0
    width: int = 0
    norm_eps: float = 1e-5
    postln_alpha: float = 1.0
    logit_scale: float = 1.0
    layers: Tuple[Dict[str, Any], ...] = ()
    initializer_range: float = 0.02

    def __post_init__(self):
        if not _positive_int(self.vocab) or not _positive_int(self.width):
            raise ConfigError(f"kelasun: vocab and width must be positive integers, got {self.vocab!r} and {self.width!r}")
        if not (_number(self.norm_eps) and self.norm_eps > 0):
            raise ConfigError(f"kelasun: norm.eps must be positive, got {self.norm_eps!r}")
        for key in ("postln_alpha", "logit_scale"):
            if not _number(getattr(self, key)):
                raise ConfigError(f"kelasun: {key} must be a number, got {getattr(self, key)!r}")
        if not self.layers:
            raise ConfigError("kelasun: the configuration lists no layers")
        for i, layer in enumerate(self.layers):
            _check_layer(i, layer)

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_hf_config(cls, hf_config: Dict[str, Any]) -> "KelasunConfig":
        for required in ("vocab", "width", "layers"):
            if required not in hf_config:
                raise ConfigError(f"kelasun: config.json lacks the key {required!r}")
        norm = hf_config.get("norm") or {}
        if not isinstance(norm, dict) or "eps" not in norm:
            raise ConfigError("kelasun: config.json lacks norm.eps")
        layers = hf_config["layers"]
        if not isinstance(layers, (list, tuple)):
            raise ConfigError("kelasun: 'layers' must be a list")
        extra = {key: hf_config[key] for key in ("postln_alpha", "logit_scale", "initializer_range") if key in hf_config}
        return cls(vocab=hf_config["vocab"], width=hf_config["width"], norm_eps=norm["eps"], layers=tuple(copy.deepcopy(list(layers))), **extra)

    def to_hf_config(self) -> Dict[str, Any]:
        return {"architecture": "Kelasun", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps}, "postln_alpha": self.postln_alpha,
                "logit_scale": self.logit_scale, "layers": copy.deepcopy(list(self.layers)), "initializer_range": self.initializer_range}

    def __hash__(self):
        return hash((self.vocab, self.width, self.norm_eps, self.postln_alpha, self.logit_scale, repr(self.layers)))

    def model_spec(self):
        from levanter_amd.models.kelasun import kelasun_model_spec

        return kelasun_model_spec(self)
