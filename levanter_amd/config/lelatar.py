"""LelatarConfig: the configuration of the Lelatar architecture under its config.json keys.

config.json: ``architecture`` ("Lelatar"), ``vocab``, ``width``, ``norm.eps``, ``layers`` (a list with one entry per layer: ``type`` (the
mixer: "mamba2" or "parallel"), ``mixer`` (its sizes and constants), ``mlp`` (``kind`` "dense" with ``ff``; or null for a layer without a
feed-forward)), optionally ``loop`` (``start``, ``stop``, ``times``: the layers start .. stop-1 run so many times in a row with the same weights
and a cache and state of their own per pass, and where a pass begins the stream is mixed with the embedding's output) and ``token_side``
(``dim``: every layer ends with an input of its own from a second token table). Layers may differ in all of it.

* mamba2: ``heads``, ``vdim``, ``state``, ``groups`` (of B and C), ``norm_groups``, ``conv`` (taps).
* parallel: ``left`` (an attention: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``scale``, ``rot`` with ``dims`` and ``base``) and ``right`` (a gated delta
  rule: ``heads``, ``kv_heads``, ``dim``, ``vdim``, ``conv``).
"""
from __future__ import annotations

import copy
from dataclasses import dataclass
from typing import Any, Dict, List, Optional, Tuple

from .lm_config import ConfigError, LmConfig

MIXER_TYPES = ("mamba2", "parallel")


def _positive_int(v) -> bool:
    return isinstance(v, int) and not isinstance(v, bool) and v > 0


def _number(v) -> bool:
    return isinstance(v, (int, float)) and not isinstance(v, bool)


def _need_ints(where: str, d: Any, keys) -> None:
    if not isinstance(d, dict):
        raise ConfigError(f"lelatar: {where} must be an object, got {d!r}")
    for key in keys:
        if not _positive_int(d.get(key)):
            raise ConfigError(f"lelatar: {where}.{key} must be a positive integer, got {d.get(key)!r}")


def _check_heads(where: str, m: dict) -> None:
    if m["heads"] % m["kv_heads"]:
        raise ConfigError(f"lelatar: {where}: {m['heads']} heads are no multiple of {m['kv_heads']} key/value heads")


def _check_layer(i: int, layer) -> None:
    if not isinstance(layer, dict) or layer.get("type") not in MIXER_TYPES:
        raise ConfigError(f"lelatar: layer {i} has type {layer.get('type') if isinstance(layer, dict) else layer!r}; known: {', '.join(MIXER_TYPES)}")
    m, where = layer.get("mixer"), f"layer {i}: mixer"
    if not isinstance(m, dict):
        raise ConfigError(f"lelatar: layer {i} has no 'mixer' sizes")
    if layer["type"] == "mamba2":
        m.setdefault("groups", 1)
        m.setdefault("norm_groups", 1)
        _need_ints(where, m, ("heads", "vdim", "state", "groups", "norm_groups", "conv"))
        if m["heads"] % m["groups"]:
            raise ConfigError(f"lelatar: {where}: {m['heads']} heads are no multiple of {m['groups']} groups")
        if (m["heads"] * m["vdim"]) % m["norm_groups"]:
            raise ConfigError(f"lelatar: {where}: {m['heads'] * m['vdim']} numbers do not split into {m['norm_groups']} equal parts")
    else:
        left, right = m.get("left"), m.get("right")
        for side, d in (("left", left), ("right", right)):
            if not isinstance(d, dict):
                raise ConfigError(f"lelatar: {where} needs 'left' and 'right'")
            d.setdefault("kv_heads", d.get("heads"))
            d.setdefault("vdim", d.get("dim"))
            _need_ints(f"{where}.{side}", d, ("heads", "kv_heads", "dim", "vdim") + (("conv",) if side == "right" else ()))
            _check_heads(f"{where}.{side}", d)
        if not _number(left.get("scale")):
            raise ConfigError(f"lelatar: {where}.left.scale must be a number, got {left.get('scale')!r}")
        rot = left.get("rot")
        if rot is not None:
            if not isinstance(rot, dict) or not isinstance(rot.get("dims"), int) or rot["dims"] < 0 or rot["dims"] % 2 or rot["dims"] > left["dim"]:
                raise ConfigError(f"lelatar: {where}.left.rot.dims must be an even number of at most dim={left['dim']}, got {rot!r}")
            if rot["dims"] and not (_number(rot.get("base")) and rot["base"] > 0):
                raise ConfigError(f"lelatar: {where}.left.rot.base must be a positive number, got {rot.get('base')!r}")
    mlp = layer.get("mlp")
    if mlp is not None:
        if not isinstance(mlp, dict) or mlp.get("kind") != "dense":
            raise ConfigError(f"lelatar: layer {i}: mlp.kind must be dense, got {mlp!r}")
        _need_ints(f"layer {i}: mlp", mlp, ("ff",))


@LmConfig.register_subclass("lelatar")
@dataclass(frozen=True)
class LelatarConfig(LmConfig):
    vocab: int = 0
    width: int = 0
    norm_eps: float = 1e-6
    layers: Tuple[Dict[str, Any], ...] = ()
    loop: Any = None
    token_side: Any = None
    initializer_range: float = 0.02

    def __post_init__(self):
        if not _positive_int(self.vocab) or not _positive_int(self.width):
            raise ConfigError(f"lelatar: vocab and width must be positive integers, got {self.vocab!r} and {self.width!r}")
        if not (_number(self.norm_eps) and self.norm_eps > 0):
            raise ConfigError(f"lelatar: norm.eps must be positive, got {self.norm_eps!r}")
        if not self.layers:
            raise ConfigError("lelatar: the configuration lists no layers")
        for i, layer in enumerate(self.layers):
            _check_layer(i, layer)
        if self.loop is not None:
            _need_ints("loop", self.loop, ("stop", "times"))
            start = self.loop.get("start")
            if not (isinstance(start, int) and not isinstance(start, bool)) or not 0 <= start < self.loop["stop"] <= len(self.layers):
                raise ConfigError(f"lelatar: loop: layers {start!r} .. {self.loop['stop']} are no stretch of the {len(self.layers)} layers")
        if self.token_side is not None:
            _need_ints("token_side", self.token_side, ("dim",))

    @property
    def n_layers(self) -> int:
        return len(self.layers)

    def layer_order(self) -> List[Tuple[int, Optional[int]]]:
        """The layers in the order they run, each with the number of the loop's pass that begins right before it (None: none)."""
        n = len(self.layers)
        if self.loop is None:
            return [(i, None) for i in range(n)]
        a, b = self.loop["start"], self.loop["stop"]
        passes = [(i, t if i == a else None) for t in range(self.loop["times"]) for i in range(a, b)]
        return [(i, None) for i in range(a)] + passes + [(i, None) for i in range(b, n)]

    @classmethod
    def from_hf_config(cls, hf_config: Dict[str, Any]) -> "LelatarConfig":
        for required in ("vocab", "width", "layers"):
            if required not in hf_config:
                raise ConfigError(f"lelatar: config.json lacks the key {required!r}")
        norm = hf_config.get("norm") or {}
        if not isinstance(norm, dict) or "eps" not in norm:
            raise ConfigError("lelatar: config.json lacks norm.eps")
        layers = hf_config["layers"]
        if not isinstance(layers, (list, tuple)):
            raise ConfigError("lelatar: 'layers' must be a list")
        extra = {"initializer_range": hf_config["initializer_range"]} if "initializer_range" in hf_config else {}
        return cls(vocab=hf_config["vocab"], width=hf_config["width"], norm_eps=norm["eps"], layers=tuple(copy.deepcopy(list(layers))),
                   loop=copy.deepcopy(hf_config.get("loop")), token_side=copy.deepcopy(hf_config.get("token_side")), **extra)

    def to_hf_config(self) -> Dict[str, Any]:
        out = {"architecture": "Lelatar", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.norm_eps},
               "layers": copy.deepcopy(list(self.layers)), "initializer_range": self.initializer_range}
        if self.loop is not None:
            out["loop"] = copy.deepcopy(self.loop)
        if self.token_side is not None:
            out["token_side"] = copy.deepcopy(self.token_side)
        return out

    def __hash__(self):
        return hash((self.vocab, self.width, self.norm_eps, repr(self.layers), repr(self.loop), repr(self.token_side)))

    def model_spec(self):
        from levanter_amd.models.lelatar import lelatar_model_spec

        return lelatar_model_spec(self)
