"""Typed Mutolix configuration read from the keys of its config.json.

A Mutolix model is a stack of layers listed in config.json, each with the kind of its mixer (`type`: "mlstm" or "attention"), the
mixer's sizes and constants (`mixer`) and its feed-forward (`mlp`: a dense one, or null for a layer without one).  Nothing is
assumed that the file does not say: attention without `q_temp` leaves its queries as they are, one without `v_mix` its values;
`embedding.scale` defaults to 1.

    {"architecture": "Mutolix", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s}, "layers": [
        {"type": "mlstm", "mixer": {"heads", "dim", "vdim", "gate_cap"}, "mlp": {"kind": "dense", "ff"} | null},
        {"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "q_temp": {"coef", "every"}, "v_mix": true | false},
         "mlp": ...}, ...]}
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from ..errors import ConfigError
from .felosun import _positive_number
from .fields import optional
from .napizen import _number
from .nobodra import MAX_POSITIONS, _positive, _section


@dataclass(frozen=True)
class MutolixMemory:
    heads: int
    dim: int
    vdim: int
    gate_cap: float

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MutolixMemory":
        return cls(*(_positive(raw, name, where) for name in ("heads", "dim", "vdim")), _positive_number(raw, "gate_cap", where))

    def to_json_dict(self) -> dict:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "gate_cap": self.gate_cap}


@dataclass(frozen=True)
class MutolixAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    temp_coef: float | None = None      # the query temperature's factor and step; None: no temperature
    temp_every: int | None = None
    v_mix: bool = False

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "MutolixAttention":
        heads, kv_heads, dim, vdim = (_positive(raw, name, where) for name in ("heads", "kv_heads", "dim", "vdim"))
        if heads % kv_heads:
            raise ConfigError(f"{where}: heads must be a multiple of kv_heads, got {heads} and {kv_heads}")
        coef = every = None
        if raw.get("q_temp") is not None:
            temp = _section(raw, "q_temp", where)
            coef, every = _number(temp, "coef", where), _positive(temp, "every", where)
        try:
            v_mix = optional(raw, "v_mix", bool, False)
        except ConfigError as exc:
            raise ConfigError(f"{where}: {exc}") from None
        return cls(heads, kv_heads, dim, vdim, _positive_number(raw, "scale", where), coef, every, v_mix)

    def to_json_dict(self) -> dict:
        out: dict = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale, "v_mix": self.v_mix}
        if self.temp_every is not None:
            out["q_temp"] = {"coef": self.temp_coef, "every": self.temp_every}
        return out


MIXERS = {"mlstm": MutolixMemory, "attention": MutolixAttention}


@dataclass(frozen=True)
class MutolixLayer:
    type: str                       # "mlstm" | "attention"
    mixer: Any                      # the dataclass MIXERS names for the type
    ff: int | None                  # the dense feed-forward's inner size; None: the layer has none

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], index: int) -> "MutolixLayer":
        where = f"layer {index}"
        if not isinstance(raw, dict):
            raise ConfigError(f"{where} must be an object")
        kind = raw.get("type")
        if kind not in MIXERS:
            raise ConfigError(f"{where}: unknown type {kind!r}; expected one of: {', '.join(MIXERS)}")
        mlp, ff = raw.get("mlp"), None
        if mlp is not None:
            if not isinstance(mlp, dict):
                raise ConfigError(f"{where}: `mlp` must be an object or null")
            if mlp.get("kind") != "dense":
                raise ConfigError(f"{where}: unknown feed-forward kind {mlp.get('kind')!r}; expected 'dense'")
            ff = _positive(mlp, "ff", where)
        return cls(kind, MIXERS[kind].from_dict(_section(raw, "mixer", where), where), ff)

    def to_json_dict(self) -> dict:
        return {"type": self.type, "mixer": self.mixer.to_json_dict(), "mlp": None if self.ff is None else {"kind": "dense", "ff": self.ff}}


@dataclass(frozen=True)
class MutolixConfig:
    vocab_size: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: tuple
    eos_token_ids: tuple = ()        # the design names no end-of-sequence token: generation runs to its length limit
    model_type: str = "mutolix"

    ARCHITECTURE = "Mutolix"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "MutolixConfig":
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("layers must be a non-empty list")
        layers = tuple(MutolixLayer.from_dict(layer, index) for index, layer in enumerate(entries))
        mixed = [(index, layer.mixer) for index, layer in enumerate(layers) if layer.type == "attention" and layer.mixer.v_mix]
        for index, mixer in mixed[1:]:
            first = mixed[0][1]
            if mixer.kv_heads * mixer.vdim != first.kv_heads * first.vdim:
                raise ConfigError(f"layer {index}: v_mix needs as many values a token as layer {mixed[0][0]} has "
                                  f"({first.kv_heads} x {first.vdim}), got {mixer.kv_heads} x {mixer.vdim}")
        scale = 1.0
        if raw.get("embedding") is not None:
            scale = _number(_section(raw, "embedding", "config.json"), "scale", "config.json embedding", 1.0)
        return cls(vocab_size=_positive(raw, "vocab", "config.json"), width=_positive(raw, "width", "config.json"),
                   norm_eps=_positive_number(_section(raw, "norm", "config.json"), "eps", "config.json norm"), embedding_scale=scale, layers=layers)

    def first_mixing_layer(self) -> int | None:
        """The number of the layer whose values the other layers with v_mix take."""
        return next((index for index, layer in enumerate(self.layers) if layer.type == "attention" and layer.mixer.v_mix), None)

    def validate_context_length(self, max_seq_len: int) -> None:
        if not 0 < max_seq_len <= MAX_POSITIONS:
            raise ConfigError(f"max_seq_len must be within 1..{MAX_POSITIONS}, got {max_seq_len}")

    def to_json_dict(self) -> dict:
        return {"architecture": self.ARCHITECTURE, "vocab": self.vocab_size, "width": self.width, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embedding_scale}, "layers": [layer.to_json_dict() for layer in self.layers]}
