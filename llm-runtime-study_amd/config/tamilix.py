"""Typed Tamilix configuration read from the keys of its config.json.

A Tamilix model is a stack of layers listed in config.json, each with the kind of its mixer (`type`: "latent_attention" or
"attention"), the mixer's sizes and constants (`mixer`) and its feed-forward (`mlp`: a dense one, routed experts, or null for a
layer without one).  A layer with `weights_of: j` owns no tensors: it runs with layer j's (mixer, feed-forward and norms) and a
cache of its own; the rest of its entry must equal layer j's (what it leaves out is layer j's).  Nothing is assumed that the file
does not say: a mixer without `mask` sees the whole context, a router without `identity` has no identity experts, experts without
`shared` no shared expert; `embedding.scale` defaults to 1.  `mask.size` is the window of a latent attention layer and the length of
an attention layer's chunks.

    {"architecture": "Tamilix", "vocab": V, "width": W, "norm": {"eps": e}, "embedding": {"scale": s}, "layers": [
        {"type": "latent_attention", "mixer": {"heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank", "scale", "mask": {"size"},
                                               "rot": {"base", "dims"}}, "mlp": {...} | null},
        {"type": "attention", "mixer": {"heads", "kv_heads", "dim", "vdim", "scale", "mask": {"size"}}, "mlp": {...} | null},
        {"type": ..., "mixer": ..., "mlp": ..., "weights_of": j}, ...]}
    mlp: {"kind": "dense", "ff"}
       | {"kind": "moe", "expert": {"ff", "limit"}, "router": {"experts", "identity", "top"}, "shared": {"ff", "limit"}}
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Mapping

from ..errors import ConfigError
from .felosun import _positive_number
from .fields import optional
from .napizen import _number
from .nobodra import MAX_POSITIONS, _positive, _section


def _mask(raw: Mapping[str, Any], where: str) -> int | None:
    return None if raw.get("mask") is None else _positive(_section(raw, "mask", where), "size", where)


@dataclass(frozen=True)
class TamilixLatent:
    heads: int
    dim: int                        # unrotated query/key dims of a head
    rot_dim: int                    # rotated ones
    vdim: int
    q_rank: int
    kv_rank: int
    scale: float
    rot_base: float
    window: int | None = None

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "TamilixLatent":
        sizes = [_positive(raw, name, where) for name in ("heads", "dim", "rot_dim", "vdim", "q_rank", "kv_rank")]
        rot = _section(raw, "rot", where)
        dims, base = _positive(rot, "dims", where), _positive_number(rot, "base", where)
        if dims != sizes[2] or dims % 2:
            raise ConfigError(f"{where}: the rotation covers a head's whole rotated part, so rot.dims must equal rot_dim and be even, got {dims} and {sizes[2]}")
        if base == 1:
            raise ConfigError(f"{where}: rot.base must not be 1")
        return cls(*sizes, _positive_number(raw, "scale", where), base, _mask(raw, where))

    def to_json_dict(self) -> dict:
        out = {"heads": self.heads, "dim": self.dim, "rot_dim": self.rot_dim, "vdim": self.vdim, "q_rank": self.q_rank, "kv_rank": self.kv_rank,
               "scale": self.scale, "rot": {"base": self.rot_base, "dims": self.rot_dim}}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class TamilixAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int | None = None

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "TamilixAttention":
        heads, kv_heads, dim, vdim = (_positive(raw, name, where) for name in ("heads", "kv_heads", "dim", "vdim"))
        if heads % kv_heads:
            raise ConfigError(f"{where}: heads must be a multiple of kv_heads, got {heads} and {kv_heads}")
        return cls(heads, kv_heads, dim, vdim, _positive_number(raw, "scale", where), _mask(raw, where))

    def to_json_dict(self) -> dict:
        out: dict = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale}
        if self.chunk is not None:
            out["mask"] = {"size": self.chunk}
        return out


MIXERS = {"latent_attention": TamilixLatent, "attention": TamilixAttention}


@dataclass(frozen=True)
class TamilixFeedForward:
    kind: str                       # "dense" | "moe"
    ff: int
    limit: float = 0.0
    experts: int = 0
    identity: int = 0
    top: int = 0
    shared_ff: int | None = None
    shared_limit: float | None = None

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], where: str) -> "TamilixFeedForward":
        kind = raw.get("kind")
        if kind == "dense":
            return cls("dense", _positive(raw, "ff", where))
        if kind != "moe":
            raise ConfigError(f"{where}: unknown feed-forward kind {kind!r}; expected one of: dense, moe")
        router, expert = _section(raw, "router", where), _section(raw, "expert", where)
        experts, top = _positive(router, "experts", where), _positive(router, "top", where)
        try:
            identity = optional(router, "identity", int, 0)
        except ConfigError as exc:
            raise ConfigError(f"{where}: {exc}") from None
        if identity < 0 or top > experts + identity:
            raise ConfigError(f"{where}: {top} choices among {experts} experts and {identity} identity experts are not possible")
        shared_ff = shared_limit = None
        if raw.get("shared") is not None:
            shared = _section(raw, "shared", where)
            shared_ff, shared_limit = _positive(shared, "ff", f"{where} shared"), _positive_number(shared, "limit", f"{where} shared")
        return cls("moe", _positive(expert, "ff", where), _positive_number(expert, "limit", where), experts, identity, top, shared_ff, shared_limit)

    def to_json_dict(self) -> dict:
        if self.kind == "dense":
            return {"kind": "dense", "ff": self.ff}
        out = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit},
               "router": {"experts": self.experts, "identity": self.identity, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff, "limit": self.shared_limit}
        return out


@dataclass(frozen=True)
class TamilixLayer:
    type: str                       # "latent_attention" | "attention"
    mixer: Any                      # the dataclass MIXERS names for the type
    mlp: TamilixFeedForward | None
    weights_of: int | None = None

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any], index: int) -> "TamilixLayer":
        where = f"layer {index}"
        if not isinstance(raw, dict):
            raise ConfigError(f"{where} must be an object")
        kind = raw.get("type")
        if kind not in MIXERS:
            raise ConfigError(f"{where}: unknown type {kind!r}; expected one of: {', '.join(MIXERS)}")
        mlp = raw.get("mlp")
        if mlp is not None and not isinstance(mlp, dict):
            raise ConfigError(f"{where}: `mlp` must be an object or null")
        shared = raw.get("weights_of")
        if shared is not None and (not isinstance(shared, int) or isinstance(shared, bool)):
            raise ConfigError(f"{where}: weights_of must be a layer's number")
        return cls(kind, MIXERS[kind].from_dict(_section(raw, "mixer", where), where), None if mlp is None else TamilixFeedForward.from_dict(mlp, where), shared)

    def to_json_dict(self) -> dict:
        out = {"type": self.type, "mixer": self.mixer.to_json_dict(), "mlp": None if self.mlp is None else self.mlp.to_json_dict()}
        if self.weights_of is not None:
            out["weights_of"] = self.weights_of
        return out


@dataclass(frozen=True)
class TamilixConfig:
    vocab_size: int
    width: int
    norm_eps: float
    embedding_scale: float
    layers: tuple
    eos_token_ids: tuple = ()        # the design names no end-of-sequence token: generation runs to its length limit
    model_type: str = "tamilix"

    ARCHITECTURE = "Tamilix"

    @classmethod
    def from_dict(cls, raw: Mapping[str, Any]) -> "TamilixConfig":
        entries = raw.get("layers")
        if not isinstance(entries, list) or not entries:
            raise ConfigError("layers must be a non-empty list")

        def owner_of(index: int, entry) -> int | None:
            """The layer whose weights an entry names, if that is another layer of the list."""
            owner = entry.get("weights_of") if isinstance(entry, dict) else None
            return owner if isinstance(owner, int) and not isinstance(owner, bool) and 0 <= owner < len(entries) and owner != index else None

        merged = []
        for index, entry in enumerate(entries):
            owner = owner_of(index, entry)
            merged.append(entry if owner is None or not isinstance(entries[owner], dict) else dict(entries[owner], **entry))
        layers = tuple(TamilixLayer.from_dict(layer, index) for index, layer in enumerate(merged))
        for index, layer in enumerate(layers):
            if layer.weights_of is None:
                continue
            if owner_of(index, entries[index]) is None:
                raise ConfigError(f"layer {index}: weights_of must name another layer, got {layer.weights_of}")
            owner = layers[layer.weights_of]
            if owner.weights_of is not None:
                raise ConfigError(f"layer {index}: weights_of names layer {layer.weights_of}, which has no tensors of its own")
            if (layer.type, layer.mixer, layer.mlp) != (owner.type, owner.mixer, owner.mlp):
                raise ConfigError(f"layer {index}: a layer that runs with layer {layer.weights_of}'s weights must equal it in type, mixer and mlp")
        scale = 1.0
        if raw.get("embedding") is not None:
            scale = _number(_section(raw, "embedding", "config.json"), "scale", "config.json embedding", 1.0)
        return cls(vocab_size=_positive(raw, "vocab", "config.json"), width=_positive(raw, "width", "config.json"),
                   norm_eps=_positive_number(_section(raw, "norm", "config.json"), "eps", "config.json norm"), embedding_scale=scale, layers=layers)

    def owners(self) -> tuple:
        """The numbers of the layers that have tensors of their own, in order."""
        return tuple(index for index, layer in enumerate(self.layers) if layer.weights_of is None)

    def validate_context_length(self, max_seq_len: int) -> None:
        if not 0 < max_seq_len <= MAX_POSITIONS:
            raise ConfigError(f"max_seq_len must be within 1..{MAX_POSITIONS}, got {max_seq_len}")

    def to_json_dict(self) -> dict:
        return {"architecture": self.ARCHITECTURE, "vocab": self.vocab_size, "width": self.width, "norm": {"eps": self.norm_eps},
                "embedding": {"scale": self.embedding_scale}, "layers": [layer.to_json_dict() for layer in self.layers]}
