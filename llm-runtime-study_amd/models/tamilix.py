"""Tamilix: configuration -> ModelSpec.

Every sublayer stands between two RMS norms: h <- h + norm1b(mixer(norm1(h))), then h <- h + norm2b(feed_forward(norm2(h))).  The
mixer is one of
  "latent_attention"  queries made from a latent row, keys and values from another one that is kept (with one rotated key part shared
                      by the heads, neighbouring pairs rotated); a sliding window; every value gated by a sigmoid of the mixer's input;
  "attention"         grouped-query attention without rotation inside chunks of the sequence: a score loses slope * distance with a
                      fixed slope per head, and a learned sink per head joins the softmax's denominator.
The feed-forward is two matrices with the square of relu between them, or routed experts with a clamped gated activation, chosen by
softmax scores plus a correction and weighted by the scores alone, some of the router's outputs standing for the token itself, with a
shared expert beside them; a layer may have none.  A layer may run with another layer's weights and a cache of its own: such a layer
is a second schedule entry of the layer it names.  The model's norm and the head follow the last layer.

Checkpoint tensors are named without a `.weight` ending: `embed`, `head`, `final.norm`, `l<i>.norm1`, `l<i>.norm1b`, `l<i>.mix.dq`,
`l<i>.mix.dq.norm`, `l<i>.mix.uq`, `l<i>.mix.dkv.norm`, `l<i>.mix.q`, `l<i>.mix.sink`, `l<i>.mlp.up`, `l<i>.mlp.router`,
`l<i>.mlp.correction`, `l<i>.mlp.e<j>.gate`, `l<i>.mlp.shared.up`, i being the layer's number in config.json.
"""

from __future__ import annotations

from ..config.nobodra import MAX_POSITIONS
from ..config.tamilix import TamilixConfig, TamilixLayer
from ..parts import PartSpec
from .felosun import SWISH_ALPHA
from .mutolix import LAYER_NAMES
from .napizen import checkpoint_name
from .spec import ModelSpec, ScheduleEntry


def _mixer(config: TamilixConfig, layer: TamilixLayer) -> PartSpec:
    sizes = layer.mixer
    if layer.type == "attention":
        return PartSpec("gqa_attention", {
            "hidden_size": config.width, "num_heads": sizes.heads, "num_kv_heads": sizes.kv_heads, "head_dim": sizes.dim, "value_dim": sizes.vdim,
            "scale": sizes.scale, "chunk": sizes.chunk, "sink": True, "distance_bias": "linear"})
    return PartSpec("latent_attention", {
        "hidden_size": config.width, "num_heads": sizes.heads, "head_dim": sizes.dim, "rot_dim": sizes.rot_dim, "value_dim": sizes.vdim,
        "q_rank": sizes.q_rank, "kv_rank": sizes.kv_rank, "position": PartSpec("rope_interleaved", {"rotary_dim": sizes.rot_dim, "theta": sizes.rot_base}),
        "norm_eps": config.norm_eps, "scale": sizes.scale, "window": sizes.window, "gate": "value"})


def _feed_forward(config: TamilixConfig, layer: TamilixLayer) -> PartSpec:
    mlp = layer.mlp
    if mlp.kind == "dense":
        return PartSpec("dense_mlp", {"hidden_size": config.width, "intermediate_size": mlp.ff, "activation": "relu_squared"})
    shared = None
    if mlp.shared_ff is not None:
        shared = PartSpec("swiglu", {"hidden_size": config.width, "intermediate_size": mlp.shared_ff, "activation": "clamped",
                                     "alpha": SWISH_ALPHA, "limit": mlp.shared_limit})
    return PartSpec("routed_experts", {
        "hidden_size": config.width, "intermediate_size": mlp.ff, "num_experts": mlp.experts, "identity": mlp.identity, "top": mlp.top,
        "rule": "softmax_scores", "router_bias": True, "bias_name": "correction", "activation": "clamped_gated", "activation_alpha": SWISH_ALPHA,
        "activation_limit": mlp.limit, "shared": shared})


def build_spec(config: TamilixConfig) -> ModelSpec:
    norm = PartSpec("rmsnorm", {"size": config.width, "eps": config.norm_eps})
    owners = config.owners()
    place = {number: index for index, number in enumerate(owners)}
    layers = []
    for number in owners:
        layer = config.layers[number]
        params = {"mixer": _mixer(config, layer), "mixer_norm": norm, "mixer_out_norm": norm, "names": LAYER_NAMES}
        if layer.mlp is not None:
            params["feed_forward"] = _feed_forward(config, layer)
            params["ff_norm"] = params["ff_out_norm"] = norm
        layers.append(PartSpec("sandwich", params))
    schedule = tuple(ScheduleEntry(place[number if layer.weights_of is None else layer.weights_of]) for number, layer in enumerate(config.layers))
    return ModelSpec(
        architecture=TamilixConfig.ARCHITECTURE, vocab_size=config.vocab_size, hidden_size=config.width, layers=tuple(layers),
        schedule=schedule, final_norm=norm, max_positions=MAX_POSITIONS, eos_token_ids=(), embedding_multiplier=config.embedding_scale,
        embedding_name="embed", head_name="head", final_norm_prefix="final.norm", layer_prefix="l{index}", layer_numbers=owners,
        checkpoint_dtype="bfloat16", checkpoint_name=checkpoint_name)
