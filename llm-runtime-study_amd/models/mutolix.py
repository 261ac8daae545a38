"""Mutolix: configuration -> ModelSpec.

Every sublayer stands between two RMS norms; what it gives out is multiplied by a sigmoid gate of its own input before the second
norm and scaled per column after it: with x = norm1(h), h <- h + ls * norm1b(sublayer(x) * sigmoid(W x + b)).  The mixer is one of
  "mlstm"      a matrix memory with exponential gates and a running maximum (parts/matrix_memory.py);
  "attention"  grouped-query attention over the whole context without rotation: biases on q, k and v, q and k normalised over the
               whole projection, queries whose length grows with the position, scores that lose rate * ln(1 + reach * distance), one
               added to the softmax's denominator (a sink of score zero), and values mixed with those of the first such layer.
The feed-forward is two matrices with the xIELU activation (two learned numbers) between them; a layer may have none.  The model's
norm and the head follow the last layer.

Checkpoint tensors are named without a `.weight` ending: `embed`, `head`, `final.norm`, `l<i>.norm1`, `l<i>.norm1b`, `l<i>.rg1`,
`l<i>.rg1.b`, `l<i>.ls1`, `l<i>.mix.q`, `l<i>.mix.q.b`, `l<i>.mix.q.norm`, `l<i>.mix.r1`, `l<i>.mix.vmix`, `l<i>.mix.i.b`,
`l<i>.mlp.up`, `l<i>.mlp.act`.
"""

from __future__ import annotations

from ..config.mutolix import MutolixConfig
from ..config.nobodra import MAX_POSITIONS
from ..parts import PartSpec
from .felosun import checkpoint_name as _short_name
from .spec import ModelSpec, ScheduleEntry

LAYER_NAMES = {"mixer": "mix", "feed_forward": "mlp", "mixer_norm": "norm1", "mixer_out_norm": "norm1b", "ff_norm": "norm2",
               "ff_out_norm": "norm2b", "mixer_gate": "rg1", "ff_gate": "rg2", "mixer_scale": "ls1", "ff_scale": "ls2"}


def checkpoint_name(name: str) -> str:
    """The checkpoint's name of the tensor that the parts call `name`."""
    return _short_name(name).replace("distance_rate", "r1").replace("distance_reach", "r2").replace("value_mix", "vmix")


def _mixer(config: MutolixConfig, index: int) -> PartSpec:
    sizes = config.layers[index].mixer
    if config.layers[index].type == "mlstm":
        return PartSpec("mlstm", {"hidden_size": config.width, "num_heads": sizes.heads, "head_dim": sizes.dim, "value_dim": sizes.vdim,
                                  "gate_cap": sizes.gate_cap, "norm_eps": config.norm_eps})
    mix = None if not sizes.v_mix else "first" if index == config.first_mixing_layer() else "later"
    return PartSpec("gqa_attention", {
        "hidden_size": config.width, "num_heads": sizes.heads, "num_kv_heads": sizes.kv_heads, "head_dim": sizes.dim, "value_dim": sizes.vdim,
        "bias": True, "qk_norm": True, "qk_norm_eps": config.norm_eps, "norm_over": "projection", "scale": sizes.scale, "sink": 0.0,
        "query_temperature": None if sizes.temp_every is None else (sizes.temp_coef, sizes.temp_every), "value_mix": mix, "distance_bias": True})


def build_spec(config: MutolixConfig) -> ModelSpec:
    norm = PartSpec("rmsnorm", {"size": config.width, "eps": config.norm_eps})
    layers = []
    for index, layer in enumerate(config.layers):
        params = {"mixer": _mixer(config, index), "mixer_norm": norm, "mixer_out_norm": norm, "gated": True, "scaled": True, "names": LAYER_NAMES}
        if layer.ff is not None:
            params["feed_forward"] = PartSpec("dense_mlp", {"hidden_size": config.width, "intermediate_size": layer.ff, "activation": "xielu"})
            params["ff_norm"] = params["ff_out_norm"] = norm
        layers.append(PartSpec("sandwich", params))
    return ModelSpec(
        architecture=MutolixConfig.ARCHITECTURE, vocab_size=config.vocab_size, hidden_size=config.width, layers=tuple(layers),
        schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm, max_positions=MAX_POSITIONS, eos_token_ids=(),
        embedding_multiplier=config.embedding_scale, embedding_name="embed", head_name="head", final_norm_prefix="final.norm",
        layer_prefix="l{index}", checkpoint_dtype="bfloat16", checkpoint_name=checkpoint_name)
