"""Small Mutolix configurations of the tests' own, differing from each other in every size, constant and layer order."""

from __future__ import annotations

import json
from pathlib import Path


def memory(heads, dim, vdim, gate_cap, ff=None):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": gate_cap},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def attention(heads, kv_heads, dim, vdim, scale, q_temp=None, v_mix=False, ff=None):
    """q_temp: (coef, every)."""
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "v_mix": v_mix}
    if q_temp is not None:
        mixer["q_temp"] = {"coef": q_temp[0], "every": q_temp[1]}
    return {"type": "attention", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def model(vocab, width, eps, embedding_scale, layers):
    return {"architecture": "Mutolix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embedding_scale}, "layers": layers}


# odd sizes throughout: values wider than keys, three heads to a key group, a temperature that steps every five positions, an odd
# inner size, an attention layer without temperature and mixed values between two that have them, a memory with a feed-forward
ODD = model(211, 72, 1e-5, 3.5, [
    attention(6, 2, 20, 40, 0.21, q_temp=(0.7, 5), v_mix=True, ff=22),
    memory(3, 10, 18, 4.0),
    attention(2, 2, 16, 16, 0.3),
    memory(2, 24, 12, 9.0, ff=30),
    attention(8, 4, 12, 20, 0.25, q_temp=(0.2, 64), v_mix=True, ff=15),
])
# sizes the matrix-core kernels take: heads of 64, 128, 32 with values half as wide, as wide, and a quarter as wide; memories whose
# keys fill the padded sizes
CORES = model(300, 128, 2e-6, 6.0, [
    memory(2, 64, 64, 12.0),
    attention(4, 2, 64, 32, 0.12, q_temp=(0.3, 24), v_mix=True, ff=96),
    attention(2, 1, 128, 64, 0.08, q_temp=(0.5, 33), v_mix=True, ff=64),
    memory(1, 128, 48, 7.0),
    attention(4, 1, 64, 64, 0.11, v_mix=True),
    attention(8, 2, 32, 32, 0.2, q_temp=(1.0, 16), v_mix=True, ff=80),
])
# what a model may make equal or one: one head, one key group, keys and values of one number, a temperature that steps at every
# position, an embedding scale of one, one layer that mixes (and so has nothing to mix with)
ONES = model(90, 48, 3e-6, 1.0, [
    memory(1, 1, 1, 1.0, ff=12),
    attention(1, 1, 8, 8, 0.35, q_temp=(0.4, 1), v_mix=True, ff=1),
    memory(1, 1, 5, 30.0),
    memory(4, 3, 1, 2.0),
])
# sizes no kernel likes: a width, heads and a vocabulary that are multiples of neither 8 nor 16, 20 query heads on one key group, keys
# of a memory beyond 128
AWKWARD = model(251, 100, 4e-6, 0.7, [
    attention(20, 1, 20, 12, 0.22, q_temp=(-0.05, 7), v_mix=True, ff=26),
    memory(5, 130, 7, 8.0),
    attention(3, 3, 36, 52, 0.16, ff=9),
    attention(6, 3, 40, 4, 0.15, v_mix=True),
])
# wide enough that prompts go through the products for many rows (the vendor library's in bfloat16)
WIDE = model(1000, 512, 1e-6, 5.0, [
    memory(2, 256, 96, 15.0),
    attention(8, 2, 64, 64, 0.125, q_temp=(0.5, 100), v_mix=True, ff=768),
    attention(4, 2, 96, 64, 0.1, v_mix=True, ff=512),
    memory(4, 64, 128, 10.0, ff=640),
])
ALL = {"odd": ODD, "cores": CORES, "ones": ONES, "awkward": AWKWARD, "wide": WIDE}


def lively(name: str, t):
    """Random tensors made so that every mechanism carries weight: forget gates mostly open and of different lengths, biases by distance from
    almost none to strong, mixed values about half and half, numbers of the activation on both sides of zero."""
    import torch

    t = t.float()
    if name.endswith(".f.b"):
        return 2.0 + 20.0 * t
    if name.endswith(".i.b"):
        return 10.0 * t
    if name.endswith(".r1"):
        return torch.linspace(0.02, 2.0, t.numel()) * t
    if name.endswith(".r2"):
        return torch.linspace(0.5, 0.05, t.numel()) * t
    if name.endswith(".vmix"):
        return 0.4 + t
    if name.endswith(".act"):
        return 8.0 * t
    if name.endswith((".rg1", ".rg2")):
        return 2.0 * t
    return t


def write_folder(raw: dict, seed: int, folder, edit=None) -> Path:
    """A model folder with random weights for `raw`; edit(tensors) may change the tensors before they are written."""
    from safetensors.torch import load_file, save_file

    from llm_runtime_study_amd.config import config_from_dict
    from llm_runtime_study_amd.weights import write_model_dir

    folder = Path(folder)
    write_model_dir(config_from_dict(raw), seed=seed, model_dir=folder, init="scaled")
    assert json.loads((folder / "config.json").read_text()) == raw
    tensors = load_file(str(folder / "model.safetensors"))
    for name in list(tensors):
        tensors[name] = lively(name, tensors[name]).to(tensors[name].dtype)
    if edit is not None:
        edit(tensors)
    save_file({name: t.contiguous() for name, t in tensors.items()}, str(folder / "model.safetensors"))
    return folder
