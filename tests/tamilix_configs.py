"""Small Tamilix configurations of the tests' own, differing from each other in every size, constant and layer order."""

from __future__ import annotations

import json
from pathlib import Path


def dense(ff):
    return {"kind": "dense", "ff": ff}


def experts(ff, limit, count, identity, top, shared=None):
    """shared: (ff, limit) of the shared expert, or None."""
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": count, "identity": identity, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base, window=None, mlp=None):
    mixer = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
             "rot": {"base": base, "dims": rot_dim}}
    if window is not None:
        mixer["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def chunked(heads, kv_heads, dim, vdim, scale, chunk=None, mlp=None):
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk is not None:
        mixer["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": mixer, "mlp": mlp}


def shares(layer, owner):
    """The entry of a layer that runs with layer `owner`'s weights: `layer`'s own entry once more, and whose weights."""
    return dict(json.loads(json.dumps(layer)), weights_of=owner)


def model(vocab, width, eps, embedding_scale, layers):
    return {"architecture": "Tamilix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": embedding_scale}, "layers": layers}


# odd sizes throughout: values narrower and wider than keys, three heads to a key group, chunks and windows that are no multiple of
# anything and shorter than a page, ranks of queries and keys that differ, an expert size that is odd, a layer without feed-forward
_ODD_0 = latent(3, 14, 6, 10, 22, 30, 0.2, 700.0, 13, experts(15, 0.8, 5, 3, 3, shared=(18, 2.0)))
_ODD_1 = chunked(6, 2, 20, 12, 0.21, 9, dense(26))
ODD = model(211, 72, 1e-5, 3.5, [_ODD_0, _ODD_1, shares(_ODD_0, 0), chunked(2, 2, 16, 24, 0.4, 21), latent(5, 8, 2, 18, 40, 11, 0.3, 50.0, 33, dense(31)),
                                 shares(_ODD_1, 1)])
# sizes the matrix-core kernels take: heads of 64, 128 and 32 (values as wide, and narrower), latent rows that are multiples of 8, chunks
# and windows of several pages, more experts than a wave has lanes
_CORES_0 = chunked(4, 2, 64, 64, 0.11, 48, experts(64, 1.0, 66, 9, 3, shared=(96, 1.2)))
_CORES_1 = latent(4, 64, 32, 32, 96, 72, 0.13, 1e4, 24, experts(32, 3.0, 6, 4, 2))
CORES = model(300, 128, 2e-6, 5.0, [_CORES_0, _CORES_1, chunked(2, 1, 128, 64, 0.08, 40, dense(192)), shares(_CORES_1, 1),
                                    chunked(8, 2, 32, 32, 0.2, 70, experts(48, 0.9, 4, 1, 4, shared=(16, 1.0))), shares(_CORES_0, 0)])
# what a model may make equal or one: one head, one key group, one expert beside one identity expert of which one is chosen, a window
# and a chunk of one, one rotated pair, no shared expert, a scale of one, no identity experts at all
_ONES_0 = chunked(1, 1, 8, 8, 0.35, 1, experts(12, 1.0, 1, 1, 1))
_ONES_1 = latent(1, 8, 2, 8, 8, 8, 0.3, 100.0, 1, experts(8, 0.5, 2, 0, 1))
ONES = model(90, 48, 3e-6, 1.0, [_ONES_0, _ONES_1, latent(1, 6, 4, 8, 16, 24, 0.25, 30.0, 5, experts(10, 1.5, 1, 3, 4)), shares(_ONES_0, 0), shares(_ONES_1, 1)])
# sizes no kernel likes: a width, heads, ranks and a vocabulary that are multiples of neither 8 nor 16, 20 query heads on one key
# group, layers that see the whole context, more identity experts than others, a layer that shares the weights of a later one
_AWKWARD_2 = chunked(20, 1, 20, 12, 0.22, 50, experts(26, 1.1, 3, 7, 2, shared=(7, 0.4)))
AWKWARD = model(251, 100, 4e-6, 0.7, [shares(_AWKWARD_2, 2), latent(3, 10, 6, 9, 13, 27, 0.2, 3000.0, None, experts(30, 2.0, 3, 0, 3)), _AWKWARD_2,
                                      chunked(3, 3, 40, 52, 0.16, None, dense(44)), latent(2, 12, 4, 20, 36, 20, 0.3, 20.0, 30)])
# wide enough that prompts go through the products for many rows (the vendor library's in bfloat16) and the grouped products with
# large tiles
_WIDE_0 = latent(8, 64, 32, 64, 192, 128, 0.1, 1e4, 150, experts(128, 1.5, 6, 2, 2, shared=(256, 1.0)))
WIDE = model(1000, 512, 1e-6, 4.0, [_WIDE_0, chunked(4, 2, 96, 96, 0.1, 130, dense(768)), shares(_WIDE_0, 0),
                                    chunked(8, 2, 128, 128, 0.09, 64, experts(256, 1.0, 4, 4, 2))])
ALL = {"odd": ODD, "cores": CORES, "ones": ONES, "awkward": AWKWARD, "wide": WIDE}


def write_folder(raw: dict, seed: int, folder, edit=None) -> Path:
    """A model folder with random weights for `raw`; edit(tensors) may change the tensors before they are written.  Sinks are drawn
    so that they carry weight in the softmax, corrections about as wide as softmax scores are, the router's rows larger so that the
    scores differ."""
    from safetensors.torch import load_file, save_file

    from llm_runtime_study_amd.config import config_from_dict
    from llm_runtime_study_amd.weights import write_model_dir

    folder = Path(folder)
    write_model_dir(config_from_dict(raw), seed=seed, model_dir=folder, init="scaled")
    assert json.loads((folder / "config.json").read_text()) == raw
    tensors = load_file(str(folder / "model.safetensors"))
    for name in list(tensors):
        t = tensors[name].float()
        if name.endswith(".sink"):
            t = t * 20.0 + 1.0
        elif name.endswith(".router"):
            t = t * 1.5
        tensors[name] = t.to(tensors[name].dtype)
    if edit is not None:
        edit(tensors)
    save_file({name: t.contiguous() for name, t in tensors.items()}, str(folder / "model.safetensors"))
    return folder
