"""Whole-sequence Tamilix forward, written out mechanism by mechanism with plain tensor operations.

No cache, no batching: every call recomputes one whole sequence, one (head, query) at a time where a mask is involved, one
(token, expert) at a time where tokens are routed.  CPU tensors in the dtype of the weights passed in (float64 in the tests).
Shares nothing with the package: names of checkpoint tensors and config.json keys are read here on their own, and the keys and
values of latent attention are made for every position as the definition has them (the package never makes them).

Notation: n tokens, width W.  A layer is x <- x + norm1b(mixer(norm1(x))), then x <- x + norm2b(ff(norm2(x))).
"""

from __future__ import annotations

import json
import math
import struct
from pathlib import Path

import torch


def rms(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) * weight over the last dimension."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * weight


def logistic(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def turn_neighbours(x: torch.Tensor, base: float, dims: int, first_position: int = 0) -> torch.Tensor:
    """x [n, ..., >= dims]: dims (2i, 2i + 1) of token t are turned by (first_position + t) * base^(-2i / dims)."""
    out = x.clone()
    for t in range(x.shape[0]):
        for i in range(dims // 2):
            angle = (first_position + t) * base ** (-2.0 * i / dims)
            u, v = x[t, ..., 2 * i], x[t, ..., 2 * i + 1]
            out[t, ..., 2 * i] = u * math.cos(angle) - v * math.sin(angle)
            out[t, ..., 2 * i + 1] = v * math.cos(angle) + u * math.sin(angle)
    return out


def in_window(i: int, j: int, size: int | None) -> bool:
    """A query at i sees itself and the size - 1 positions before it (None: all of them)."""
    return 0 <= i - j and (size is None or i - j < size)


def in_chunk(i: int, j: int, size: int | None) -> bool:
    """A query at i sees the positions up to its own of its own chunk; chunks are size positions long, from position 0 on."""
    return j <= i and (size is None or i // size == j // size)


def slope(head: int, heads: int) -> float:
    return 2.0 ** (-8.0 * (head + 1) / heads)


def softmax_with(scores: torch.Tensor, sink: float | None = None) -> torch.Tensor:
    """exp(scores) over their sum, plus exp(sink) in the sum if there is one."""
    top = float(scores.max()) if sink is None else max(float(scores.max()), sink)
    raised = torch.exp(scores - top)
    return raised / (raised.sum() + (0.0 if sink is None else math.exp(sink - top)))


def size_of(m: dict) -> int | None:
    return None if m.get("mask") is None else m["mask"]["size"]


def latent_attention(x: torch.Tensor, w: dict, m: dict, eps: float, weights_out: list | None = None) -> torch.Tensor:
    """w: dq, dq.norm, uq, dkv, dkv.norm, uk, uv, g, o.  Keys and values of a head from the latent row, one rotated key part for all."""
    n, heads, d, r, e, c = x.shape[0], m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    queries = (rms(x @ w["dq"].T, w["dq.norm"], eps) @ w["uq"].T).view(n, heads, d + r)
    down = x @ w["dkv"].T
    latent = rms(down[:, :c], w["dkv.norm"], eps)
    shared = turn_neighbours(down[:, c:], m["rot"]["base"], m["rot"]["dims"])
    turned = turn_neighbours(queries[..., d:], m["rot"]["base"], m["rot"]["dims"])
    out = torch.zeros(n, heads, e, dtype=x.dtype)
    for h in range(heads):
        keys = latent @ w["uk"][h * d:(h + 1) * d].T
        values = latent @ w["uv"][h * e:(h + 1) * e].T
        for i in range(n):
            seen = [j for j in range(n) if in_window(i, j, size_of(m))]
            weights = softmax_with((keys[seen] @ queries[i, h, :d] + shared[seen] @ turned[i, h]) * m["scale"])
            if weights_out is not None:
                weights_out.append((h, i, seen, weights))
            out[i, h] = weights @ values[seen]
    return (out.reshape(n, heads * e) * logistic(x @ w["g"].T)) @ w["o"].T


def attention(x: torch.Tensor, w: dict, m: dict, weights_out: list | None = None) -> torch.Tensor:
    """w: q, k, v, sink, o.  No rotation: a score loses slope * distance; a chunk's keys only; a sink a head in the denominator."""
    n, heads, groups, d, e = x.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q, k, v = (x @ w["q"].T).view(n, heads, d), (x @ w["k"].T).view(n, groups, d), (x @ w["v"].T).view(n, groups, e)
    out = torch.zeros(n, heads, e, dtype=x.dtype)
    for h in range(heads):
        g = h // (heads // groups)
        for i in range(n):
            seen = [j for j in range(n) if in_chunk(i, j, size_of(m))]
            distance = torch.tensor([float(i - j) for j in seen], dtype=x.dtype)
            weights = softmax_with((k[seen, g] @ q[i, h]) * m["scale"] - slope(h, heads) * distance, float(w["sink"][h]))
            if weights_out is not None:
                weights_out.append((h, i, seen, weights))
            out[i, h] = weights @ v[seen, g]
    return out.reshape(n, heads * e) @ w["o"].T


def dense_ff(x: torch.Tensor, up: torch.Tensor, down: torch.Tensor) -> torch.Tensor:
    z = x @ up.T
    return torch.where(z > 0, z * z, torch.zeros_like(z)) @ down.T


def expert(x: torch.Tensor, gate: torch.Tensor, up: torch.Tensor, down: torch.Tensor, limit: float) -> torch.Tensor:
    """g = min(W_gate x, limit); u = clamp(W_up x, -limit, limit); W_down (g sigmoid(1.702 g) (u + 1))."""
    g = torch.clamp(x @ gate.T, max=limit)
    u = torch.clamp(x @ up.T, min=-limit, max=limit)
    return (g * logistic(1.702 * g) * (u + 1.0)) @ down.T


def choose(logits: torch.Tensor, correction: torch.Tensor, top: int, margins: list | None = None):
    """Per token: the indices of the `top` largest softmax scores with the correction added, and those scores without it."""
    chosen, shares = [], []
    for z in logits:
        raised = torch.exp(z - z.max())
        s = raised / raised.sum()
        choice = s + correction
        ranked = sorted(range(len(z)), key=lambda e: (-float(choice[e]), e))
        if margins is not None and top < len(ranked):
            margins.append(float(choice[ranked[top - 1]] - choice[ranked[top]]))
        chosen.append(ranked[:top])
        shares.append([float(s[e]) for e in ranked[:top]])
    return chosen, shares


def routed_ff(x: torch.Tensor, w: dict, mlp: dict, margins: list | None = None, picks: list | None = None) -> torch.Tensor:
    """The weighted outputs of the chosen experts (those behind the last real one give x itself), and the shared expert's."""
    router = mlp["router"]
    chosen, shares = choose(x @ w["router"].T, w["correction"], router["top"], margins)
    if picks is not None:
        picks.append(chosen)
    out = torch.zeros_like(x)
    for t in range(x.shape[0]):
        for e, share in zip(chosen[t], shares[t]):
            if e >= router["experts"]:
                out[t] += share * x[t]
            else:
                out[t] += share * expert(x[t], w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], mlp["expert"]["limit"])
    if mlp.get("shared") is not None:
        out = out + expert(x, w["shared.gate"], w["shared.up"], w["shared.down"], mlp["shared"]["limit"])
    return out


def under(weights: dict, prefix: str) -> dict:
    return {name[len(prefix):]: t for name, t in weights.items() if name.startswith(prefix)}


def forward(weights: dict, raw: dict, ids, streams: list | None = None, margins: list | None = None, picks: list | None = None) -> torch.Tensor:
    """Logits [n, vocab] of one sequence from position 0; streams: gets the stream after every layer."""
    eps = raw["norm"]["eps"]
    x = weights["embed"][torch.as_tensor(ids, dtype=torch.long)] * raw["embedding"]["scale"]
    for index, layer in enumerate(raw["layers"]):
        w = under(weights, f"l{layer.get('weights_of', index)}.")
        mix, seen = under(w, "mix."), rms(x, w["norm1"], eps)
        y = latent_attention(seen, mix, layer["mixer"], eps) if layer["type"] == "latent_attention" else attention(seen, mix, layer["mixer"])
        x = x + rms(y, w["norm1b"], eps)
        mlp = layer.get("mlp")
        if mlp is not None:
            ff, seen = under(w, "mlp."), rms(x, w["norm2"], eps)
            y = dense_ff(seen, ff["up"], ff["down"]) if mlp["kind"] == "dense" else routed_ff(seen, ff, mlp, margins, picks)
            x = x + rms(y, w["norm2b"], eps)
        if streams is not None:
            streams.append(x.clone())
    return rms(x, weights["final.norm"], eps) @ weights["head"].T


def read_safetensors(path, dtype=torch.float64) -> dict:
    """name -> tensor from a safetensors file (8-byte length, a JSON header, the data); bfloat16 and float32 data widened to
    `dtype`, int32 tables left as they are."""
    data = Path(path).read_bytes()
    (size,) = struct.unpack("<Q", data[:8])
    header = json.loads(data[8:8 + size])
    kinds = {"BF16": torch.bfloat16, "F32": torch.float32, "I32": torch.int32}
    out = {}
    for name, entry in header.items():
        if name == "__metadata__":
            continue
        lo, hi = entry["data_offsets"]
        t = torch.frombuffer(bytearray(data[8 + size + lo:8 + size + hi]), dtype=kinds[entry["dtype"]]).reshape(entry["shape"])
        out[name] = t if entry["dtype"] == "I32" else t.to(dtype)
    return out


def load_model_dir(folder, dtype=torch.float64):
    folder = Path(folder)
    return read_safetensors(folder / "model.safetensors", dtype), json.loads((folder / "config.json").read_text())
