"""Whole-sequence Mutolix forward, written out mechanism by mechanism with plain tensor operations.

No cache, no batching: every call recomputes one whole sequence.  CPU tensors in the dtype of the weights passed in (float64
in the tests).  Shares nothing with the package: names of checkpoint tensors and config.json keys are read here on their own.

Notation: n tokens, width W.  One update of the stream x by a sublayer f with norms a (before) and b (after):
    u = a(x);  y = f(u) * logistic(R u + r);  x <- x + s * b(y)          (R, r: the residual's gate; s: the layer scale)
"""

from __future__ import annotations

import json
import struct
from pathlib import Path

import torch


def rms_norm(x: torch.Tensor, weight: torch.Tensor | None, eps: float) -> torch.Tensor:
    """x / sqrt(mean(x^2) + eps) over the last dimension (eps under the root), times a weight if there is one."""
    y = x / torch.sqrt(x.pow(2).mean(-1, keepdim=True) + eps)
    return y if weight is None else y * weight


def logistic(x: torch.Tensor) -> torch.Tensor:
    return 1.0 / (1.0 + torch.exp(-x))


def softplus(x: torch.Tensor) -> torch.Tensor:
    return torch.clamp(x, min=0) + torch.log1p(torch.exp(-x.abs()))


def log_gates(u: torch.Tensor, w: dict, cap: float):
    """(log input gates, log forget gates) [n, heads]: both capped by cap * tanh(z / cap), the second then log(logistic(.))."""
    def soft(z):
        return cap * torch.tanh(z / cap)

    return soft(u @ w["i"].T + w["i.b"]), -softplus(-soft(u @ w["f"].T + w["f.b"]))


def matrix_memory(q, k, v, i, f, record: list | None = None) -> torch.Tensor:
    """One head: q, k [n, d], v [n, e], log gates i, f [n] -> read-outs [n, e], token by token with the running maximum m."""
    n, d = q.shape
    e = v.shape[1]
    S, norm, m = torch.zeros(d, e, dtype=q.dtype), torch.zeros(d, dtype=q.dtype), torch.zeros((), dtype=q.dtype)
    out = torch.zeros(n, e, dtype=q.dtype)
    for t in range(n):
        before, m = m, torch.maximum(f[t] + m, i[t])
        old, new = torch.exp(f[t] + before - m), torch.exp(i[t] - m)
        S = old * S + new * torch.outer(k[t], v[t])
        norm = old * norm + new * k[t]
        out[t] = (S.T @ q[t]) / (torch.maximum((norm @ q[t]).abs(), torch.exp(-m)) + 1e-6)
        if record is not None:
            record.append((S.clone(), norm.clone(), float(m)))
    return out


def mlstm(u: torch.Tensor, w: dict, m: dict, eps: float) -> torch.Tensor:
    n, heads, d, e = u.shape[0], m["heads"], m["dim"], m["vdim"]
    q = (u @ w["q"].T).view(n, heads, d) * d ** -0.5
    k, v = (u @ w["k"].T).view(n, heads, d), (u @ w["v"].T).view(n, heads, e)
    i, f = log_gates(u, w, m["gate_cap"])
    o = torch.stack([matrix_memory(q[:, h], k[:, h], v[:, h], i[:, h], f[:, h]) for h in range(heads)], 1)
    o = rms_norm(o, None, eps).reshape(n, heads * e) * w["norm"]
    return (o * logistic(u @ w["g"].T)) @ w["o"].T


def temperature(positions: torch.Tensor, q_temp: dict | None, dtype) -> torch.Tensor:
    """What a query is multiplied by at each position: grows by steps of `every` positions."""
    if q_temp is None:
        return torch.ones(len(positions), dtype=dtype)
    steps = torch.tensor([(int(p) + 1) // q_temp["every"] for p in positions], dtype=dtype)
    return 1.0 + q_temp["coef"] * torch.log(steps + 1.0)


def distance_bias(i: int, r1, r2, dtype) -> torch.Tensor:
    """What is taken off the scores of query position i, for key positions 0 .. i."""
    far = torch.arange(i, -1, -1, dtype=dtype)
    return r1 * torch.log(1.0 + r2 * far)


def attention(u: torch.Tensor, w: dict, m: dict, eps: float, first_values: list | None, weights_out: list | None = None) -> torch.Tensor:
    """first_values: a list that the layers with v_mix share; the first of them puts its values there, the others mix."""
    n, heads, groups, d, e = u.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rms_norm(u @ w["q"].T + w["q.b"], w["q.norm"], eps).view(n, heads, d)
    k = rms_norm(u @ w["k"].T + w["k.b"], w["k.norm"], eps).view(n, groups, d)
    v = u @ w["v"].T + w["v.b"]                                          # [n, groups * e]: mixed value by value
    q = q * temperature(torch.arange(n), m.get("q_temp"), u.dtype)[:, None, None]
    if m.get("v_mix"):
        if first_values:
            v = (1.0 - w["vmix"]) * v + w["vmix"] * first_values[0]
        else:
            first_values.append(v)
    v = v.view(n, groups, e)
    out = torch.zeros(n, heads, e, dtype=u.dtype)
    for h in range(heads):
        g = h // (heads // groups)
        for i in range(n):
            scores = (k[: i + 1, g] @ q[i, h]) * m["scale"] - distance_bias(i, w["r1"][h], w["r2"][h], u.dtype)
            top = torch.clamp(scores.max(), min=0.0)
            weights = torch.exp(scores - top)
            weights = weights / (torch.exp(-top) + weights.sum())       # the one in the denominator: a key of score 0 without value
            if weights_out is not None:
                weights_out.append((h, i, weights))
            out[i, h] = weights @ v[: i + 1, g]
    return out.reshape(n, heads * e) @ w["o"].T


def xielu(z: torch.Tensor, p, q) -> torch.Tensor:
    above = softplus(p) * z * z + z / 2
    below = (0.5 + softplus(q)) * (torch.expm1(torch.clamp(z, max=0)) - torch.clamp(z, max=0)) + z / 2
    return torch.where(z > 0, above, below)


def feed_forward(u: torch.Tensor, w: dict) -> torch.Tensor:
    return xielu(u @ w["up"].T, w["act"][0], w["act"][1]) @ w["down"].T


def under(weights: dict, prefix: str) -> dict:
    return {name[len(prefix):]: t for name, t in weights.items() if name.startswith(prefix)}


def update(x, w, number: int, sublayer, eps: float) -> torch.Tensor:
    u = rms_norm(x, w[f"norm{number}"], eps)
    y = sublayer(u) * logistic(u @ w[f"rg{number}"].T + w[f"rg{number}.b"])
    return x + w[f"ls{number}"] * rms_norm(y, w[f"norm{number}b"], eps)


def forward(weights: dict, raw: dict, ids, streams: list | None = None) -> torch.Tensor:
    """Logits [n, vocab] of one sequence from position 0; streams: gets the stream after every layer."""
    ids = torch.as_tensor(ids, dtype=torch.long)
    eps = raw["norm"]["eps"]
    x = weights["embed"][ids] * raw["embedding"]["scale"]
    first_values: list = []
    for index, layer in enumerate(raw["layers"]):
        w, m = under(weights, f"l{index}."), layer["mixer"]
        mix, mlp = under(w, "mix."), under(w, "mlp.")
        if layer["type"] == "mlstm":
            x = update(x, w, 1, lambda u: mlstm(u, mix, m, eps), eps)
        else:
            x = update(x, w, 1, lambda u: attention(u, mix, m, eps, first_values), eps)
        if layer.get("mlp") is not None:
            x = update(x, w, 2, lambda u: feed_forward(u, mlp), eps)
        if streams is not None:
            streams.append(x.clone())
    return rms_norm(x, weights["final.norm"], eps) @ weights["head"].T


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
    raw = json.loads((folder / "config.json").read_text())
    return read_safetensors(folder / "model.safetensors", dtype), raw
