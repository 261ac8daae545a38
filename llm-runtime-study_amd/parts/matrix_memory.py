"""Matrix memory with exponential gates (the mLSTM of xLSTM): a mixer whose memory is one matrix per head, written by weighted
outer products, with a running normaliser beside it.

For a token with input x, per head:
    q, k, v = W_q x * head_dim ** -0.5, W_k x, W_v x
    i       = soft(W_i x + b_i)                                       the log of the input gate
    f       = log(sigmoid(soft(W_f x + b_f)))                         the log of the forget gate;  soft(z) = cap * tanh(z / cap)
    m'      = max(f + m, i)                                           a running maximum, 0 at a sequence's start
    S <- exp(f + m - m') S + exp(i - m') k v^T                        S [head_dim, value_dim], zero at the start
    n <- exp(f + m - m') n + exp(i - m') k
    o       = S^T q / (max(|n . q|, exp(-m')) + 1e-6)
    out     = W_o (rms_norm(o) * norm_weight * sigmoid(W_g x))        the norm per head over value_dim, a weight per value of every head
The gates, m, S, n, the read-out and its gated norm are float32 in every run; the six input projections are one stacked product
written in float32.

The recurrence is the scan of the gated delta rule's kernels without its correction and with a weight on what is written
(csrc/delta.hip, RULE_WEIGHTED); n is one more column of S, whose value is always one.  A request keeps one float32 row: the matrices of
all heads in the order the scan's threads hold them, then m of every head (`StateNeed`; the cache manager clears a row at
admission, which is what a sequence starts from).

The scan is sequential over a request's tokens.  bfloat16 runs take another form for steps that hold more than single tokens: chunks
of 64 tokens on the matrix cores, the state carried between them in float32 (csrc/mlstm_chunks.hip).  float32 runs always scan, so
that their sums do not depend on how a prompt was cut.
"""

from __future__ import annotations

import torch

from ..kernels import ops
from .base import Part, StateNeed, TensorSpec, register
from .delta import STATE_LANES, state_rows
from .linear import linear, materialize, rows_of


class MatrixMemory(Part):
    CHUNK_FROM = 16     # tokens of a step beyond one a request from which on the chunked form serves a bfloat16 run

    graph_safe = True   # launches only this package's kernels on arena buffers, reads the step's data on the device
    plan_safe = True
    can_overwrite = True
    carries_rows = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, gate_cap: float, norm_eps: float):
        for name, value in (("hidden_size", hidden_size), ("num_heads", num_heads), ("head_dim", head_dim), ("value_dim", value_dim)):
            if value <= 0:
                raise ValueError(f"{name} must be positive, got {value}")
        if head_dim > 256:
            raise ValueError(f"the scan kernel takes head_dim up to 256, got {head_dim}")
        if not gate_cap > 0:
            raise ValueError(f"gate_cap must be positive, got {gate_cap}")
        if norm_eps <= 0:
            raise ValueError(f"norm_eps must be positive, got {norm_eps}")
        self.hidden_size, self.num_heads, self.head_dim, self.value_dim = hidden_size, num_heads, head_dim, value_dim
        self.gate_cap, self.norm_eps = float(gate_cap), norm_eps
        self.w_in = self.w_o = self.i_bias = self.f_bias = self.norm = None

    def _projections(self):
        qk, v = self.num_heads * self.head_dim, self.num_heads * self.value_dim
        return (("q_proj", qk), ("k_proj", qk), ("v_proj", v), ("g_proj", v), ("i_proj", self.num_heads), ("f_proj", self.num_heads))

    def tensors(self):
        specs = {f"{name}.weight": TensorSpec((width, self.hidden_size)) for name, width in self._projections()}
        specs["i_proj.bias"] = TensorSpec((self.num_heads,), role="bias")
        specs["f_proj.bias"] = TensorSpec((self.num_heads,), role="bias")
        specs["norm.weight"] = TensorSpec((self.num_heads * self.value_dim,), role="norm")
        specs["o_proj.weight"] = TensorSpec((self.hidden_size, self.num_heads * self.value_dim))
        return specs

    def bind(self, weights, dtype):
        self.w_in = self.stack_rows([weights[f"{name}.weight"] for name, _ in self._projections()], dtype)
        self.i_bias, self.f_bias = weights["i_proj.bias"].float().contiguous(), weights["f_proj.bias"].float().contiguous()
        self.norm = weights["norm.weight"].float().contiguous()
        self.w_o = weights["o_proj.weight"].to(dtype).contiguous()

    def weight_bytes(self):
        return (self.w_in.numel() + self.w_o.numel()) * self.w_o.element_size()

    def flops(self, tokens, pairs):
        # the projections, and per token and head the state's update and its read-out
        return super().flops(tokens, pairs) + 4.0 * tokens * self.num_heads * self.head_dim * (self.value_dim + 1)

    def state_floats(self) -> int:
        return self.num_heads * state_rows(self.head_dim) * STATE_LANES * (self.value_dim + 1) + self.num_heads

    def cache_need(self):
        return StateNeed((self.state_floats(),), torch.float32)

    def forward(self, ctx, x, residual, cache, then_norm=None, accumulate: bool = True):
        if cache is None or cache.state is None:
            raise ValueError("the matrix memory needs a state row per request")
        t, heads = rows_of(x), self.num_heads
        x = materialize(ctx, x)
        proj = ctx.scratch("mlstm_proj", (t, self.w_in.shape[0]), torch.float32)
        linear(ctx, proj, x, self.w_in)
        self.hand_out_carried(ctx, proj)
        out = ctx.scratch("mlstm_out", (t, heads * self.value_dim), ctx.dtype)
        floors = ctx.scratch("mlstm_floors", (t, heads), torch.float32)
        raw = ctx.scratch("mlstm_read_out", (t, heads * (self.value_dim + 1)), torch.float32)
        if ctx.dtype == torch.bfloat16 and t - ctx.R >= self.CHUNK_FROM:
            packs = tuple(ctx.scratch(f"mlstm_pack{number}", (size,), torch.float32 if number == 3 else torch.bfloat16)
                          for number, size in enumerate(ops.mlstm_pack_sizes(t, ctx.R, heads, self.head_dim)))
            maxima = ctx.scratch("mlstm_maxima", (ctx.R, heads), torch.float32)
            ops.mlstm_chunks(out, proj, cache.state, ctx.token_request, ctx.cu_seqlens_q, ctx.slot_ids, ctx.R, heads, self.head_dim, self.value_dim,
                             self.i_bias, self.f_bias, self.gate_cap, self.norm, self.norm_eps, maxima, floors, raw, packs, ctx.single_rows)
        else:
            gates = ctx.scratch("mlstm_gates", (t, 2 * heads), torch.float32)
            ops.mlstm(out, proj, cache.state, ctx.cu_seqlens_q, ctx.slot_ids, ctx.R, heads, self.head_dim, self.value_dim, self.i_bias, self.f_bias,
                      self.gate_cap, self.norm, self.norm_eps, gates, floors, raw)
        linear(ctx, residual, out, self.w_o, accumulate=accumulate)
        return None


register("mixer", "mlstm", MatrixMemory)
