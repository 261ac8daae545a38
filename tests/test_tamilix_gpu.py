"""Tamilix on the GPU against the plain implementation (tests/plain/tamilix.py): each mechanism and kernel alone (requests of unequal
length stepped side by side, pages given back and used again), then whole models of the tests' own sizes under every way of cutting
their requests into steps, keys planted on either side of a window's and a chunk's edge and at page borders, long decoding, and greedy
generation through Engine and scheduler."""

import math

import numpy as np
import pytest
import torch

from tests import tamilix_configs as configs
from tests import traces
from tests.plain import tamilix as plain
from tests.test_felosun_gpu import LENGTHS, bf16_values, part_weights, step_through
from tests.test_felosun_gpu import short as short_name
from tests.test_parts_gpu import PartHarness, close
from tests.test_replay_gpu import round64, run_replay

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


def short(name: str) -> str:
    name = short_name(name)
    return name[:-len("_norm")] + ".norm" if name.endswith("_norm") else name


def bound(part, w, dtype):
    for name, spec in part.tensors().items():
        if spec.role == "norm":
            w[name] = (1.0 + 0.3 * w[name]).to(torch.bfloat16).double()
    part.bind({name: t.to(torch.bfloat16).cuda() for name, t in w.items()}, dtype)
    return {short(name): t for name, t in w.items()}


# ------------------------------------------------------------------------------------- attention in chunks
CHUNKED_SHAPES = [
    # heads, kv, d, e, scale, chunk
    (4, 2, 16, 24, 0.3, None),      # values wider than keys, the whole context
    (6, 2, 32, 16, 0.2, 9),         # chunks shorter than a page, values narrower
    (2, 1, 64, 64, 0.125, 16),      # chunks of just a page
    (4, 4, 64, 64, 0.125, 20),      # chunks that begin inside pages
    (2, 2, 128, 128, 0.09, 21),
    (8, 2, 128, 64, 0.09, None),    # heads of 128 with narrower values, the whole context
    (1, 1, 8, 8, 0.35, 1),          # a chunk of one
    (5, 1, 48, 40, 0.15, 33),       # head sizes that are no power of two
    (16, 1, 32, 32, 0.2, 40),       # sixteen heads on one key group
    (12, 4, 96, 96, 0.1, 24),
    (3, 3, 20, 20, 0.25, 17),       # a head size that is no multiple of eight
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,groups,d,e,scale,chunk", CHUNKED_SHAPES)
def test_attention_in_chunks_with_slopes_and_sinks_part(dtype, heads, groups, d, e, scale, chunk):
    from llm_runtime_study_amd.parts import PartSpec, create

    width = 56
    part = create("mixer", PartSpec("gqa_attention", {"hidden_size": width, "num_heads": heads, "num_kv_heads": groups, "head_dim": d, "value_dim": e,
                                                     "scale": scale, "chunk": chunk, "sink": True, "distance_bias": "linear"}))
    w = part_weights(part, 50)
    w["sink"] = (w["sink"] * 3.0 + 1.0).to(torch.bfloat16).double()          # sinks that weigh as much as a handful of keys
    named = bound(part, w, dtype)
    assert set(named) == {"q", "k", "v", "sink", "o"}
    m = {"heads": heads, "kv_heads": groups, "dim": d, "vdim": e, "scale": scale}
    if chunk is not None:
        m["mask"] = {"size": chunk}
    inputs = {key: bf16_values(n, width, seed=300 + i) for i, (key, n) in enumerate(LENGTHS.items())}
    want = {key: plain.attention(x, named, m) for key, x in inputs.items()}
    for page_size in (16, 4):
        got, live = step_through(part, dtype, inputs, width, page_size=page_size)
        for key in inputs:
            close(got[key], want[key][:got[key].shape[0]], dtype, f32=5e-5, bf16=2e-2)
    if chunk is not None:
        assert live["a"].first_live[0] == live["a"].length // chunk * chunk // 4       # the pages of past chunks went back


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d,e", [(64, 64), (64, 16), (128, 128), (128, 64), (32, 48), (192, 192)])
def test_linear_bias_and_chunks_with_everything_else_on_the_scores(dtype, d, e):
    """The linear bias by distance alone, behind a cap, with a window that keeps first positions, in chunks, with a gate a head, sinks:
    parameters of the same kernels, whoever combines them.  Keys divided between workgroups too (700 positions), slopes from steep
    (a far key's score is hundreds below a near one's) to almost none, a far key that outweighs every near one all the same."""
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(d + e)
    heads, groups, length, page, window, kept, scale = 4, 2, 700, 16, 90, 5, 0.1
    q = torch.randn(length, heads, d, generator=g).to(dtype)
    k, v = torch.randn(length, groups, d, generator=g).to(dtype), torch.randn(length, groups, e, generator=g).to(dtype)
    k[3, 1] = (20.0 * (q[699, 2] + q[699, 3]).float()).to(dtype)      # the third head finds it, the fourth's slope is too steep
    gate = torch.randn(length, heads, generator=g).to(dtype)
    slopes = torch.tensor([0.8, 0.07, 0.004, 1.3])
    sinks = torch.tensor([0.0, -4.0, 1.0, -2.0])
    blocks = -(-length // page)
    order = torch.randperm(blocks, generator=g)
    k_pages, v_pages = torch.zeros(blocks, groups, page, d, dtype=dtype), torch.zeros(blocks, groups, e, page, dtype=dtype)
    for p in range(length):
        k_pages[order[p // page], :, p % page] = k[p]
        v_pages[order[p // page], :, :, p % page] = v[p]
    table = order.int().view(1, -1).cuda()
    k_pages, v_pages = k_pages.cuda(), v_pages.cuda()

    def wanted(rows, reach, keep, cap):
        out = torch.zeros(len(rows), heads, e, dtype=F64)
        for n, i in enumerate(rows):
            j = torch.arange(i + 1)
            if reach > 0:
                j = j[(i - j < reach) | (j < keep)]
            elif reach < 0:
                j = j[j // -reach == i // -reach]
            for h in range(heads):
                s = (k[j, h // 2].double() @ q[i, h].double()) * scale
                if cap:
                    s = cap * torch.tanh(s / cap)
                s = s - slopes[h].double() * (i - j)
                top = torch.maximum(s.max(), sinks[h].double())
                p = torch.exp(s - top)
                out[n, h] = (p / (p.sum() + torch.exp(sinks[h].double() - top))) @ v[j, h // 2].double() * torch.sigmoid(gate[i, h].double())
        return out.reshape(len(rows), heads * e)

    for reach, keep, cap in ((0, 0, 0.0), (0, 0, 2.0), (window, kept, 0.0), (window, 0, 2.0), (-130, 0, 0.0), (-700, 0, 2.0), (-699, 0, 0.0)):
        more = {"window": reach, "keep_first": keep, "sinks": sinks.cuda(), "softcap": cap, "distance": slopes.cuda()}
        for rows in ([699], [3], list(range(640, 700))):
            positions = torch.tensor(rows, dtype=torch.int32, device="cuda")
            of = torch.zeros(len(rows), dtype=torch.int32, device="cuda")
            mine, gates = q[rows].reshape(len(rows), heads * d).cuda(), gate[rows].cuda()
            out = torch.zeros(len(rows), heads * e, dtype=dtype, device="cuda")
            ops.attention(out, mine, k_pages, v_pages, table, of, positions, heads, scale, gates=gates, **more)
            want = wanted(rows, reach, keep, cap)
            close(out, want, dtype, f32=3e-5, bf16=1.5e-2)
            if not ops.attention_decode_supported(dtype, heads, groups, d, page, e):
                continue
            extra = 1 if keep else 0
            for splits in (1, 3):
                part_o = torch.empty(len(rows), heads * (splits + extra) * e, device="cuda")
                part_ml = torch.empty(len(rows), heads * (splits + extra) * 2, device="cuda")
                if len(rows) == 1:
                    for form in (0, 1, 2):
                        out.zero_()
                        ops.attention_decode(out, mine, k_pages, v_pages, table, of, positions, heads, scale, splits=splits, part_o=part_o,
                                             part_ml=part_ml, form=form, gates=gates, **more)
                        close(out, want, dtype, bf16=1.5e-2)
                    if d == e and not keep and not cap:    # the new key and value come in the query's row and are stored by the kernel
                        i = rows[0]
                        own = (int(order[i // page]), i % page)
                        k_kept, v_kept = k_pages[own[0], :, own[1]].clone(), v_pages[own[0], :, :, own[1]].clone()
                        k_pages[own[0], :, own[1]] = 9.0
                        v_pages[own[0], :, :, own[1]] = 9.0
                        row = torch.cat((mine, k[i].reshape(1, -1).cuda(), v[i].reshape(1, -1).cuda()), 1).contiguous()
                        out.zero_()
                        ops.attention_decode(out, row, k_pages, v_pages, table, of, positions, heads, scale, splits=splits, part_o=part_o, part_ml=part_ml,
                                             form=1, gates=gates, prepare=ops.DecodePrepare(None, None, 0.0, None, None, groups), **more)
                        close(out, want, dtype, bf16=1.5e-2)
                        assert torch.equal(k_pages[own[0], :, own[1]], k_kept) and torch.equal(v_pages[own[0], :, :, own[1]], v_kept)
                for size in (16, 32):
                    starts = torch.arange(0, len(rows), size, dtype=torch.int32, device="cuda")
                    counts = torch.clamp(len(rows) - starts, max=size).int()
                    out.zero_()
                    ops.attention_prefill(out, mine, k_pages, v_pages, table, of, positions, starts, counts, heads, scale, splits=splits,
                                          part_o=part_o, part_ml=part_ml, max_count=size, gates=gates, **more)
                    close(out, want, dtype, bf16=1.5e-2)


# ------------------------------------------------------------------------------------- latent attention
LATENT_SHAPES = [
    # heads, d, r, e, q_rank, c, scale, base, window, chunk
    (3, 16, 8, 24, 40, 40, 0.3, 1e4, 13, None),
    (1, 8, 2, 8, 8, 8, 0.35, 50.0, 1, None),            # a window of one, one pair, equal ranks
    (4, 64, 32, 64, 96, 96, 0.12, 1e4, 24, None),       # the matrix cores' shape
    (16, 32, 16, 32, 24, 64, 0.15, 500.0, 16, None),    # ranks of queries below the rank of keys, a window of just a page
    (2, 128, 64, 128, 192, 256, 0.09, 1e6, 40, None),
    (5, 24, 4, 10, 33, 20, 0.2, 9.0, None, None),       # odd sizes, the whole context
    (6, 32, 16, 64, 80, 128, 0.15, 1e4, None, 21),      # chunks instead of a window
    (70, 16, 8, 8, 56, 40, 0.2, 300.0, 30, None),       # more heads than a wave has lanes
]


def latent_part(width, shape, dtype, seed, gate="value", edit=None):
    from llm_runtime_study_amd.parts import PartSpec, create

    heads, d, r, e, q_rank, c, scale, base, window, chunk = shape
    part = create("mixer", PartSpec("latent_attention", {
        "hidden_size": width, "num_heads": heads, "head_dim": d, "rot_dim": r, "value_dim": e, "q_rank": q_rank, "kv_rank": c, "window": window, "chunk": chunk,
        "position": PartSpec("rope_interleaved", {"rotary_dim": r, "theta": base}), "norm_eps": 1e-3, "scale": scale, "gate": gate}))
    w = part_weights(part, seed)
    if edit is not None:
        edit(w)
    m = {"heads": heads, "dim": d, "rot_dim": r, "vdim": e, "q_rank": q_rank, "kv_rank": c, "scale": scale, "rot": {"base": base, "dims": r}}
    if window is not None:
        m["mask"] = {"size": window}
    return part, bound(part, w, dtype), m


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("shape", LATENT_SHAPES)
def test_latent_attention_part(dtype, shape, monkeypatch):
    width = 64
    part, named, m = latent_part(width, shape, dtype, 70)
    assert set(named) == {"dq", "dq.norm", "uq", "dkv", "dkv.norm", "uk", "uv", "g", "o"} and named["g"].shape == (shape[0] * shape[3], width)
    if shape[9] is not None:           # the plain mixer in chunks: the same function with the other mask
        monkeypatch.setattr(plain, "in_window", lambda i, j, size: plain.in_chunk(i, j, shape[9]))
    inputs = {key: bf16_values(n, width, seed=400 + i) for i, (key, n) in enumerate(LENGTHS.items())}
    want = {key: plain.latent_attention(x, named, m, 1e-3) for key, x in inputs.items()}
    for page_size in (16, 8):
        got, live = step_through(part, dtype, inputs, width, page_size=page_size)
        for key in inputs:
            close(got[key], want[key][:got[key].shape[0]], dtype, f32=5e-5, bf16=3e-2)
    if shape[8] is not None:
        assert live["a"].first_live[0] == (live["a"].length - shape[8] + 1) // 8


@pytest.mark.parametrize("dtype", DTYPES)
def test_latent_queries_from_a_row_of_their_own_with_a_gate_a_head_or_none(dtype):
    """The query's latent row beside the other kinds of gate: one number a head multiplies all of a head's values."""
    width, shape = 48, (4, 16, 8, 16, 24, 32, 0.3, 100.0, 11, None)
    x = bf16_values(30, width, seed=9)
    for gate in (True, False):
        part, named, m = latent_part(width, shape, dtype, 90, gate=gate)
        full = dict(named)
        full["g"] = named["g"].repeat_interleave(16, 0) if gate else torch.zeros(64, width, dtype=F64)
        want = plain.latent_attention(x, full, m, 1e-3) * (1.0 if gate else 2.0)
        got, _ = step_through(part, dtype, {"a": x}, width, schedule=[[("a", 13)], [("a", 1)], [("a", 16)]], release_before=None)
        close(got["a"], want, dtype, f32=5e-5, bf16=3e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens,heads,n,k,rot", [(1, 3, 40, 16, 8), (9, 2, 64, 24, 2), (70, 5, 96, 32, 16), (130, 1, 7, 5, 4), (33, 4, 200, 128, 64)])
def test_per_head_product_that_rotates_and_gates(dtype, tokens, heads, n, k, rot):
    from llm_runtime_study_amd.kernels import ops

    a = bf16_values(tokens, heads, k + rot, seed=1)
    w = bf16_values(heads, n, k, scale=1 / math.sqrt(k), seed=2)
    gate = bf16_values(tokens, heads * n + 5, seed=3)
    angle = torch.randn(tokens, rot // 2, generator=torch.Generator().manual_seed(4), dtype=F64)
    want = torch.empty(tokens, heads, n + rot, dtype=F64)
    want[..., :n] = torch.einsum("thk,hnk->thn", a[..., :k], w) * torch.sigmoid(gate[:, :heads * n]).view(tokens, heads, n)
    u, v = a[..., k::2], a[..., k + 1::2]
    c, s = angle.cos()[:, None], angle.sin()[:, None]
    want[..., n::2], want[..., n + 1::2] = u * c - v * s, v * c + u * s
    for transposed in (False, True):
        out = torch.full((tokens, heads, n + rot), 7.0, dtype=dtype, device="cuda")
        mine = (w.transpose(1, 2) if transposed else w).contiguous().to(dtype).cuda()
        ops.head_gemm(out, a.to(dtype).cuda(), mine, transposed=transposed, rotate=(angle.cos().float().cuda(), angle.sin().float().cuda()),
                      gate=gate.to(dtype).cuda()[:, :heads * n])
        close(out, want, dtype, f32=2e-5, bf16=8e-3)


# ------------------------------------------------------------------------------------- feed-forwards
@pytest.mark.parametrize("tokens", [1, 20, 32, 33, 300])
@pytest.mark.parametrize("count,identity,top", [(6, 3, 2), (1, 1, 1), (66, 14, 5), (4, 0, 4), (3, 9, 12)])
def test_choice_and_sort_with_identity_experts(count, identity, top, tokens):
    """Softmax scores of every output of the router: choices, weights, and the sorted list, in which identity choices have no row."""
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(count + tokens)
    choices = count + identity
    padded = torch.zeros(tokens, choices + 5)
    padded[:, :choices] = 2.0 * torch.randn(tokens, choices, generator=g)
    padded[0, 0] = 90.0                              # a score of one, and others that underflow
    logits, bias = padded.cuda()[:, :choices], (0.05 * torch.randn(choices, generator=g)).cuda()
    rule = ops.RouteRule("softmax_scores")
    tile, tiles = ops.moe_tile_rows(tokens * top, count), ops.moe_max_tiles(tokens * top, count)

    def lists():
        return (torch.empty(tokens, top, dtype=torch.int32, device="cuda"), torch.empty(tokens, top, device="cuda"),
                torch.empty(tiles * tile, dtype=torch.int32, device="cuda"), torch.empty(tokens * top, dtype=torch.int32, device="cuda"),
                torch.empty(tiles, dtype=torch.int32, device="cuda"))

    margins = []
    chosen, shares = plain.choose(padded[:, :choices].double(), bias.double().cpu(), top, margins)
    runs = []
    ids, weights, order, place, owner = lists()
    ops.moe_route(logits, bias, ids, weights, rule)
    ops.moe_align(ids, count, order, place, owner, identity=identity)
    runs.append((ids, weights, order, place, owner))
    if tokens <= ops.ROUTE_ALIGN_TOKENS:
        ids, weights, order, place, owner = lists()
        ops.moe_route_align(logits, bias, ids, weights, order, place, owner, rule, identity=identity)
        runs.append((ids, weights, order, place, owner))
    for ids, weights, order, place, owner in runs:
        ids, weights, order, place, owner = (t.cpu() for t in (ids, weights, order, place, owner))
        for t in range(tokens):
            if margins and margins[t] < 1e-5:
                continue
            assert ids[t].tolist() == chosen[t]
            torch.testing.assert_close(weights[t].double(), torch.tensor(shares[t], dtype=F64), rtol=2e-6, atol=1e-9)
        flat = ids.flatten().tolist()
        rows = [r for r in order.tolist() if r >= 0]
        assert sorted(rows) == [pair for pair, e in enumerate(flat) if e < count]
        for pair, e in enumerate(flat):
            if e >= count:
                assert place[pair] == -1
            else:
                assert order[place[pair]] == pair and owner[int(place[pair]) // tile] == e
    # without a correction the choice follows the logits
    ids, weights, *_ = lists()
    ops.moe_route(logits, None, ids, weights, rule)
    assert torch.equal(ids.long().cpu().sort(1).values, torch.topk(padded[:, :choices], top, 1).indices.sort(1).values)


ROUTED_SHAPES = [
    # width, ff, experts, identity, top, limit, shared (ff, limit), tokens
    (64, 48, 6, 3, 2, 1.0, (32, 0.7), 50),
    (128, 64, 12, 20, 3, 0.5, None, 90),          # mostly identity choices
    (72, 15, 5, 2, 3, 2.0, (18, 1.0), 33),        # an odd expert size
    (128, 128, 4, 0, 2, 1.5, (64, 1.5), 200),     # no identity experts, large tiles
    (48, 24, 1, 1, 2, 1.0, None, 7),              # every choice taken
    (100, 26, 70, 9, 4, 1.1, (7, 0.4), 40),       # more outputs than a wave has lanes, a width that is no multiple of eight
    (2050, 16, 3, 1, 2, 1.0, None, 9),            # a width beyond 2,048
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,count,identity,top,limit,shared,tokens", ROUTED_SHAPES)
def test_routed_experts_part(dtype, width, ff, count, identity, top, limit, shared, tokens):
    from llm_runtime_study_amd.parts import BoundNorm, PartSpec, create

    shared_spec = None if shared is None else PartSpec("swiglu", {"hidden_size": width, "intermediate_size": shared[0], "activation": "clamped",
                                                                  "alpha": 1.702, "limit": shared[1]})
    part = create("feed_forward", PartSpec("routed_experts", {
        "hidden_size": width, "intermediate_size": ff, "num_experts": count, "identity": identity, "top": top, "rule": "softmax_scores", "router_bias": True,
        "bias_name": "correction", "activation": "clamped_gated", "activation_limit": limit, "shared": shared_spec}))
    w = part_weights(part, 20)
    w["correction"] = (0.1 * w["correction"]).to(torch.bfloat16).double()
    for name in w:                                   # projections large enough that the clamps bite for a good share of the features
        if name.endswith(("gate.weight", "up.weight", "gate_proj.weight", "up_proj.weight")):
            w[name] = (w[name] * 1.5).to(torch.bfloat16).double()
    named = bound(part, w, dtype)
    mlp = configs.experts(ff, limit, count, identity, top, shared)
    x = bf16_values(tokens, width, seed=31)
    margins, picks = [], []
    want = plain.routed_ff(x, named, mlp, margins, picks)
    assert not identity or any(e >= count for row in picks[0] for e in row)
    sure = torch.tensor([m > (1e-5 if dtype == torch.float32 else 1e-3) for m in margins]) if margins else torch.ones(tokens, dtype=torch.bool)
    assert sure.float().mean() > 0.7
    harness = PartHarness([], dtype, max_step_tokens=512)
    ctx = harness.context([(harness.cache.admit("a"), [0] * tokens)])
    mine = x.to(dtype).cuda()
    for accumulate in (True, False):
        residual = torch.full((tokens, width), 0.25, dtype=torch.float32, device="cuda")
        part.forward(ctx, mine, residual, accumulate=accumulate)
        close(residual.cpu().double()[sure] - (0.25 if accumulate else 0.0), want[sure], dtype, f32=1e-4, bf16=2e-2)
    # the norm of the output, and the norm that comes next, in the kernel that adds the rows up
    weight, after = 1.0 + 0.1 * bf16_values(width, seed=5), 1.0 + 0.1 * bf16_values(width, seed=6)
    stream = bf16_values(tokens, width, seed=7)
    new = stream + plain.rms(want, weight, 1e-5)
    for following in (True, False):
        residual = stream.float().cuda()
        buffer = torch.zeros(tokens, width, dtype=dtype, device="cuda")
        part.forward(ctx, mine, residual, output_norm=BoundNorm(weight.float().cuda(), 1e-5), next_norm=(after.float().cuda(), 1e-4, buffer) if following else None)
        close(residual.cpu()[sure], new[sure], dtype, f32=2e-4, bf16=2e-2)
        if following:
            close(buffer.cpu()[sure], plain.rms(new, after, 1e-4)[sure], dtype, f32=2e-4, bf16=2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width,ff,tokens", [(64, 96, 5), (72, 50, 33), (40, 27, 3), (256, 512, 150)])
def test_square_of_relu_part(dtype, width, ff, tokens):
    from llm_runtime_study_amd.parts import PartSpec, create

    part = create("feed_forward", PartSpec("dense_mlp", {"hidden_size": width, "intermediate_size": ff, "activation": "relu_squared"}))
    named = bound(part, part_weights(part, 8), dtype)
    x = bf16_values(tokens, width, seed=2)
    harness = PartHarness([], dtype)
    ctx = harness.context([(harness.cache.admit("a"), [0] * tokens)])
    out = torch.full((tokens, width), 3.0, dtype=torch.float32, device="cuda")
    part.forward(ctx, x.to(dtype).cuda(), out, accumulate=False)
    close(out, plain.dense_ff(x, named["up"], named["down"]), dtype, f32=3e-5, bf16=1e-2)


def test_every_activation_in_pieces_and_one_by_one():
    from llm_runtime_study_amd.kernels import ops

    formulas = {"gelu": lambda z: torch.nn.functional.gelu(z), "gelu_tanh": lambda z: torch.nn.functional.gelu(z, approximate="tanh"),
                "silu": lambda z: z * torch.sigmoid(z), "relu": torch.relu, "relu_squared": lambda z: torch.relu(z) ** 2}
    assert set(formulas) == set(ops.ACTIVATIONS)
    for dtype in DTYPES:
        for count in (4096, 4099, 7):
            x = (2.0 * torch.randn(1, count, generator=torch.Generator().manual_seed(count))).to(dtype)
            for kind, formula in formulas.items():
                out = torch.zeros_like(x, device="cuda")
                ops.activation(out, x.cuda(), kind)
                close(out, formula(x.double()), dtype, f32=2e-6, bf16=4e-3)


# ------------------------------------------------------------------------------------- whole models
RAW = {name: configs.ALL[name] for name in ("odd", "cores", "ones", "awkward")}
MODEL_LENGTHS = {"odd": [70, 33, 9, 1, 52, 17, 66], "cores": [150, 64, 2, 97, 33], "ones": [40, 1, 65, 16, 5], "awkward": [90, 31, 3, 48, 17]}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for number, (name, raw) in enumerate(RAW.items()):
        folder = configs.write_folder(raw, 360 + number, tmp_path_factory.mktemp(f"tamilix_{name}"))
        tensors, _ = plain.load_model_dir(folder)
        rng = np.random.default_rng(321 + number)
        requests = {f"{name}{i}": rng.integers(0, raw["vocab"], n).tolist() for i, n in enumerate(MODEL_LENGTHS[name])}
        out[name] = (folder, raw, requests, {key: plain.forward(tensors, raw, tokens) for key, tokens in requests.items()})
    return out


def check(got, want, dtype):
    """float32: rows within 2e-4 of the plain row as a whole (relative L2; a row whose expert choice is a close call may differ, so one
    row in fifty may be off).  bfloat16: these models are a few dozen values wide, normalise every sublayer's output and choose
    experts, which is a discrete choice that a rounding can turn (and the token's row, and those that attend to it, with it): 80 rows
    in 100 within 4 % as a whole, and none off by more than its own length."""
    errors = np.array([float((row.double() - want[key][position]).norm() / want[key][position].norm())
                       for key, rows in got.items() for position, row in rows.items()])
    if dtype == "float32":
        assert np.mean(errors < 2e-4) >= 0.98, f"{np.mean(errors < 2e-4):.3f} of the rows are close, the worst is off by {errors.max():.3g}"
        return len(errors)
    assert np.mean(errors < 4e-2) >= 0.8 and errors.max() < 1.0, f"{np.mean(errors < 4e-2):.2f} of the rows are close, the worst is off by {errors.max():.3g}"
    return len(errors)


def test_the_stream_after_every_layer_run(models):
    """One step function call on a whole prompt in float32, the stream read after every run of a layer (a layer that shares weights
    counts each time) against the plain implementation's."""
    from llm_runtime_study_amd.engine import trace
    from llm_runtime_study_amd.engine.step import StepEntry

    for name in RAW:
        folder, raw, requests, _ = models[name]
        tokens = requests[f"{name}4"]
        tensors, _ = plain.load_model_dir(folder)
        streams = []
        plain.forward(tensors, raw, tokens, streams)
        runner = trace.make_runner(folder, "float32", 128, 16)
        seen = []
        for layer in runner.model.layers:
            inner = layer.forward

            def watched(ctx, h, *args, _inner=inner, **kwargs):
                result = _inner(ctx, h, *args, **kwargs)
                seen.append(h.detach().clone())
                return result

            layer.forward = watched
        runner.step([StepEntry(runner.cache.admit("r"), tokens, [len(tokens) - 1])])
        torch.cuda.synchronize()
        assert len(seen) == len(streams) == len(raw["layers"])
        for mine, theirs in zip(seen, streams):
            torch.testing.assert_close(mine[:len(tokens)].cpu().double(), theirs, rtol=2e-4, atol=2e-4)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", list(RAW))
def test_whole_then_last_tokens_one_by_one_then_portions(models, name, dtype, tmp_path):
    folder, raw, requests, want = models[name]
    longest = max(round64(len(t)) for t in requests.values())
    steps = traces.whole(requests)
    got = traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "whole"), raw["vocab"])
    assert check(got, want, dtype) == sum(len(t) for t in requests.values())
    steps = traces.prefill_then_decode(requests, tail=50)        # longer than most windows: they pass over decoded tokens
    check(traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "tail"), raw["vocab"]), want, dtype)
    steps = traces.portions(requests)
    check(traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "portions", page_size=32), raw["vocab"]), want, dtype)
    few = {key: tokens for key, tokens in requests.items() if len(tokens) < 70}
    steps = traces.portions(few, sizes=(2, 2, 3, 2))
    check(traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "twos"), raw["vocab"]), want, dtype)


def test_cuts_batch_mates_and_pages_change_no_bit_in_float32(models, tmp_path):
    """float32 sums depend on the position alone: the same rows under every cutting, to the bit."""
    folder, raw, requests, _ = models["odd"]
    longest = max(round64(len(t)) for t in requests.values())
    steps = traces.whole(requests)
    whole = traces.collect(steps, run_replay(folder, "float32", steps, longest, tmp_path / "whole"), raw["vocab"])
    steps, peak = traces.mixed(requests, seed=8, max_live=4, max_tokens=2 * longest)
    mixed = traces.collect(steps, run_replay(folder, "float32", steps, peak, tmp_path / "mixed", page_size=32), raw["vocab"])
    steps = traces.portions(requests, sizes=(3, 2, 19, 2))
    cut = traces.collect(steps, run_replay(folder, "float32", steps, longest, tmp_path / "cut"), raw["vocab"])
    compared = 0
    for key, rows in mixed.items():
        for position, row in rows.items():
            assert torch.equal(row, whole[key][position]) and torch.equal(cut[key][position], row), (key, position)
            compared += 1
    assert compared > 40


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,seed", [("odd", 0), ("odd", 1), ("cores", 2), ("ones", 3), ("awkward", 6)])
def test_mixed_steps_with_pages_and_slots_used_again(models, name, seed, dtype, tmp_path):
    folder, raw, requests, want = models[name]
    budget = 2 * max(round64(len(t)) for t in requests.values())
    steps, peak = traces.mixed(requests, seed=seed, max_live=4, max_tokens=budget)
    assert max(len(s["entries"]) for s in steps) >= 3
    got = traces.collect(steps, run_replay(folder, dtype, steps, peak, tmp_path), raw["vocab"])
    assert check(got, want, dtype) > 30
    assert peak < sum(round64(len(t)) for t in requests.values())


@pytest.mark.parametrize("name", ["odd", "cores"])
def test_the_engines_path_of_graphs_and_recorded_steps(models, name, tmp_path):
    """On a stream of the runner's own with graphs on: single-token steps are graph replays, shapes that come back are launched from
    their recorded plan."""
    folder, raw, requests, want = models[name]
    longest = max(round64(len(t)) for t in requests.values())
    seen = {}
    steps = traces.prefill_then_decode(requests, tail=40)
    out = run_replay(folder, "float32", steps, longest, tmp_path / "tail", as_the_engine=True, counters=seen)
    check(traces.collect(steps, out, raw["vocab"]), want, "float32")
    assert seen["graph_replays"] >= 20 * (len(requests) - 2)
    steps, peak = traces.mixed(requests, seed=5, max_live=4, max_tokens=2 * longest)
    out = run_replay(folder, "bfloat16", steps, peak, tmp_path / "mixed", as_the_engine=True, counters=seen)
    check(traces.collect(steps, out, raw["vocab"]), want, "bfloat16")
    steps = traces.portions(requests, sizes=(16, 16, 16, 2))
    out = run_replay(folder, "float32", steps, longest, tmp_path / "portions", as_the_engine=True, counters=seen)
    check(traces.collect(steps, out, raw["vocab"]), want, "float32")
    assert seen["plan_replays"] >= 10


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_wider_model_through_the_products_for_many_rows(tmp_path, dtype):
    """Width 512 and prompts of 330 and 140 tokens: the projections of a prompt are products of hundreds of rows (the vendor library's
    in bfloat16), the experts get enough rows for the large tiles, windows and chunks lie inside the longer prompt."""
    raw = configs.WIDE
    folder = configs.write_folder(raw, 21, tmp_path / "wide")
    tensors, _ = plain.load_model_dir(folder, torch.float32)
    rng = np.random.default_rng(4)
    requests = {"long": rng.integers(0, raw["vocab"], 330).tolist(), "short": rng.integers(0, raw["vocab"], 140).tolist()}
    want = {key: plain.forward(tensors, raw, tokens).double() for key, tokens in requests.items()}
    steps = [{"step": 0, "entries": [{"id": key, "tokens": tokens[:-6], "want": list(range(0, len(tokens) - 6, 7))} for key, tokens in requests.items()], "end": []}]
    for i in range(6, 0, -1):
        steps.append({"step": len(steps), "entries": [{"id": key, "tokens": [tokens[-i]], "want": [0]} for key, tokens in requests.items()],
                      "end": list(requests) if i == 1 else []})
    got = traces.collect(steps, run_replay(folder, dtype, steps, 512, tmp_path / "o"), raw["vocab"])
    assert check(got, want, dtype) > 70


def test_bfloat16_path_follows_float32_at_real_layer_sizes():
    """Four layers at the sizes of a real model's (width 1,024, 16 heads of 128 on 8 key groups in chunks of 600, latent attention with
    512 latent values behind a window of 512, 2 of 8 experts of 1,024 and 2 identity experts, a shared one, dense layers of 3,072): the
    bfloat16 path with everything it uses at that size (graphs, the vendor's products for many rows, the grouped products' large tiles,
    key splits, the prefill kernel for heads of 128, keys and values stored by the decode kernel) against the float32 path of the same
    weights, over prompts in two portions beside decoding requests and decode steps.  Experts are a discrete choice, so a share of the
    rows may differ."""
    from llm_runtime_study_amd.benchmarks.shapes import SHAPES, tamilix_like
    from llm_runtime_study_amd.cache import CacheManager
    from llm_runtime_study_amd.config import config_from_dict, spec_for
    from llm_runtime_study_amd.engine.step import ModelRunner, StepEntry
    from llm_runtime_study_amd.models import DecoderModel
    from llm_runtime_study_amd.weights import random_init

    raw = tamilix_like(dict(SHAPES["0.6b"], vocab_size=8000), 4, experts=8, identity=2, top=2, chunk=600, window=512)
    cfg = config_from_dict(raw)
    device = torch.device("cuda", 0)
    weights = random_init.device_weights(DecoderModel(spec_for(cfg)), 0, torch.bfloat16, device, "scaled")
    rng = np.random.default_rng(1)
    prompts = [rng.integers(0, cfg.vocab_size, n).tolist() for n in (700, 33, 1500, 257, 64, 5, 1023, 90)]
    tails = [rng.integers(0, cfg.vocab_size, 14).tolist() for _ in prompts]
    logits_of = {}
    for dtype in (torch.float32, torch.bfloat16):
        model = DecoderModel(spec_for(cfg))
        model.bind(weights, dtype)
        cache = CacheManager(model.cache_needs(), page_size=16, num_pages=400, max_requests=8, max_seq_len=2048, dtype=dtype, device=device)
        runner = ModelRunner(model, cache, max_step_tokens=2048, dtype=dtype, device=device, use_graph=dtype == torch.bfloat16)
        rows = []
        with torch.cuda.stream(torch.cuda.Stream(device)):
            caches = [cache.admit(i) for i in range(len(prompts))]
            fed = {}
            for i, prompt in enumerate(prompts):
                # the first half of the prompt beside one token of every earlier request, then the rest alone
                half = len(prompt) // 2
                decoding = [StepEntry(caches[j], [tails[j][fed[j]]], [0]) for j in sorted(fed)]
                for j in fed:
                    fed[j] += 1
                mixed = runner.step(decoding + [StepEntry(caches[i], prompt[:half], [half - 1])])
                rows.append(mixed.float().cpu())
                rows.append(runner.step([StepEntry(caches[i], prompt[half:], [0, len(prompt) - half - 1])]).float().cpu())
                fed[i] = 0
            for _ in range(6):
                rows.append(runner.step([StepEntry(caches[j], [tails[j][fed[j]]], [0]) for j in sorted(fed)]).float().cpu())
                for j in fed:
                    fed[j] += 1
            if dtype == torch.bfloat16:
                assert runner.graph_replays >= 3
                runner.drop_graphs()
        logits_of[dtype] = torch.cat(rows)
        cache.check_invariants()
        del runner, cache, model
    exact, fast = logits_of[torch.float32], logits_of[torch.bfloat16]
    assert exact.shape == fast.shape and exact.shape[0] > 80
    error = (exact - fast).norm(dim=1) / exact.norm(dim=1)
    assert (error < 3e-2).float().mean() >= 0.9 and error.median() < 1.5e-2, f"median {error.median():.3g}, {(error < 3e-2).float().mean():.2f} of the rows close"


# ------------------------------------------------------------------------------------- planted inputs
CHUNK, WINDOW = 37, 21


def planted_model(tmp_path, kind):
    """A model of one layer whose attention's query of token B is the key of token A when A's embedding is B's with its two halves
    swapped: the match then scores so high that it towers over every other score, and a B adds A's value to the stream exactly when A
    is visible from B.  Token 0 is A, token 1 B."""
    width = 64
    if kind == "attention":
        layer = configs.chunked(2, 2, 32, 32, 0.5, CHUNK)
    else:
        layer = configs.latent(2, 32, 4, 24, 32, 40, 0.7, 1e4, WINDOW)
    raw = configs.model(50, width, 1e-6, 1.0, [layer])

    def swapped(t):
        return torch.cat((t[:, width // 2:], t[:, :width // 2]), 1)

    def edit(tensors):
        embed = tensors["embed"]
        embed[0] = torch.cat((embed[1, width // 2:], embed[1, :width // 2]))
        tensors["l0.norm1"].fill_(1.0)
        if kind == "attention":
            tensors["l0.mix.q"] = swapped(tensors["l0.mix.k"])
            tensors["l0.mix.sink"].zero_()
            return
        # a head's plain query and key are the first 32 latent values of the query's and the key's row; the rotated parts are zero
        tensors["l0.mix.dq"] = swapped(tensors["l0.mix.dkv"][:32])
        tensors["l0.mix.dq.norm"].fill_(1.0)
        tensors["l0.mix.dkv.norm"].fill_(1.0)
        uq, uk = torch.zeros_like(tensors["l0.mix.uq"]).view(2, 36, 32), torch.zeros_like(tensors["l0.mix.uk"]).view(2, 32, 40)
        uq[:, :32], uk[:, :, :32] = torch.eye(32), torch.eye(32)
        tensors["l0.mix.uq"], tensors["l0.mix.uk"] = uq.reshape(72, 32), uk.reshape(64, 40)

    return raw, configs.write_folder(raw, 77, tmp_path / "planted", edit=edit)


def planted_requests(raw, places, length, seed=2):
    """{label: tokens} with an A at `first` and a B at `asked` for every (label, first, asked) in `places`."""
    rng = np.random.default_rng(seed)
    requests, asked = {}, {}
    for label, first, second in places:
        tokens = rng.integers(2, raw["vocab"], length).tolist()
        tokens[first], tokens[second] = 0, 1
        requests[label], asked[label] = tokens, second
    return requests, asked


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["attention", "latent_attention"])
def test_keys_on_either_side_of_an_edge(tmp_path, kind, dtype):
    raw, folder = planted_model(tmp_path, kind)
    tensors, _ = plain.load_model_dir(folder)
    if kind == "attention":
        # the first token of a chunk from its last one and from the next chunk's first; the last token of a chunk (and just before
        # it) from the next chunk's first; the same inside one chunk; at a page's border; in the sequence's first chunk
        pairs = {"chunk": ((CHUNK, 2 * CHUNK - 1), (CHUNK, 2 * CHUNK)), "border": ((2 * CHUNK - 2, 2 * CHUNK - 1), (2 * CHUNK - 1, 2 * CHUNK)),
                 "page": ((80, 95), (64, 80)), "first": ((0, CHUNK - 1), (0, CHUNK))}
    else:
        pairs = {"edge": ((40, 40 + WINDOW - 1), (40, 40 + WINDOW)), "early": ((0, WINDOW - 1), (0, WINDOW)), "page": ((31, 31 + WINDOW - 1), (31, 31 + WINDOW)),
                 "later": ((80, 80 + WINDOW - 1), (80, 80 + WINDOW))}
    places = [(f"{label}_{side}", *place) for label, both in pairs.items() for side, place in zip(("in", "out"), both)]
    requests, asked = planted_requests(raw, places, 120)
    want = {key: plain.forward(tensors, raw, tokens) for key, tokens in requests.items()}
    for key, position in asked.items():                            # the planted key matters exactly where it is seen
        other = list(requests[key])
        other[places[[p[0] for p in places].index(key)][1]] = 9
        moved = (plain.forward(tensors, raw, other)[position] - want[key][position]).norm() / want[key][position].norm()
        assert moved > 0.2 if key.endswith("_in") else moved < 1e-9, (key, float(moved))

    def rows_match(got):
        for key, position in asked.items():                       # the rows that matter, one by one
            row, ref = got[key][position].double(), want[key][position]
            assert (row - ref).norm() < (1e-4 if dtype == "float32" else 5e-2) * ref.norm(), (key, position)

    for steps in (traces.whole(requests), traces.prefill_then_decode(requests, tail=100), traces.portions(requests, sizes=(5, 2, 30, 3, 17))):
        got = traces.collect(steps, run_replay(folder, dtype, steps, 128, tmp_path / f"o{len(steps)}"), raw["vocab"])
        check(got, want, dtype)
        rows_match(got)
    steps, peak = traces.mixed(requests, seed=3, max_live=4, max_tokens=384)
    for step in steps:                                           # the rows that matter are asked for in every schedule
        for entry in step["entries"]:
            place = asked[entry["id"]] - entry["_at"]
            if 0 <= place < len(entry["tokens"]) and place not in entry["want"]:
                entry["want"] = sorted(entry["want"] + [place])
    got = traces.collect(steps, run_replay(folder, dtype, steps, peak, tmp_path / "mixed"), raw["vocab"])
    check(got, want, dtype)
    rows_match(got)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("planted,last", [(0, 499), (512, 1023), (500, 511), (15, 16), (255, 256), (300, 301), (127, 500), (640, 1000)])
def test_a_key_far_back_in_a_chunk_among_hundreds(dtype, planted, last):
    """One head with a small slope, chunks of 512: the one matching key is found from a prompt's portion and from a decoded token, and a
    chunk's hundreds of other keys take next to nothing."""
    from llm_runtime_study_amd.parts import PartSpec, create

    width, d = 64, 64
    part = create("mixer", PartSpec("gqa_attention", {"hidden_size": width, "num_heads": 2, "num_kv_heads": 1, "head_dim": d, "value_dim": d, "scale": 0.6,
                                                     "chunk": 512, "sink": True, "distance_bias": "linear"}))
    w = part_weights(part, 5)
    half = width // 2
    k = w["k_proj.weight"]
    w["q_proj.weight"] = torch.cat((k[:, half:], k[:, :half]), 1).repeat(2, 1)
    w["sink"] = torch.tensor([1.0, -2.0], dtype=F64)
    named = bound(part, w, dtype)
    m = {"heads": 2, "kv_heads": 1, "dim": d, "vdim": d, "scale": 0.6, "mask": {"size": 512}}
    x = bf16_values(last + 1, width, seed=40)
    x[planted] = torch.cat((x[last, half:], x[last, :half]))
    first = last // 512 * 512 if last // 512 * 512 <= planted else last
    # the plain rows of the last chunk alone (what lies before it is not seen)
    shares = []
    tail = plain.attention(x[first:], named, m, shares)[-1]
    for h, i, seen, share in shares:
        if i == last - first and h == 1:
            assert float(share[seen.index(planted - first)]) > 0.9
    for cut in (last - 1, max(1, last - 5)):
        harness = PartHarness([part.cache_need()], dtype, max_step_tokens=1024)
        request = harness.cache.admit("a")
        for begin, end in [(0, cut)] + ([(cut, last + 1)] if cut == last - 1 else [(i, i + 1) for i in range(cut, last + 1)]):
            ctx = harness.context([(request, [0] * (end - begin))])
            out = torch.zeros(end - begin, width, dtype=torch.float32, device="cuda")
            part.forward(ctx, x[begin:end].to(dtype).cuda(), out, ctx.layer_cache(0), accumulate=False)
            harness.cache.trim(request)
        close(out[-1], tail, dtype, f32=5e-5, bf16=3e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_beside_a_second_request(models, dtype, tmp_path):
    """240 tokens one by one behind a prompt of ten, a second request's tokens beside them: windows and chunks pass over decoded tokens,
    pages are given back while the request runs."""
    folder, raw, _, _ = models["cores"]
    tensors, _ = plain.load_model_dir(folder)
    rng = np.random.default_rng(17)
    requests = {"x": rng.integers(0, raw["vocab"], 250).tolist(), "y": rng.integers(0, raw["vocab"], 120).tolist()}
    want = {key: plain.forward(tensors, raw, tokens) for key, tokens in requests.items()}
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": requests["x"][:10], "want": [9]}, {"id": "y", "tokens": requests["y"][:3], "want": [2]}], "end": []}]
    for i in range(10, 250):
        entries = [{"id": "x", "tokens": [requests["x"][i]], "want": [0]}]
        j = i - 7
        if j < 120:
            entries.append({"id": "y", "tokens": [requests["y"][j]], "want": [0]})
        steps.append({"step": len(steps), "entries": entries, "end": (["y"] if j == 119 else []) + (["x"] if i == 249 else [])})
    got = traces.collect(steps, run_replay(folder, dtype, steps, 384, tmp_path / "o"), raw["vocab"])
    assert 249 in got["x"] and 119 in got["y"]
    check(got, want, dtype)


# ------------------------------------------------------------------------------------- generation
def test_greedy_generation_through_engine_and_scheduler(models):
    """Three prompts on two slots (the third waits and takes a freed slot and its pages), prompts fed in portions of at most 16 tokens
    beside decoding requests: the tokens are the plain implementation's own greedy continuation."""
    from llm_runtime_study_amd import Engine

    folder, raw, requests, _ = models["odd"]
    tensors, _ = plain.load_model_dir(folder)
    prompts = [requests["odd2"], requests["odd6"][:30], requests["odd1"]]
    want = []
    for prompt in prompts:
        ids = list(prompt)
        for _ in range(6):
            ids.append(int(plain.forward(tensors, raw, ids)[-1].argmax()))
        want.append(ids[len(prompt):])
    engine = Engine.from_model_dir(folder, dtype="float32", max_seq_len=128, max_batch_size=2, max_num_batched_tokens=16)
    assert engine.generate_tokens(prompts, max_new_tokens=6) == want
    assert engine.cache_manager.active_requests == 0 and engine.cache_manager.used_pages(0) == 0


def test_command_line_and_trace_run_as_programs(models, tmp_path):
    """The two programs, each a process of its own, find the architecture by the folder's config.json: greedy tokens from the command
    line (token ids in, token ids out, random weights from a seed as well), and a mixed replay through bin/trace_run."""
    import os
    import subprocess
    import sys
    from pathlib import Path

    root = Path(__file__).resolve().parents[1]
    env = dict(os.environ, PYTHONPATH=str(root))
    folder, raw, requests, want = models["awkward"]
    tensors, _ = plain.load_model_dir(folder)
    prompt = requests["awkward2"]
    ids = list(prompt)
    for _ in range(5):
        ids.append(int(plain.forward(tensors, raw, ids)[-1].argmax()))
    proc = subprocess.run([sys.executable, "-m", "llm_runtime_study_amd", "--model", str(folder), "--prompt-ids", ",".join(map(str, prompt)),
                           "--max-new-tokens", "5", "--dtype", "float32", "--max-seq-len", "64", "--no-metrics"],
                          capture_output=True, text=True, timeout=300, env=env, cwd=tmp_path)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [int(t) for t in proc.stdout.split()] == ids[len(prompt):]
    only_config = tmp_path / "only_config"
    only_config.mkdir()
    (only_config / "config.json").write_text((folder / "config.json").read_text())
    proc = subprocess.run([sys.executable, "-m", "llm_runtime_study_amd", "--model", str(only_config), "--random-weights", "3", "--prompt-ids", "1,2,3",
                           "--max-new-tokens", "4", "--max-seq-len", "64", "--no-metrics"], capture_output=True, text=True, timeout=300, env=env, cwd=tmp_path)
    assert proc.returncode == 0 and len(proc.stdout.split()) == 4, proc.stderr[-2000:]
    steps, peak = traces.mixed(requests, seed=9, max_live=3)
    out = tmp_path / "replayed"
    proc = subprocess.run([sys.executable, str(root / "bin" / "trace_run"), "--model", str(folder), "--dtype", "float32", "--out", str(out),
                           "--max-tokens", str(peak)], input=traces.strip(steps), capture_output=True, text=True, timeout=300, env=env, cwd=tmp_path)
    assert proc.returncode == 0, proc.stderr[-2000:]
    assert [line for line in proc.stdout.splitlines() if line.startswith("done ")] == [f"done {s['step']}" for s in steps]
    check(traces.collect(steps, out, raw["vocab"]), want, "float32")
