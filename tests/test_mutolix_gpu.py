"""Mutolix on the GPU against the plain implementation (tests/plain/mutolix.py): each mechanism alone (requests of unequal length
stepped side by side, slots and pages given back and used again), then whole models of the tests' own sizes under every way of cutting
their requests into steps, a key far back among hundreds, tokens at the edges of pages, of chunks and of the temperature's steps, gates
at their extremes, long decoding, and greedy generation through Engine and scheduler."""

import math

import numpy as np
import pytest
import torch

from tests import mutolix_configs as configs
from tests import traces
from tests.plain import mutolix as plain
from tests.test_felosun_gpu import LENGTHS, bf16_values, bound, part_weights, step_through
from tests.test_parts_gpu import PartHarness, close
from tests.test_replay_gpu import round64, run_replay

pytestmark = pytest.mark.gpu

DTYPES = [torch.float32, torch.bfloat16]
F64 = torch.float64


# ------------------------------------------------------------------------------------- mechanisms alone
# portions that end inside, at and just behind chunks of 64 tokens, beside single tokens; a slot that is given back and used again
LONG_SCHEDULE = [[("a", 64), ("b", 1)], [("a", 1), ("b", 65)], [("b", 63), ("a", 2)], [("a", 128)], [("a", 1), ("b", 1)], [("b", 40), ("a", 20)],
                 [("c", 130)], [("c", 1), ("a", 3)], [("a", 1), ("c", 1)]]
LONG_LENGTHS = {"a": 220, "b": 170, "c": 132}
MEMORIES = [
    # heads, dim, vdim, cap
    (2, 32, 48, 14.0),
    (3, 10, 18, 4.0),          # keys that are no multiple of four
    (1, 1, 1, 1.0),
    (5, 130, 7, 8.0),          # keys beyond 128
    (2, 256, 96, 15.0),        # the widest keys
    (4, 64, 33, 10.0),
    (12, 128, 128, 12.0),      # enough columns for the wider workgroups of the chunked form
]


def memory_part(width, heads, dim, vdim, cap, eps, dtype, seed, edit=None):
    from llm_runtime_study_amd.parts import PartSpec, create

    part = create("mixer", PartSpec("mlstm", {"hidden_size": width, "num_heads": heads, "head_dim": dim, "value_dim": vdim, "gate_cap": cap, "norm_eps": eps}))
    w = part_weights(part, seed)
    w["f_proj.bias"] = (2.0 + 4.0 * w["f_proj.bias"]).to(torch.bfloat16).double()
    w["i_proj.bias"] = (3.0 * w["i_proj.bias"]).to(torch.bfloat16).double()
    if edit is not None:
        edit(w)
    return part, bound(part, w, dtype), {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,dim,vdim,cap", MEMORIES)
def test_matrix_memory_part(dtype, heads, dim, vdim, cap):
    width = 56
    part, named, m = memory_part(width, heads, dim, vdim, cap, 1e-3, dtype, 60)
    assert named["i.b"].shape == (heads,) and named["norm"].shape == (heads * vdim,)
    for schedule, lengths, release in ((None, LENGTHS, (6, "b")), (LONG_SCHEDULE, LONG_LENGTHS, (6, "b"))):
        inputs = {key: bf16_values(n, width, seed=300 + i) for i, (key, n) in enumerate(lengths.items())}
        want = {key: plain.mlstm(x, named, m, 1e-3) for key, x in inputs.items()}
        kwargs = {} if schedule is None else {"schedule": schedule, "release_before": release}
        got, _ = step_through(part, dtype, inputs, width, **kwargs)
        for key in inputs:
            close(got[key], want[key][:got[key].shape[0]], dtype, f32=1e-4, bf16=2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("which", ["forgets at once", "never forgets", "one token outweighs", "writes next to nothing"])
def test_matrix_memory_with_gates_at_their_extremes(dtype, which):
    """Log gates far from zero: a memory that keeps one token only, one that keeps everything for hundreds of tokens, a single token
    whose input gate towers over all others (the running maximum jumps, and later tokens are measured against it), and input gates so
    small that the floor exp(-m) of the normaliser decides (with a maximum that starts at zero)."""
    width, heads, dim, vdim, cap = 64, 2, 32, 32, 20.0

    def edit(w):
        for name in ("i_proj.weight", "f_proj.weight"):
            w[name] = torch.zeros_like(w[name])
        w["i_proj.bias"] = torch.full_like(w["i_proj.bias"], {"writes next to nothing": -9.0}.get(which, 0.5))
        w["f_proj.bias"] = torch.full_like(w["f_proj.bias"], -18.0 if which == "forgets at once" else 16.0)
        if which == "one token outweighs":
            w["i_proj.weight"][:, 0] = 1.0                                # column 0 of the input is the input gate

    part, named, m = memory_part(width, heads, dim, vdim, cap, 1e-5, dtype, 70, edit)
    length = 220
    x = bf16_values(length, width, seed=4)
    x[:, 0] = 0.0
    x[100, 0] = 14.0
    want = plain.mlstm(x, named, m, 1e-5)
    if which == "one token outweighs":
        # what is read right behind the big token is that token's value (up to the sign of q . k): without it the row is another one
        other = x.clone()
        other[100, 0] = 0.0
        assert (plain.mlstm(other, named, m, 1e-5)[140] - want[140]).norm() > 0.5 * want[140].norm()
    for schedule in ([[("a", 219)], [("a", 1)]], [[("a", 90)], [("a", 2)], [("a", 3)], [("a", 64)]] + [[("a", 1)]] * 61):
        got, _ = step_through(part, dtype, {"a": x}, width, schedule=schedule, release_before=None)
        close(got["a"], want, dtype, f32=1e-4, bf16=2e-2)


def test_chunked_form_against_the_scan_on_the_same_numbers():
    """The two forms of a bfloat16 run on projections that bfloat16 holds exactly: read-outs and state rows agree to the two halves'
    precision, also where they take turns over one request, and the chunked form leaves rows beyond the request's slot alone."""
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(1)
    for heads, dim, vdim, lengths, singles in ((3, 24, 40, (130, 1, 64, 65), 0), (2, 256, 70, (200, 3), 0), (10, 128, 96, (64, 128, 5, 1, 63), 0),
                                               (1, 100, 17, (1,) * 70 + (300,), 0), (1, 100, 17, (1,) * 70 + (300, 1, 2), 70), (4, 64, 50, (1, 1, 1, 90), 2)):
        tokens, requests = sum(lengths), len(lengths)
        columns = 2 * heads * (dim + vdim + 1)
        proj = torch.randn(tokens, columns + 3, generator=g).to(torch.bfloat16).float().cuda()
        i_bias, f_bias = torch.randn(heads, generator=g).cuda(), (torch.randn(heads, generator=g) + 3).cuda()
        norm = (torch.rand(heads * vdim, generator=g) + 0.5).cuda()
        floats = ops.mlstm_state_floats(heads, dim, vdim)
        begun = (0.1 * torch.randn(requests + 1, floats, generator=g)).cuda()
        cu = torch.tensor([0] + list(np.cumsum(lengths)), dtype=torch.int32, device="cuda")
        of = torch.repeat_interleave(torch.arange(requests), torch.tensor(lengths)).int().cuda()
        slots = torch.randperm(requests, generator=g).int().cuda()
        floors, raw = torch.empty(tokens * heads, device="cuda"), torch.empty(tokens * heads * (vdim + 1), device="cuda")
        outs, states = [], []
        for chunked in (False, True):
            out, state = torch.zeros(tokens, heads * vdim, dtype=torch.bfloat16, device="cuda"), begun.clone()
            for _ in range(2):
                if chunked:
                    packs = tuple(torch.empty(n, dtype=torch.float32 if k == 3 else torch.bfloat16, device="cuda")
                                  for k, n in enumerate(ops.mlstm_pack_sizes(tokens, requests, heads, dim)))
                    ops.mlstm_chunks(out, proj, state, of, cu, slots, requests, heads, dim, vdim, i_bias, f_bias, 12.0, norm, 1e-5,
                                     torch.empty(requests * heads, device="cuda"), floors, raw, packs, singles)
                else:
                    ops.mlstm(out, proj, state, cu, slots, requests, heads, dim, vdim, i_bias, f_bias, 12.0, norm, 1e-5,
                              torch.empty(tokens * 2 * heads, device="cuda"), floors, raw)
            torch.cuda.synchronize()
            outs.append(out.double().cpu()), states.append(state.double().cpu())
        assert torch.equal(states[1][requests], begun[requests].double().cpu())
        assert (states[0] - states[1]).norm() < 2e-5 * states[0].norm(), (heads, dim, vdim)
        assert (outs[0] - outs[1]).norm() < 2e-3 * outs[0].norm(), (heads, dim, vdim)


ATTENTIONS = [
    # heads, kv, d, e, scale, temperature (coef, every)
    (6, 2, 20, 40, 0.21, (0.7, 5)),          # values wider than keys
    (6, 2, 64, 32, 0.13, (0.3, 24)),         # the matrix cores' shape, values half as wide
    (2, 1, 128, 128, 0.09, (0.5, 16)),       # heads of 128, values as wide
    (3, 1, 128, 48, 0.09, None),             # ... and narrower, three query heads on one key group
    (4, 4, 96, 96, 0.1, (1.0, 1)),           # a temperature that steps at every position
    (1, 1, 8, 8, 0.35, (0.4, 1000)),         # ... and one that never does
    (16, 1, 32, 16, 0.2, (-0.1, 7)),         # sixteen heads on one key group, a temperature that falls
    (3, 3, 20, 4, 0.25, None),
    (2, 2, 192, 64, 0.07, (0.2, 40)),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("mix", ["first", "later"])
@pytest.mark.parametrize("heads,groups,d,e,scale,temperature", ATTENTIONS)
def test_attention_part(dtype, heads, groups, d, e, scale, temperature, mix):
    from llm_runtime_study_amd.parts import PartSpec, create

    width, eps = 56, 1e-4

    def make(which, seed):
        part = create("mixer", PartSpec("gqa_attention", {
            "hidden_size": width, "num_heads": heads, "num_kv_heads": groups, "head_dim": d, "value_dim": e, "bias": True, "qk_norm": True,
            "qk_norm_eps": eps, "norm_over": "projection", "scale": scale, "sink": 0.0, "query_temperature": temperature, "value_mix": which,
            "distance_bias": True}))
        w = part_weights(part, seed)
        w["distance_rate"] = torch.linspace(0.02, 2.0, heads, dtype=F64).to(torch.bfloat16).double()
        w["distance_reach"] = torch.linspace(0.6, 0.05, heads, dtype=F64).to(torch.bfloat16).double()
        w["value_mix"] = torch.tensor(0.4375, dtype=F64)
        for name in ("q_norm.weight", "k_norm.weight"):
            w[name] = (1.0 + 0.3 * bf16_values(*w[name].shape, seed=seed)).to(torch.bfloat16).double()
        named = bound(part, w, dtype)
        named.update({"q.norm": w["q_norm.weight"], "k.norm": w["k_norm.weight"], "r1": w["distance_rate"], "r2": w["distance_reach"], "vmix": w["value_mix"]})
        return part, named

    m = {"heads": heads, "kv_heads": groups, "dim": d, "vdim": e, "scale": scale, "v_mix": True}
    if temperature is not None:
        m["q_temp"] = {"coef": temperature[0], "every": temperature[1]}
    inputs = {key: bf16_values(n, width, seed=400 + i) for i, (key, n) in enumerate(LENGTHS.items())}
    first, first_named = make("first", 50)
    shared = {key: [] for key in inputs}
    want = {key: plain.attention(x, first_named, m, eps, shared[key]) for key, x in inputs.items()}
    part = first
    if mix == "later":
        later, later_named = make("later", 90)
        want = {key: plain.attention(x, later_named, m, eps, shared[key]) for key, x in inputs.items()}

        class Both:
            """The first layer, for its values alone, and the one that mixes: two layers of one step."""

            def cache_need(self):
                return later.cache_need()

            def forward(self, ctx, x, out, cache, accumulate):
                aside = torch.zeros_like(out)
                first.forward(ctx, x, aside, cache, accumulate=False)          # (the pages it writes are written again by the next)
                later.forward(ctx, x, out, cache, accumulate=accumulate)

        # both layers write the same pages, so the first one's keys and values of earlier steps are gone: its output is not looked at
        part = Both()
    for page_size in (16, 4):
        got, _ = step_through(part, dtype, inputs, width, page_size=page_size)
        for key in inputs:
            close(got[key], want[key][:got[key].shape[0]], dtype, f32=5e-5, bf16=2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d,e", [(64, 64), (64, 16), (128, 128), (128, 64), (32, 48)])
def test_distance_bias_with_everything_else_on_the_scores(dtype, d, e):
    """A bias by distance behind a cap, with a window that keeps first positions and a gate a head: parameters of one mixer, whoever
    combines them.  Keys divided between workgroups too (700 positions)."""
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(d + e)
    heads, groups, length, page, window, kept, cap, scale = 4, 2, 700, 16, 90, 5, 2.0, 0.1
    q = torch.randn(length, heads, d, generator=g).to(dtype)
    k, v = torch.randn(length, groups, d, generator=g).to(dtype), torch.randn(length, groups, e, generator=g).to(dtype)
    gate = torch.randn(length, heads, generator=g).to(dtype)
    distance = torch.tensor([[0.02, 0.9, 2.0, 1.1], [0.5, 0.1, 0.3, 3.0]])
    sinks = torch.tensor([0.0, 0.0, 1.0, -2.0])
    blocks = -(-length // page)
    order = torch.randperm(blocks, generator=g)
    k_pages, v_pages = torch.zeros(blocks, groups, page, d, dtype=dtype), torch.zeros(blocks, groups, e, page, dtype=dtype)
    for p in range(length):
        k_pages[order[p // page], :, p % page] = k[p]
        v_pages[order[p // page], :, :, p % page] = v[p]
    table = order.int().view(1, -1).cuda()

    def wanted(rows, windowed):
        out = torch.zeros(len(rows), heads, e, dtype=F64)
        for n, i in enumerate(rows):
            for h in range(heads):
                j = torch.tensor([x for x in range(i + 1) if not windowed or i - x < window or x < kept])
                s = (k[j, h // 2].double() @ q[i, h].double()) * scale
                s = cap * torch.tanh(s / cap) - distance[0, h].double() * torch.log(1 + distance[1, h].double() * (i - j))
                p = torch.exp(s)
                out[n, h] = (p / (p.sum() + torch.exp(sinks[h].double()))) @ v[j, h // 2].double() * torch.sigmoid(gate[i, h].double())
        return out.reshape(len(rows), heads * e)

    for windowed in (False, True):
        more = {"window": window if windowed else 0, "keep_first": kept if windowed else 0, "sinks": sinks.cuda(), "softcap": cap, "distance": distance.cuda()}
        for rows in ([699], [3], list(range(640, 700))):
            positions = torch.tensor(rows, dtype=torch.int32, device="cuda")
            of = torch.zeros(len(rows), dtype=torch.int32, device="cuda")
            mine, gates = q[rows].reshape(len(rows), heads * d).cuda(), gate[rows].cuda()
            out = torch.zeros(len(rows), heads * e, dtype=dtype, device="cuda")
            ops.attention(out, mine, k_pages.cuda(), v_pages.cuda(), table, of, positions, heads, scale, gates=gates, **more)
            want = wanted(rows, windowed)
            close(out, want, dtype, f32=3e-5, bf16=1.5e-2)
            if not ops.attention_decode_supported(dtype, heads, groups, d, page, e):
                continue
            extra = 1 if windowed else 0
            for splits in (1, 3):
                part_o = torch.empty(len(rows), heads * (splits + extra) * e, device="cuda")
                part_ml = torch.empty(len(rows), heads * (splits + extra) * 2, device="cuda")
                out.zero_()
                if len(rows) == 1:
                    ops.attention_decode(out, mine, k_pages.cuda(), v_pages.cuda(), table, of, positions, heads, scale, splits=splits, part_o=part_o,
                                         part_ml=part_ml, form=1, gates=gates, **more)
                    close(out, want, dtype, bf16=1.5e-2)
                for size in (16, 32):
                    starts = torch.arange(0, len(rows), size, dtype=torch.int32, device="cuda")
                    counts = torch.clamp(len(rows) - starts, max=size).int()
                    out.zero_()
                    ops.attention_prefill(out, mine, k_pages.cuda(), v_pages.cuda(), table, of, positions, starts, counts, heads, scale, splits=splits,
                                          part_o=part_o, part_ml=part_ml, max_count=size, gates=gates, **more)
                    close(out, want, dtype, bf16=1.5e-2)


@pytest.mark.parametrize("stream,gate", [(torch.float32, torch.float32), (torch.bfloat16, torch.bfloat16), (torch.bfloat16, torch.float32)])
@pytest.mark.parametrize("cols", [48, 100, 37, 4096, 8192, 9000])
def test_gated_norm_add_kernel(stream, gate, cols):
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(cols)
    rows = 5
    h, y = torch.randn(rows, cols, generator=g), 3.0 * torch.randn(rows, cols, generator=g)
    wide = torch.randn(rows, cols + 24, generator=g).to(gate)
    z, bias = wide[:, 8:8 + cols], torch.randn(cols, generator=g)
    weight, following = torch.randn(cols, generator=g), torch.rand(cols, generator=g) + 0.5
    for gated, biased, normed in ((True, True, True), (True, False, True), (False, False, True), (True, True, False)):
        u = y.double() * (torch.sigmoid(z.double() + (bias.double() if biased else 0.0)) if gated else 1.0)
        want = h.double() + weight.double() * plain.rms_norm(u, None, 1e-3)
        out = h.clone().cuda()
        beside = torch.zeros(rows, cols, dtype=stream, device="cuda")
        ops.gated_norm_add(out, y.cuda(), wide.cuda()[:, 8:8 + cols] if gated else None, bias.cuda() if biased else None, weight.cuda(), 1e-3,
                           following.cuda() if normed else None, 1e-4, beside if normed else None)
        torch.testing.assert_close(out.cpu().double(), want, rtol=2e-5, atol=2e-5)
        if normed:
            close(beside, plain.rms_norm(want, following.double(), 1e-4), stream, f32=3e-5, bf16=5e-3)


@pytest.mark.parametrize("dtype", DTYPES)
def test_xielu_kernel_on_rows_of_any_stride(dtype):
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(2)
    for rows, cols, stride in ((7, 40, 40), (3, 15, 31), (9, 64, 96)):
        x = (2.0 * torch.randn(rows, stride, generator=g)).to(dtype)
        x[0, 0], x[0, 1], x[1, 0] = 0.0, 1e-6, -30.0
        numbers = torch.tensor([0.83, 0.5 + 0.37])
        src = x[:, :cols].double()
        want = torch.where(src > 0, 0.83 * src * src + src / 2, 0.87 * (torch.expm1(src) - src) + src / 2)
        out = torch.zeros(rows, cols, dtype=dtype, device="cuda")
        ops.xielu(out, x.cuda()[:, :cols], numbers.cuda())
        close(out, want, dtype, f32=1e-5, bf16=4e-3)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_block_with_and_without_gate_scale_and_feed_forward(dtype):
    """The arrangement of norms alone, every combination of its parameters, with a mixer that carries the gate's matrix and one that does
    not (attention with per-head norms), against the plain update."""
    from llm_runtime_study_amd.parts import PartSpec, create

    width, tokens = 64, 9
    norm = PartSpec("rmsnorm", {"size": width, "eps": 1e-4})
    memory = PartSpec("mlstm", {"hidden_size": width, "num_heads": 2, "head_dim": 16, "value_dim": 24, "gate_cap": 6.0, "norm_eps": 1e-4})
    ff = PartSpec("dense_mlp", {"hidden_size": width, "intermediate_size": 40, "activation": "xielu"})
    ff_plain = PartSpec("dense_mlp", {"hidden_size": width, "intermediate_size": 40, "activation": "gelu"})
    names = {"mixer": "mix", "feed_forward": "mlp", "mixer_norm": "norm1", "mixer_out_norm": "norm1b", "ff_norm": "norm2", "ff_out_norm": "norm2b",
             "mixer_gate": "rg1", "ff_gate": "rg2", "mixer_scale": "ls1", "ff_scale": "ls2"}
    m = {"heads": 2, "dim": 16, "vdim": 24, "gate_cap": 6.0}
    for gated, scaled, feed in ((True, True, ff), (True, False, ff_plain), (False, True, ff), (False, False, None), (True, True, None)):
        params = {"mixer": memory, "mixer_norm": norm, "mixer_out_norm": norm, "gated": gated, "scaled": scaled, "names": names}
        if feed is not None:
            params.update(feed_forward=feed, ff_norm=norm, ff_out_norm=norm)
        block = create("block", PartSpec("sandwich", params))
        w = part_weights(block, 33)
        for name in w:
            if name.endswith(("norm1.weight", "norm1b.weight", "norm2.weight", "norm2b.weight", "norm.weight")):
                w[name] = (1.0 + 0.2 * w[name]).to(torch.bfloat16).double()
        named = bound(block, w, dtype)
        named.update({"norm1": named.get("norm1"), "rg1": named.get("rg1", torch.zeros(width, width, dtype=F64))})
        # a gate that is not there is one (a bias of 60), a scale that is not there is one
        for number in (1, 2):
            named.setdefault(f"rg{number}", torch.zeros(width, width, dtype=F64))
            named.setdefault(f"rg{number}.b", torch.full((width,), 60.0, dtype=F64))
            named.setdefault(f"ls{number}", torch.ones(width, dtype=F64))
        if not gated:
            named["rg1"] = torch.zeros(width, width, dtype=F64)
        x = bf16_values(tokens, width, seed=3)
        mix, mlp = plain.under(named, "mix."), plain.under(named, "mlp.")
        want = plain.update(x, named, 1, lambda u: plain.mlstm(u, mix, m, 1e-4), 1e-4)
        if feed is ff:
            want = plain.update(want, named, 2, lambda u: plain.feed_forward(u, mlp), 1e-4)
        elif feed is ff_plain:
            want = plain.update(want, named, 2, lambda u: torch.nn.functional.gelu(u @ mlp["up"].T) @ mlp["down"].T, 1e-4)
        harness = PartHarness([block.cache_need()], dtype)
        ctx = harness.context([(harness.cache.admit("a"), [0] * tokens)])
        h = x.float().cuda()
        after = create("norm", norm)
        after.bind({"weight": torch.ones(width, device="cuda")}, dtype)
        handed = block.forward(ctx, h, ctx.layer_cache(0), next_norm=after)
        close(h, want, dtype, f32=1e-4, bf16=1e-2)
        assert handed[0] is after
        close(handed[1], plain.rms_norm(want, None, 1e-4), dtype, f32=1e-4, bf16=1e-2)


# ------------------------------------------------------------------------------------- whole models
RAW = {name: configs.ALL[name] for name in ("odd", "cores", "ones", "awkward")}
MODEL_LENGTHS = {"odd": [70, 33, 9, 1, 52, 17, 66], "cores": [150, 64, 2, 97, 33], "ones": [40, 1, 65, 16, 5], "awkward": [90, 31, 3, 48, 17]}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    out = {}
    for number, (name, raw) in enumerate(RAW.items()):
        folder = configs.write_folder(raw, 260 + number, tmp_path_factory.mktemp(f"mutolix_{name}"))
        tensors, _ = plain.load_model_dir(folder)
        rng = np.random.default_rng(221 + number)
        requests = {f"{name}{i}": rng.integers(0, raw["vocab"], n).tolist() for i, n in enumerate(MODEL_LENGTHS[name])}
        out[name] = (folder, raw, requests, {key: plain.forward(tensors, raw, tokens) for key, tokens in requests.items()})
    return out


def check(got, want, dtype, share=1.0):
    """Every row as a whole (relative L2): float32 within 2e-4; bfloat16 within 8 % (these models are a few dozen values wide and
    normalise every sublayer's output, so that a small one is blown up with its rounding), half of them within 3 %.  share: how many of
    a bfloat16 run's rows must be that close (a memory whose heads hold one value each gives out that value's sign, which a rounding
    can turn)."""
    errors = np.array([float((row.double() - want[key][position]).norm() / want[key][position].norm())
                       for key, rows in got.items() for position, row in rows.items()])
    if dtype == "float32":
        assert errors.max() < 2e-4, f"the worst row is off by {errors.max():.3g}"
    else:
        assert np.mean(errors < 8e-2) >= share and np.median(errors) < 3e-2, f"the worst row is off by {errors.max():.3g}, the median by {np.median(errors):.3g}"
    return len(errors)


def test_the_stream_after_every_layer(models):
    """One step function call on a whole prompt in float32, the stream read after every layer, against the plain implementation's."""
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
    share = 0.85 if name == "ones" else 1.0
    longest = max(round64(len(t)) for t in requests.values())
    steps = traces.whole(requests)
    got = traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "whole"), raw["vocab"])
    assert check(got, want, dtype, share) == sum(len(t) for t in requests.values())
    steps = traces.prefill_then_decode(requests, tail=50)
    check(traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "tail"), raw["vocab"]), want, dtype, share)
    steps = traces.portions(requests)
    check(traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "portions", page_size=32), raw["vocab"]), want, dtype, share)
    few = {key: tokens for key, tokens in requests.items() if len(tokens) < 70}
    steps = traces.portions(few, sizes=(2, 2, 3, 2))
    check(traces.collect(steps, run_replay(folder, dtype, steps, longest, tmp_path / "twos"), raw["vocab"]), want, dtype, share)


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
    assert check(got, want, dtype, 0.85 if name == "ones" else 1.0) > 30
    assert peak < sum(round64(len(t)) for t in requests.values())


@pytest.mark.parametrize("name", ["odd", "cores"])
def test_the_engines_path_of_graphs_and_recorded_steps(models, name, tmp_path):
    """On a stream of the runner's own with graphs on: single-token steps are graph replays, shapes that come back are launched from
    their recorded plan."""
    folder, raw, requests, want = models[name]
    longest = max(round64(len(t)) for t in requests.values())
    seen = {}
    for dtype in ("float32", "bfloat16"):
        steps = traces.prefill_then_decode(requests, tail=40)
        out = run_replay(folder, dtype, steps, longest, tmp_path / f"tail_{dtype}", as_the_engine=True, counters=seen)
        check(traces.collect(steps, out, raw["vocab"]), want, dtype)
        assert seen["graph_replays"] >= 20 * (len(requests) - 2)
        steps = traces.portions(requests, sizes=(16, 16, 16, 2)) if dtype == "float32" else traces.portions(requests, sizes=(24, 24, 24, 2))
        out = run_replay(folder, dtype, steps, longest, tmp_path / f"portions_{dtype}", as_the_engine=True, counters=seen)
        check(traces.collect(steps, out, raw["vocab"]), want, dtype)
        assert seen["plan_replays"] >= 3
    steps, peak = traces.mixed(requests, seed=5, max_live=4, max_tokens=2 * longest)
    out = run_replay(folder, "bfloat16", steps, peak, tmp_path / "mixed", as_the_engine=True, counters=seen)
    check(traces.collect(steps, out, raw["vocab"]), want, "bfloat16")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_a_wider_model_through_the_products_for_many_rows(tmp_path, dtype):
    """Width 512 and prompts of 330 and 140 tokens: the projections of a prompt are products of hundreds of rows (the vendor library's
    in bfloat16), the memories walk five chunks, the temperature steps inside the prompt."""
    raw = configs.WIDE
    folder = configs.write_folder(raw, 21, tmp_path / "wide")
    tensors, _ = plain.load_model_dir(folder)
    rng = np.random.default_rng(4)
    requests = {"long": rng.integers(0, raw["vocab"], 330).tolist(), "short": rng.integers(0, raw["vocab"], 140).tolist()}
    want = {key: plain.forward(tensors, raw, tokens) for key, tokens in requests.items()}
    steps = [{"step": 0, "entries": [{"id": key, "tokens": tokens[:-6], "want": list(range(0, len(tokens) - 6, 7))} for key, tokens in requests.items()], "end": []}]
    for i in range(6, 0, -1):
        steps.append({"step": len(steps), "entries": [{"id": key, "tokens": [tokens[-i]], "want": [0]} for key, tokens in requests.items()],
                      "end": list(requests) if i == 1 else []})
    got = traces.collect(steps, run_replay(folder, dtype, steps, 512, tmp_path / "o"), raw["vocab"])
    assert check(got, want, dtype) > 70


def test_a_checkpoint_that_holds_the_first_mixing_layers_own_factor(models, tmp_path):
    """The layer whose values the others take has no use for a factor of its own; a checkpoint may hold one all the same."""
    from llm_runtime_study_amd.engine import trace
    from llm_runtime_study_amd.engine.step import StepEntry

    raw = RAW["odd"]
    folder = configs.write_folder(raw, 260, tmp_path / "with", edit=lambda tensors: tensors.update({"l0.mix.vmix": torch.tensor(0.9, dtype=torch.bfloat16)}))
    _, _, requests, want = models["odd"]
    runner = trace.make_runner(folder, "float32", 128, 16)
    logits = runner.step([StepEntry(runner.cache.admit("r"), requests["odd1"], list(range(33)))]).cpu().double()
    assert (logits - want["odd1"]).norm() < 1e-4 * want["odd1"].norm()


def test_bfloat16_path_follows_float32_at_real_layer_sizes():
    """Four layers at the sizes of a real model's (width 1,024, memories of 256 x 512, 16 heads of 128 on 8 key groups, a feed-forward of
    3,072, a vocabulary of 8,000): the bfloat16 path with everything it uses at that size (graphs, the vendor's products, chunks on the
    matrix cores, the prefill kernel for heads of 128 with a bias by distance, key splits, values stored as runs) against the float32
    path of the same weights, over prompts in two portions beside decoding requests and decode steps."""
    from llm_runtime_study_amd.benchmarks.shapes import SHAPES, mutolix_like
    from llm_runtime_study_amd.cache import CacheManager
    from llm_runtime_study_amd.config import config_from_dict, spec_for
    from llm_runtime_study_amd.engine.step import ModelRunner, StepEntry
    from llm_runtime_study_amd.models import DecoderModel
    from llm_runtime_study_amd.weights import random_init

    cfg = config_from_dict(mutolix_like(dict(SHAPES["0.6b"], vocab_size=8000), 4))
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
                half = len(prompt) // 2
                decoding = [StepEntry(caches[j], [tails[j][fed[j]]], [0]) for j in sorted(fed)]
                for j in fed:
                    fed[j] += 1
                rows.append(runner.step(decoding + [StepEntry(caches[i], prompt[:half], [half - 1])]).float().cpu())
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
    # (two sublayers in three are normalised to a size of their own, so a row whose memory reads out next to nothing is blown up)
    assert (error < 5e-2).float().mean() > 0.97 and error.max() < 0.15 and error.median() < 1.5e-2, f"median {error.median():.3g}, worst {error.max():.3g}"


# ------------------------------------------------------------------------------------- planted inputs
def planted_model(tmp_path, layer):
    """A model of one attention layer whose query matrix is its key matrix behind a swap of the two halves of the stream: the query of
    token B is the key of token A when A's embedding is B's with its halves swapped (no biases, the norms' weights all one).  Both are
    of unit size over the whole projection, so the match scores about dim * scale, which towers over every other score: a B reads A's
    value exactly when it sees it.  Token 0 is A, token 1 B."""
    raw = configs.model(50, 32, 1e-6, 1.0, [layer])

    def edit(tensors):
        k = tensors["l0.mix.k"]
        tensors["l0.mix.q"] = torch.cat((k[:, 16:], k[:, :16]), 1).contiguous()
        for name in ("l0.mix.q.b", "l0.mix.k.b"):
            tensors[name].zero_()
        for name in ("l0.norm1", "l0.mix.q.norm", "l0.mix.k.norm"):
            tensors[name].fill_(1.0)
        embed = tensors["embed"]
        embed[0] = torch.cat((embed[1, 16:], embed[1, :16]))

    return raw, configs.write_folder(raw, 77, tmp_path / "planted", edit=edit)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("dim,vdim", [(32, 32), (64, 32), (128, 128), (24, 40)])
def test_a_key_far_back_among_hundreds(tmp_path, dtype, dim, vdim):
    """The one matching key lies 600 positions back, in the prompt's first page, and is found (by a head with a small rate) from a
    prompt's portion and from a single decoded token, and at the borders of pages."""
    layer = configs.attention(2, 2, dim, vdim, 16.0 / dim, q_temp=(0.3, 50))
    raw, folder = planted_model(tmp_path, layer)
    tensors, _ = plain.load_model_dir(folder)
    rng = np.random.default_rng(2)
    base = rng.integers(2, raw["vocab"], 660).tolist()
    places = {"with": (7, 607), "decoded": (15, 650), "page_first": (16, 608), "page_last": (31, 639), "very_first": (0, 640)}
    requests = {}
    for key, (first, second) in places.items():
        requests[key] = list(base)
        requests[key][first], requests[key][second] = 0, 1
    requests["without"] = list(requests["with"])
    requests["without"][7] = 9
    asked = {**{key: second for key, (_, second) in places.items()}, "without": 607}
    want = {key: plain.forward(tensors, raw, tokens) for key, tokens in requests.items()}
    assert (want["with"][607] - want["without"][607]).norm() > 0.1 * want["with"][607].norm()
    steps = []
    for key, tokens in requests.items():
        cut = asked[key] if key != "with" else 300                        # the asking token alone, or inside a portion
        steps.append({"step": len(steps), "entries": [{"id": key, "tokens": tokens[:cut], "want": [cut - 1]}], "end": []})
        if key == "with":
            steps.append({"step": len(steps), "entries": [{"id": key, "tokens": tokens[cut:], "want": list(range(300, 360))}], "end": [key]})
        else:
            steps.append({"step": len(steps), "entries": [{"id": key, "tokens": [tokens[cut]], "want": [0]}], "end": []})
            steps.append({"step": len(steps), "entries": [{"id": key, "tokens": tokens[cut + 1:cut + 3], "want": [0, 1]}], "end": [key]})
    got = traces.collect(steps, run_replay(folder, dtype, steps, 704, tmp_path / "o"), raw["vocab"])
    check(got, want, dtype)
    for key, position in asked.items():
        row, ref = got[key][position].double(), want[key][position]
        assert (row - ref).norm() < (1e-4 if dtype == "float32" else 5e-2) * ref.norm(), (key, position)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_places_just_before_and_just_behind_a_step_of_the_temperature(tmp_path, dtype):
    """A coarse temperature (queries four times as long behind every step): the rows on either side of a step, in prompts, in portions of two
    and decoded alone; without the step the row behind it would be another one."""
    every = 16
    raw = configs.model(60, 40, 1e-6, 1.0, [configs.attention(2, 1, 16, 16, 0.4, q_temp=(3.0, every), v_mix=True, ff=24)])
    folder = configs.write_folder(raw, 5, tmp_path / "stepped")
    tensors, _ = plain.load_model_dir(folder)
    tokens = np.random.default_rng(3).integers(0, 60, 70).tolist()
    want = {"t": plain.forward(tensors, raw, tokens)}
    late = configs.model(60, 40, 1e-6, 1.0, [configs.attention(2, 1, 16, 16, 0.4, q_temp=(3.0, every + 1), v_mix=True, ff=24)])
    moved = plain.forward(tensors, late, tokens)
    for p in (every - 1, 2 * every - 1):                                  # (p + 1) / every steps there: a step one place later shows
        assert (moved[p] - want["t"][p]).norm() > 0.05 * want["t"][p].norm()
    for number, steps in enumerate((traces.whole({"t": tokens}), traces.prefill_then_decode({"t": tokens}, tail=60), traces.portions({"t": tokens}, sizes=(2, 3, 2, 5)))):
        got = traces.collect(steps, run_replay(folder, dtype, steps, 128, tmp_path / f"o{number}"), raw["vocab"])
        check(got, want, dtype)
        for p in [q for edge in range(every, 70, every) for q in (edge - 2, edge - 1, edge)]:
            assert (got["t"][p].double() - want["t"][p]).norm() < (1e-4 if dtype == "float32" else 3e-2) * want["t"][p].norm(), p


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sink_of_score_zero_where_every_score_is_far_below_it(dtype):
    """Scores around minus six through a strong bias by distance and a query far from its keys: most of the weight goes to the sink, and
    an attention without it would give rows many times as long."""
    from llm_runtime_study_amd.kernels import ops

    g = torch.Generator().manual_seed(9)
    heads, d, length, page = 2, 64, 96, 16
    k = torch.randn(length, 1, d, generator=g).abs().to(dtype)
    q = (-torch.rand(length, heads, d, generator=g)).to(dtype)
    v = torch.randn(length, 1, d, generator=g).to(dtype)
    distance = torch.tensor([[0.5, 2.0], [0.2, 0.4]])
    k_pages, v_pages = torch.zeros(6, 1, page, d, dtype=dtype), torch.zeros(6, 1, d, page, dtype=dtype)
    for p in range(length):
        k_pages[p // page, 0, p % page], v_pages[p // page, 0, :, p % page] = k[p, 0], v[p, 0]
    want, total = torch.zeros(length, heads * d, dtype=F64), []
    for i in range(length):
        for h in range(heads):
            s = (k[:i + 1, 0].double() @ q[i, h].double()) * 0.25 - distance[0, h].double() * torch.log(1 + distance[1, h].double() * torch.arange(i, -1, -1))
            p = torch.exp(s)
            total.append(float(p.sum()))
            want[i, h * d:(h + 1) * d] = (p / (1 + p.sum())) @ v[:i + 1, 0].double()
    assert max(total) < 0.2
    rows = torch.arange(length, dtype=torch.int32, device="cuda")
    of, table = torch.zeros_like(rows), torch.arange(6, dtype=torch.int32, device="cuda").view(1, -1)
    out = torch.zeros(length, heads * d, dtype=dtype, device="cuda")
    more = {"sinks": torch.zeros(heads, device="cuda"), "distance": distance.cuda()}
    ops.attention(out, q.reshape(length, -1).cuda(), k_pages.cuda(), v_pages.cuda(), table, of, rows, heads, 0.25, **more)
    close(out, want, dtype, f32=1e-6, bf16=1e-2)
    if dtype == torch.bfloat16:
        starts = torch.arange(0, length, 16, dtype=torch.int32, device="cuda")
        out.zero_()
        ops.attention_prefill(out, q.reshape(length, -1).cuda(), k_pages.cuda(), v_pages.cuda(), table, of, rows, starts, torch.full_like(starts, 16),
                              heads, 0.25, max_count=16, **more)
        close(out, want, dtype, bf16=1e-2)
        one = torch.zeros(1, heads * d, dtype=dtype, device="cuda")
        ops.attention_decode(one, q[95:].reshape(1, -1).cuda(), k_pages.cuda(), v_pages.cuda(), table, of, rows[95:], heads, 0.25, **more)
        close(one, want[95:], dtype, bf16=1e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_beside_a_second_request(models, dtype, tmp_path):
    """240 tokens one by one behind a prompt of ten, a second request's tokens beside them."""
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
    """Three prompts on two slots (the third waits and takes a freed slot, its state and its pages), prompts fed in portions of at most
    16 tokens beside decoding requests: the tokens are the plain implementation's own greedy continuation."""
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
    assert engine.cache_manager.active_requests == 0
    fast = Engine.from_model_dir(folder, dtype="bfloat16", max_seq_len=128, max_batch_size=3, max_num_batched_tokens=64)
    assert [len(tokens) for tokens in fast.generate_tokens(prompts, max_new_tokens=6)] == [6, 6, 6]


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
