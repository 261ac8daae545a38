"""Tamilix without a GPU: its configuration, the tensors it asks a checkpoint for, what its layers keep between steps and when they give
it back, and the plain implementation's mechanisms against properties that follow from their definitions."""

import copy
import math

import pytest
import torch

from tests import tamilix_configs as configs
from tests.plain import tamilix as plain

F64 = torch.float64


def values(*shape, seed=0, scale=1.0):
    return scale * torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


# ------------------------------------------------------------------------------------- configuration, names, needs
def test_configuration_reads_back_and_names_its_tensors():
    from llm_runtime_study_amd.config import config_from_dict, spec_for
    from llm_runtime_study_amd.config.tamilix import TamilixConfig
    from llm_runtime_study_amd.models import DecoderModel
    from llm_runtime_study_amd.parts import PagedKVNeed

    for raw in configs.ALL.values():
        config = config_from_dict(raw)
        assert isinstance(config, TamilixConfig) and config.to_json_dict() == raw
        model = DecoderModel(spec_for(config))
        names, width = model.tensors(), raw["width"]
        expected = {"embed": (raw["vocab"], width), "head": (raw["vocab"], width), "final.norm": (width,)}
        for index, layer in enumerate(raw["layers"]):
            if "weights_of" in layer:
                continue
            m, mlp, p = layer["mixer"], layer["mlp"], f"l{index}."
            shapes = {"norm1": (width,), "norm1b": (width,)}
            h, d, e = m["heads"], m["dim"], m["vdim"]
            if layer["type"] == "attention":
                g = m["kv_heads"]
                shapes.update({"mix.q": (h * d, width), "mix.k": (g * d, width), "mix.v": (g * e, width), "mix.sink": (h,), "mix.o": (width, h * e)})
            else:
                q, c, r = m["q_rank"], m["kv_rank"], m["rot_dim"]
                shapes.update({"mix.dq": (q, width), "mix.dq.norm": (q,), "mix.uq": (h * (d + r), q), "mix.dkv": (c + r, width), "mix.dkv.norm": (c,),
                               "mix.uk": (h * d, c), "mix.uv": (h * e, c), "mix.g": (h * e, width), "mix.o": (width, h * e)})
            if mlp is not None:
                shapes.update({"norm2": (width,), "norm2b": (width,)})
                if mlp["kind"] == "dense":
                    shapes.update({"mlp.up": (mlp["ff"], width), "mlp.down": (width, mlp["ff"])})
                else:
                    ff, outputs = mlp["expert"]["ff"], mlp["router"]["experts"] + mlp["router"]["identity"]
                    shapes.update({"mlp.router": (outputs, width), "mlp.correction": (outputs,)})
                    for x in range(mlp["router"]["experts"]):
                        shapes.update({f"mlp.e{x}.gate": (ff, width), f"mlp.e{x}.up": (ff, width), f"mlp.e{x}.down": (width, ff)})
                    if "shared" in mlp:
                        sf = mlp["shared"]["ff"]
                        shapes.update({"mlp.shared.gate": (sf, width), "mlp.shared.up": (sf, width), "mlp.shared.down": (width, sf)})
            expected.update({p + name: shape for name, shape in shapes.items()})
        assert {name: tuple(spec.shape) for name, spec in names.items()} == expected
        assert len(model.cache_needs()) == len(raw["layers"])
        for layer, need in zip(raw["layers"], model.cache_needs()):
            m = layer["mixer"]
            size = m["mask"]["size"] if "mask" in m else None
            assert isinstance(need, PagedKVNeed) and need.span == size
            if layer["type"] == "attention":
                assert (need.num_kv_heads, need.head_dim, need.chunk, need.window) == (m["kv_heads"], m["dim"], size, None)
                assert (need.value_dim or need.head_dim) == m["vdim"]
            else:
                assert (need.num_kv_heads, need.head_dim, need.chunk, need.window) == (1, m["kv_rank"] + m["rot_dim"], None, size)


def test_what_the_file_leaves_out_does_not_exist():
    from llm_runtime_study_amd.config import config_from_dict, spec_for

    raw = copy.deepcopy(configs.ODD)
    del raw["embedding"], raw["layers"][1]["mixer"]["mask"], raw["layers"][5]["mixer"]["mask"], raw["layers"][3]["mlp"]
    del raw["layers"][0]["mlp"]["shared"], raw["layers"][2]["mlp"]["shared"], raw["layers"][0]["mlp"]["router"]["identity"], raw["layers"][2]["mlp"]["router"]["identity"]
    config = config_from_dict(raw)
    assert config.embedding_scale == 1.0 and config.layers[1].mixer.chunk is None and config.layers[3].mlp is None
    assert config.layers[0].mlp.identity == 0 and config.layers[0].mlp.shared_ff is None
    spec = spec_for(config)
    assert spec.layers[1].params["mixer"].params["chunk"] is None and "feed_forward" not in spec.layers[2].params
    # an entry that runs with another layer's weights may leave out what equals the owner's
    short = copy.deepcopy(configs.ODD)
    short["layers"][2] = {"weights_of": 0}
    assert config_from_dict(short).to_json_dict() == configs.ODD


def refused(change):
    from llm_runtime_study_amd.config import config_from_dict
    from llm_runtime_study_amd.errors import ConfigError

    raw = copy.deepcopy(configs.ODD)
    change(raw)
    with pytest.raises(ConfigError) as caught:
        config_from_dict(raw)
    return str(caught.value)


def test_refusals_name_the_layer():
    assert "layer 3" in refused(lambda raw: raw["layers"][3].update(type="mamba"))
    assert "heads" in refused(lambda raw: raw["layers"][1]["mixer"].update(kv_heads=4))
    assert "layer 0" in refused(lambda raw: raw["layers"][0]["mixer"].pop("q_rank"))
    assert "rot" in refused(lambda raw: raw["layers"][0]["mixer"]["rot"].update(dims=4))
    assert "rot" in refused(lambda raw: raw["layers"][4]["mixer"].pop("rot"))
    assert "base" in refused(lambda raw: raw["layers"][4]["mixer"]["rot"].update(base=1.0))
    assert "scale" in refused(lambda raw: raw["layers"][3]["mixer"].pop("scale"))
    assert "size" in refused(lambda raw: raw["layers"][3]["mixer"]["mask"].update(size=0))
    assert "kind" in refused(lambda raw: raw["layers"][4]["mlp"].update(kind="gated"))
    assert "identity" in refused(lambda raw: raw["layers"][0]["mlp"]["router"].update(identity=-1))
    assert "choices" in refused(lambda raw: raw["layers"][0]["mlp"]["router"].update(top=9))
    assert "limit" in refused(lambda raw: raw["layers"][0]["mlp"]["expert"].pop("limit"))
    assert "shared" in refused(lambda raw: raw["layers"][0]["mlp"]["shared"].update(limit=0.0))
    assert "mlp" in refused(lambda raw: raw["layers"][4].update(mlp=4))
    assert "weights_of" in refused(lambda raw: raw["layers"][2].update(weights_of=2))
    assert "weights_of" in refused(lambda raw: raw["layers"][2].update(weights_of=17))
    assert "own" in refused(lambda raw: raw["layers"].append({"weights_of": 2}))
    assert "equal" in refused(lambda raw: raw["layers"][2]["mixer"].update(scale=0.5))
    assert "eps" in refused(lambda raw: raw["norm"].update(eps=0.0))
    assert "layers" in refused(lambda raw: raw.update(layers=[]))


def test_parts_refuse_what_they_cannot_run():
    from llm_runtime_study_amd.parts import PartSpec, create

    sizes = {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16}
    for bad in ({"chunk": 0}, {"chunk": 4, "window": 4}, {"chunk": 4, "keep_first": 2}, {"distance_bias": "log"}):
        with pytest.raises(ValueError):
            create("mixer", PartSpec("gqa_attention", dict(sizes, **bad)))
    latent = {"hidden_size": 32, "num_heads": 2, "head_dim": 16, "rot_dim": 4, "value_dim": 8, "kv_rank": 12,
              "position": PartSpec("rope_interleaved", {"rotary_dim": 4, "theta": 10.0})}
    create("mixer", PartSpec("latent_attention", latent))
    for bad in ({"q_rank": 0}, {"gate": "head"}, {"window": 3, "chunk": 3}, {"chunk": -1}, {"q_rank": 4, "position": PartSpec("none")}):
        with pytest.raises(ValueError):
            create("mixer", PartSpec("latent_attention", dict(latent, **bad)))
    routed = {"hidden_size": 32, "intermediate_size": 8, "num_experts": 3, "top": 4, "rule": "softmax_scores"}
    assert create("feed_forward", PartSpec("routed_experts", dict(routed, identity=1))).choices == 4
    for bad in ({}, {"identity": -1, "top": 1}, {"identity": 510, "top": 1}, {"identity": 1, "groups": 2, "keep": 1, "rule": "sigmoid"},
                {"identity": 1, "activation": "clamped_gated", "activation_limit": 1.0, "weight_on": "input"}):
        with pytest.raises(ValueError):
            create("feed_forward", PartSpec("routed_experts", dict(routed, **bad)))


# ------------------------------------------------------------------------------------- pages of layers that see a chunk
def test_pages_of_past_chunks_are_given_back():
    from llm_runtime_study_amd.cache import CacheManager
    from llm_runtime_study_amd.parts import PagedKVNeed

    for page, chunk in ((4, 10), (16, 16), (4, 3), (8, 1), (5, 40)):
        need = PagedKVNeed(2, 16, chunk=chunk)
        cache = CacheManager([need, PagedKVNeed(2, 16)], page_size=page, num_pages=64, max_requests=2, max_seq_len=200, allocate_storage=False)
        request = cache.admit("a")
        other = cache.admit("b")
        cache.extend(other, 7)
        for portion in (1, 2, 7, 1, 1, 19, 4, 1, 30, 1, 1, 1, 12):
            before = request.length
            cache.extend(request, portion)
            for position in range(before, request.length):        # everything a query of this step sees is still there
                for j in range(position // chunk * chunk, position + 1):
                    cache.slot_of_position(request, 0, j)
            cache.trim(request)
            cache.check_invariants()
            first = request.length // chunk * chunk               # where the next query's chunk begins
            held = [b for b, p in enumerate(request.tables[0]) if p >= 0]
            assert held == list(range(first // page, -(-request.length // page)))
            assert all(p >= 0 for p in request.tables[1])         # the layer that sees everything keeps everything
        assert cache.pages_for(0, 200, 20) == min(-(-200 // page), -(-chunk // page) + -(-20 // page) + 2)
        cache.release(request)
        cache.release(other)
        assert cache.used_pages(0) == 0


def test_layers_of_different_chunks_and_windows_have_pools_of_their_own():
    from llm_runtime_study_amd.cache import CacheManager
    from llm_runtime_study_amd.parts import PagedKVNeed

    needs = [PagedKVNeed(1, 8, chunk=6), PagedKVNeed(1, 8, window=6), PagedKVNeed(1, 8, chunk=6), PagedKVNeed(1, 8)]
    cache = CacheManager(needs, page_size=4, num_pages=9, max_requests=1, max_seq_len=36, allocate_storage=False)
    assert [c.group for c in cache.layer_caches] == [0, 1, 0, 2]
    assert [n.first_needed(11) for n in needs] == [6, 6, 6, 0] and [n.first_needed(12) for n in needs] == [12, 7, 12, 0]


# ------------------------------------------------------------------------------------- the plain mechanisms
def test_masks_at_their_edges():
    assert [plain.in_window(9, j, 3) for j in range(12)] == [j in (7, 8, 9) for j in range(12)]
    assert [plain.in_chunk(9, j, 4) for j in range(12)] == [j in (8, 9) for j in range(12)]
    assert [plain.in_chunk(11, j, 4) for j in range(13)] == [8 <= j <= 11 for j in range(13)] and [plain.in_chunk(12, j, 4) for j in range(13)] == [j == 12 for j in range(13)]
    assert all(plain.in_chunk(5, j, None) == (j <= 5) == plain.in_window(5, j, None) for j in range(9))


def test_slopes():
    assert [plain.slope(h, 8) for h in range(8)] == [2.0 ** -(h + 1) for h in range(8)]
    assert plain.slope(0, 1) == 2.0 ** -8 and plain.slope(5, 6) == 2.0 ** -8 and math.isclose(plain.slope(0, 6), 2.0 ** (-4 / 3))


def test_attention_in_chunks_against_its_definition_at_one_place():
    m = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 5, "scale": 0.4, "mask": {"size": 5}}
    width = 24
    w = {"q": values(24, width, seed=1, scale=0.3), "k": values(12, width, seed=2, scale=0.3), "v": values(10, width, seed=3), "sink": values(4, seed=4), "o": torch.eye(20, dtype=F64)}
    x = values(14, width, seed=5)
    seen = []
    out = plain.attention(x, w, m, seen)
    i, h, g = 13, 3, 1
    q, k, v = x[i] @ w["q"][h * 6:h * 6 + 6].T, x @ w["k"][g * 6:g * 6 + 6].T, x @ w["v"][g * 5:g * 5 + 5].T
    raised = {j: math.exp(float(q @ k[j]) * 0.4 - 2.0 ** -8 * (i - j)) for j in (10, 11, 12, 13)}
    total = sum(raised.values()) + math.exp(float(w["sink"][h]))
    assert torch.allclose(out[i, h * 5:h * 5 + 5], sum(raised[j] / total * v[j] for j in raised))
    for head, place, keys, weights in seen:
        assert keys == list(range(place // 5 * 5, place + 1)) and 0 < float(weights.sum()) < 1          # the rest is the sink's share
    # the first token of a chunk sees itself alone
    only = [weights for head, place, keys, weights in seen if place == 10]
    assert all(len(weights) == 1 for weights in only)


def test_latent_attention_against_its_definition_at_one_place():
    m = {"heads": 2, "dim": 5, "rot_dim": 4, "vdim": 3, "q_rank": 7, "kv_rank": 6, "scale": 0.5, "mask": {"size": 3}, "rot": {"base": 20.0, "dims": 4}}
    width, eps = 16, 1e-3
    w = {"dq": values(7, width, seed=1), "dq.norm": 1 + values(7, seed=2) * 0.1, "uq": values(18, 7, seed=3), "dkv": values(10, width, seed=4),
         "dkv.norm": 1 + values(6, seed=5) * 0.1, "uk": values(10, 6, seed=6), "uv": values(6, 6, seed=7), "g": values(6, width, seed=8), "o": torch.eye(6, dtype=F64)}
    x = values(8, width, seed=9)
    out = plain.latent_attention(x, w, m, eps)
    i, h = 7, 1

    def unit(t, weight):
        return t / (float((t * t).mean()) + eps) ** 0.5 * weight

    def rotated(t, p):
        a0, a1 = p * 1.0, p * 20.0 ** -0.5
        return [t[0] * math.cos(a0) - t[1] * math.sin(a0), t[1] * math.cos(a0) + t[0] * math.sin(a0),
                t[2] * math.cos(a1) - t[3] * math.sin(a1), t[3] * math.cos(a1) + t[2] * math.sin(a1)]

    q = w["uq"] @ unit(w["dq"] @ x[i], w["dq.norm"])
    q = q[h * 9:h * 9 + 9]
    raised, vs = [], []
    for j in (5, 6, 7):
        down = w["dkv"] @ x[j]
        c = unit(down[:6], w["dkv.norm"])
        key = w["uk"][h * 5:h * 5 + 5] @ c
        score = float(q[:5] @ key) + sum(float(a) * float(b) for a, b in zip(rotated(q[5:], i), rotated(down[6:], j)))
        raised.append(math.exp(0.5 * score))
        vs.append(w["uv"][h * 3:h * 3 + 3] @ c)
    head = sum(r / sum(raised) * v for r, v in zip(raised, vs))
    assert torch.allclose(out[i, h * 3:h * 3 + 3], head * torch.sigmoid(w["g"][h * 3:h * 3 + 3] @ x[i]))


def test_rotation_of_a_score_depends_on_the_distance_alone():
    q, k = values(1, 1, 6, seed=1), values(1, 1, 6, seed=2)
    scores = [float((plain.turn_neighbours(q, 30.0, 6, 9 + s) * plain.turn_neighbours(k, 30.0, 6, 4 + s)).sum()) for s in (0, 5, 100)]
    assert max(scores) - min(scores) < 1e-9
    assert torch.equal(plain.turn_neighbours(q, 30.0, 6, 0), q)


def test_choice_by_corrected_scores_and_weights_without_the_correction():
    logits = torch.tensor([[2.0, 1.0, 0.0, -1.0, 0.5]], dtype=F64)
    s = torch.softmax(logits[0], 0)
    correction = torch.tensor([-1.0, 0.0, 0.0, 0.9, 0.0], dtype=F64)
    chosen, shares = plain.choose(logits, correction, 2)
    assert chosen == [[3, 1]] and torch.allclose(torch.tensor(shares[0], dtype=F64), s[[3, 1]])
    assert sum(shares[0]) < 0.5                                            # not renormalised
    margins = []
    plain.choose(logits, correction, 2, margins)
    assert math.isclose(margins[0], float(s[1] - s[4]))


def test_identity_experts_and_the_shared_expert():
    width = 6
    mlp = configs.experts(4, 0.7, 2, 2, 4, shared=(5, 1.1))
    w = {"router": values(4, width, seed=1), "correction": values(4, seed=2) * 0.1, "shared.gate": values(5, width, seed=3), "shared.up": values(5, width, seed=4),
         "shared.down": values(width, 5, seed=5)}
    for e in range(2):
        w.update({f"e{e}.gate": values(4, width, seed=6 + e), f"e{e}.up": values(4, width, seed=8 + e), f"e{e}.down": values(width, 4, seed=10 + e)})
    x = values(3, width, seed=20)
    s = torch.softmax(x @ w["router"].T, -1)
    out = plain.routed_ff(x, w, mlp)
    want = sum(s[:, e, None] * plain.expert(x, w[f"e{e}.gate"], w[f"e{e}.up"], w[f"e{e}.down"], 0.7) for e in range(2)) + (s[:, 2] + s[:, 3])[:, None] * x
    want = want + plain.expert(x, w["shared.gate"], w["shared.up"], w["shared.down"], 1.1)
    assert torch.allclose(out, want)


def test_expert_clamps_and_the_square_of_relu():
    one = torch.ones(1, 1, dtype=F64)
    x = torch.tensor([[5.0], [-5.0], [0.3]], dtype=F64)
    y = plain.expert(x, one, one, one, 2.0)[:, 0]
    sig = [1 / (1 + math.exp(-1.702 * g)) for g in (2.0, -5.0, 0.3)]
    assert torch.allclose(y, torch.tensor([2.0 * sig[0] * 3.0, -5.0 * sig[1] * -1.0, 0.3 * sig[2] * 1.3], dtype=F64))
    assert torch.allclose(plain.dense_ff(x, one, one)[:, 0], torch.tensor([25.0, 0.0, 0.09], dtype=F64))


def test_causality_and_shared_weights():
    from llm_runtime_study_amd.config import config_from_dict, spec_for
    from llm_runtime_study_amd.models import DecoderModel

    raw = configs.ODD
    names = DecoderModel(spec_for(config_from_dict(raw))).tensors()
    weights = {name: values(*spec.shape, seed=5 + n) / math.sqrt(spec.shape[-1]) + (1.0 if spec.role == "norm" else 0.0) for n, (name, spec) in enumerate(names.items())}
    streams = []
    ids = [17, 4, 17, 200, 17, 3, 9, 17, 5, 17, 17]
    out = plain.forward(weights, raw, ids, streams)
    assert torch.isfinite(out).all() and len(streams) == len(raw["layers"])
    assert torch.allclose(plain.forward(weights, raw, ids[:4]), out[:4])
    assert not torch.allclose(out[0], out[2], atol=1e-3)
