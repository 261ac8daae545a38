"""Mutolix without a GPU: its configuration, the tensors it asks a checkpoint for, what its layers keep between steps, and the plain
implementation's mechanisms against properties that follow from their definitions."""

import copy
import math

import pytest
import torch

from tests import mutolix_configs as configs
from tests.plain import mutolix as plain

F64 = torch.float64


def values(*shape, seed=0, scale=1.0):
    return scale * torch.randn(shape, generator=torch.Generator().manual_seed(seed), dtype=F64)


def test_configuration_reads_back_and_names_its_tensors():
    from llm_runtime_study_amd.config import config_from_dict, spec_for
    from llm_runtime_study_amd.config.mutolix import MutolixConfig
    from llm_runtime_study_amd.models import DecoderModel
    from llm_runtime_study_amd.parts import PagedKVNeed, StateNeed

    for raw in configs.ALL.values():
        config = config_from_dict(raw)
        assert isinstance(config, MutolixConfig) and config.to_json_dict() == raw
        model = DecoderModel(spec_for(config))
        names, width = model.tensors(), raw["width"]
        assert {"embed", "head", "final.norm"} <= set(names) and not any(name.endswith(".weight") for name in names)
        expected = {"embed", "head", "final.norm"}
        first = next((i for i, layer in enumerate(raw["layers"]) if layer["mixer"].get("v_mix")), None)
        for index, layer in enumerate(raw["layers"]):
            m, p = layer["mixer"], f"l{index}."
            shapes = {"norm1": (width,), "norm1b": (width,), "ls1": (width,), "rg1": (width, width), "rg1.b": (width,)}
            if layer["type"] == "mlstm":
                h, d, e = m["heads"], m["dim"], m["vdim"]
                shapes.update({"mix.q": (h * d, width), "mix.k": (h * d, width), "mix.v": (h * e, width), "mix.g": (h * e, width), "mix.o": (width, h * e),
                               "mix.norm": (h * e,), "mix.i": (h, width), "mix.i.b": (h,), "mix.f": (h, width), "mix.f.b": (h,)})
            else:
                h, g, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
                shapes.update({"mix.q": (h * d, width), "mix.k": (g * d, width), "mix.v": (g * e, width), "mix.q.b": (h * d,), "mix.k.b": (g * d,),
                               "mix.v.b": (g * e,), "mix.q.norm": (h * d,), "mix.k.norm": (g * d,), "mix.r1": (h,), "mix.r2": (h,), "mix.o": (width, h * e)})
                if m["v_mix"]:
                    shapes["mix.vmix"] = ()
                    assert names[p + "mix.vmix"].optional == (index == first)
            if layer["mlp"] is not None:
                ff = layer["mlp"]["ff"]
                shapes.update({"norm2": (width,), "norm2b": (width,), "ls2": (width,), "rg2": (width, width), "rg2.b": (width,),
                               "mlp.up": (ff, width), "mlp.down": (width, ff), "mlp.act": (2,)})
            for name, shape in shapes.items():
                assert tuple(names[p + name].shape) == shape, p + name
            expected |= {p + name for name in shapes}
        assert set(names) == expected
        for layer, need in zip(raw["layers"], model.cache_needs()):
            m = layer["mixer"]
            if layer["type"] == "mlstm":
                rows = 4 if m["dim"] <= 64 else 8 if m["dim"] <= 128 else 16
                assert isinstance(need, StateNeed) and need.dtype == torch.float32
                assert need.shape == (m["heads"] * (rows * 16 * (m["vdim"] + 1) + 1),)
            else:
                assert isinstance(need, PagedKVNeed) and need.window is None and (need.num_kv_heads, need.head_dim) == (m["kv_heads"], m["dim"])
                assert (need.value_dim or need.head_dim) == m["vdim"]


def test_what_the_file_leaves_out_does_not_exist():
    from llm_runtime_study_amd.config import config_from_dict, spec_for

    raw = copy.deepcopy(configs.ODD)
    del raw["embedding"], raw["layers"][0]["mixer"]["q_temp"], raw["layers"][0]["mixer"]["v_mix"], raw["layers"][1]["mlp"]
    config = config_from_dict(raw)
    assert config.embedding_scale == 1.0 and config.layers[0].mixer.temp_every is None and not config.layers[0].mixer.v_mix
    assert config.first_mixing_layer() == 4 and config.layers[1].ff is None
    layers = spec_for(config).layers
    assert layers[0].params["mixer"].params["query_temperature"] is None and layers[0].params["mixer"].params["value_mix"] is None
    assert layers[4].params["mixer"].params["value_mix"] == "first"


def refused(change):
    from llm_runtime_study_amd.config import config_from_dict
    from llm_runtime_study_amd.errors import ConfigError

    raw = copy.deepcopy(configs.ODD)
    change(raw)
    with pytest.raises(ConfigError) as caught:
        config_from_dict(raw)
    return str(caught.value)


def test_refusals_name_the_layer():
    assert "layer 2" in refused(lambda raw: raw["layers"][2].update(type="mamba"))
    assert "heads" in refused(lambda raw: raw["layers"][0]["mixer"].update(heads=5))
    assert "layer 1" in refused(lambda raw: raw["layers"][1]["mixer"].pop("gate_cap"))
    assert "gate_cap" in refused(lambda raw: raw["layers"][1]["mixer"].update(gate_cap=0.0))
    assert "every" in refused(lambda raw: raw["layers"][0]["mixer"]["q_temp"].update(every=0))
    assert "coef" in refused(lambda raw: raw["layers"][0]["mixer"]["q_temp"].pop("coef"))
    assert "scale" in refused(lambda raw: raw["layers"][0]["mixer"].pop("scale"))
    assert "v_mix" in refused(lambda raw: raw["layers"][4]["mixer"].update(vdim=21))
    assert "v_mix" in refused(lambda raw: raw["layers"][4]["mixer"].update(v_mix=1))
    assert "kind" in refused(lambda raw: raw["layers"][0]["mlp"].update(kind="moe"))
    assert "mlp" in refused(lambda raw: raw["layers"][0].update(mlp=4))
    assert "eps" in refused(lambda raw: raw["norm"].update(eps=0.0))
    assert "layers" in refused(lambda raw: raw.update(layers=[]))


def test_parts_refuse_what_they_cannot_run():
    from llm_runtime_study_amd.parts import PartSpec, create

    sizes = {"hidden_size": 32, "num_heads": 2, "num_kv_heads": 1, "head_dim": 16}
    for bad in ({"value_mix": "some"}, {"query_temperature": (0.5, 0)}, {"query_temperature": (0.5, 4), "unit_norm_after_rotation": True},
                {"value_mix": "later", "unit_norm_after_rotation": True}, {"distance_bias": True, "kv_shared": True}):
        with pytest.raises(ValueError):
            create("mixer", PartSpec("gqa_attention", dict(sizes, **bad)))
    memory = {"hidden_size": 32, "num_heads": 2, "head_dim": 16, "value_dim": 8, "gate_cap": 5.0, "norm_eps": 1e-6}
    for bad in ({"head_dim": 257}, {"gate_cap": 0.0}, {"norm_eps": 0.0}, {"value_dim": 0}):
        with pytest.raises(ValueError):
            create("mixer", PartSpec("mlstm", dict(memory, **bad)))
    norm, mixer = PartSpec("rmsnorm", {"size": 32, "eps": 1e-6}), PartSpec("mlstm", memory)
    block = {"mixer": mixer, "mixer_norm": norm, "mixer_out_norm": norm}
    assert set(create("block", PartSpec("sandwich", block)).tensors()) == {f"mixer.{n}" for n in create("mixer", mixer).tensors()} | {"mixer_norm.weight", "mixer_out_norm.weight"}
    with pytest.raises(ValueError):                                       # a feed-forward without its norms
        create("block", PartSpec("sandwich", dict(block, feed_forward=PartSpec("dense_mlp", {"hidden_size": 32, "intermediate_size": 8}))))
    with pytest.raises(ValueError):                                       # a layer norm cannot stand on either side
        create("block", PartSpec("sandwich", dict(block, mixer_norm=PartSpec("layernorm", {"size": 32, "eps": 1e-6}))))
    with pytest.raises(ValueError):
        create("feed_forward", PartSpec("dense_mlp", {"hidden_size": 32, "intermediate_size": 8, "activation": "elu"}))


def test_a_matrix_carried_behind_a_parts_first_product():
    from llm_runtime_study_amd.parts import PartSpec, create

    part = create("feed_forward", PartSpec("dense_mlp", {"hidden_size": 24, "intermediate_size": 10, "activation": "xielu"}))
    w = {"up_proj.weight": values(10, 24, seed=1), "down_proj.weight": values(24, 10, seed=2), "act": values(2, seed=3)}
    extra = values(24, 24, seed=4)
    part.carry(extra)
    part.bind(w, torch.float32)
    assert part.up.shape == (48, 24)                                      # 10 rows and 6 of zeros, 24 rows and 8 of zeros
    torch.testing.assert_close(part.up[16:40], extra.float())
    assert part.up[10:16].abs().max() == 0 and part.up[40:].abs().max() == 0

    class Ctx:
        memo: dict = {}

    ctx = Ctx()
    part.hand_out_carried(ctx, torch.arange(96.0).view(2, 48))
    assert torch.equal(ctx.memo["carried_rows"], torch.arange(96.0).view(2, 48)[:, 16:40])
    part.bind(w, torch.float32)                                           # bound again without it: nothing is carried
    ctx.memo.clear()
    part.hand_out_carried(ctx, torch.zeros(2, 10))
    assert part.up.shape == (10, 24) and not ctx.memo


# ------------------------------------------------------------------------------------- the plain mechanisms
def test_the_running_maximum_changes_nothing_but_the_scale():
    """S over exp(-m) is the plain sum of exp(i) k v^T, decayed by sigmoid(f): written out without any maximum (in float64, gates small)."""
    n, d, e = 9, 5, 4
    q, k, v = values(n, d, seed=1), values(n, d, seed=2), values(n, e, seed=3)
    i, f = values(n, seed=4), -plain.softplus(values(n, seed=5))
    record = []
    out = plain.matrix_memory(q, k, v, i, f, record)
    for t in range(n):
        S, norm = torch.zeros(d, e, dtype=F64), torch.zeros(d, dtype=F64)
        for s in range(t + 1):
            weight = torch.exp(f[s + 1:t + 1].sum() + i[s])
            S, norm = S + weight * torch.outer(k[s], v[s]), norm + weight * k[s]
        m = record[t][2]
        assert torch.allclose(record[t][0], S * math.exp(-m)) and torch.allclose(record[t][1], norm * math.exp(-m))
        want = (S.T @ q[t]) / (max(abs(float(norm @ q[t])), 1.0) + 1e-6 * math.exp(m))     # exp(-m) over exp(-m) is one
        assert torch.allclose(out[t], want)
    assert max(m for _, _, m in record) == max(record[t][2] for t in range(n))


def test_the_maximum_starts_at_zero():
    """The first token of a sequence with an input gate far below zero: m stays at f, close to zero, so the floor exp(-m) is about
    one and the read-out is small; a maximum that started at minus infinity would give v scaled by q . k / |q . k|."""
    q, k, v = values(1, 4, seed=1), values(1, 4, seed=2), values(1, 3, seed=3)
    out = plain.matrix_memory(q, k, v, torch.tensor([-6.0], dtype=F64), torch.tensor([-0.01], dtype=F64))
    assert torch.allclose(out[0], math.exp(-6.0) * (q[0] @ k[0]) * v[0] / (math.exp(0.0) + 1e-6 * math.exp(-0.01)), rtol=1e-3)
    assert out.abs().max() < 0.1 * v.abs().max()


def test_gates_are_capped_on_a_log_scale():
    w = {"i": 100.0 * torch.ones(1, 1, dtype=F64), "i.b": torch.zeros(1, dtype=F64), "f": 100.0 * torch.ones(1, 1, dtype=F64), "f.b": torch.zeros(1, dtype=F64)}
    i, f = plain.log_gates(torch.tensor([[5.0], [-5.0], [0.0]], dtype=F64), w, 3.0)
    assert torch.allclose(i[:, 0], torch.tensor([3.0, -3.0, 0.0], dtype=F64))
    assert torch.allclose(f[:, 0], torch.log(torch.sigmoid(torch.tensor([3.0, -3.0, 0.0], dtype=F64))))


def attention_weights(m, width=24, seed=1):
    h, g, d, e = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    return {"q": values(h * d, width, seed=seed), "k": values(g * d, width, seed=seed + 1), "v": values(g * e, width, seed=seed + 2),
            "q.b": values(h * d, seed=seed + 3), "k.b": values(g * d, seed=seed + 4), "v.b": values(g * e, seed=seed + 5),
            "q.norm": 1 + 0.1 * values(h * d, seed=seed + 6), "k.norm": 1 + 0.1 * values(g * d, seed=seed + 7),
            "r1": values(h, seed=seed + 8).abs(), "r2": values(h, seed=seed + 9).abs(), "vmix": torch.tensor(0.3, dtype=F64), "o": torch.eye(h * e, dtype=F64)}


def test_temperature_steps_where_it_should():
    t = plain.temperature(torch.arange(12), {"coef": 0.5, "every": 4}, F64)
    assert t[:3].tolist() == [1.0, 1.0, 1.0]                              # (p + 1) / 4 rounds down to zero
    assert torch.allclose(t[3:7], torch.full((4,), 1 + 0.5 * math.log(2.0), dtype=F64))
    assert torch.allclose(t[7:11], torch.full((4,), 1 + 0.5 * math.log(3.0), dtype=F64)) and t[11] > t[10]


def test_attention_against_its_definition_at_one_place():
    m = {"heads": 4, "kv_heads": 2, "dim": 6, "vdim": 5, "scale": 0.4, "q_temp": {"coef": 0.5, "every": 3}}
    w = attention_weights(m)
    x = values(8, 24, seed=9)
    seen = []
    out = plain.attention(x, w, m, 1e-5, [], weights_out=seen)
    q = plain.rms_norm(x @ w["q"].T + w["q.b"], w["q.norm"], 1e-5)        # over all heads at once: a head alone is not of unit size
    assert abs(float((q[0] / w["q.norm"]).pow(2).mean()) - 1) < 1e-4 and abs(float((q[0, :6] / w["q.norm"][:6]).pow(2).mean()) - 1) > 1e-2
    k = plain.rms_norm(x @ w["k"].T + w["k.b"], w["k.norm"], 1e-5)
    v = x @ w["v"].T + w["v.b"]
    i, h, g = 7, 3, 1
    heat = 1 + 0.5 * math.log((i + 1) // 3 + 1)
    e = [math.exp(float(heat * (q[i, h * 6:h * 6 + 6] @ k[j, g * 6:g * 6 + 6]) * 0.4 - w["r1"][h] * math.log(1 + float(w["r2"][h]) * (i - j)))) for j in range(i + 1)]
    want = sum(e[j] / (1 + sum(e)) * v[j, g * 5:g * 5 + 5] for j in range(i + 1))
    assert torch.allclose(out[i, h * 5:h * 5 + 5], want)
    for _, _, weights in seen:
        assert 0 < float(weights.sum()) < 1                               # the rest is the sink's share


def test_values_are_mixed_with_the_first_mixing_layers():
    m = {"heads": 2, "kv_heads": 1, "dim": 4, "vdim": 3, "scale": 0.4, "v_mix": True}
    a, b = attention_weights(m, seed=1), attention_weights(m, seed=30)
    x, y = values(5, 24, seed=3), values(5, 24, seed=4)
    shared = []
    first = plain.attention(x, a, m, 1e-5, shared)
    assert torch.allclose(first, plain.attention(x, dict(a, vmix=torch.tensor(0.9, dtype=F64)), m, 1e-5, []))       # its own lambda is unused
    assert len(shared) == 1 and torch.allclose(shared[0].reshape(5, 3), x @ a["v"].T + a["v.b"])
    mixed = plain.attention(y, b, m, 1e-5, shared)
    only_first = plain.attention(y, dict(b, vmix=torch.tensor(1.0, dtype=F64)), m, 1e-5, shared)
    only_own = plain.attention(y, b, dict(m, v_mix=False), 1e-5, shared)
    assert torch.allclose(mixed, 0.7 * only_own + 0.3 * only_first) and len(shared) == 1     # attention is linear in the values


def test_xielu_and_its_slope_on_both_sides():
    p, q = torch.tensor(0.3, dtype=F64), torch.tensor(-0.8, dtype=F64)
    z = torch.tensor([-3.0, -1e-7, 0.0, 1e-7, 2.0], dtype=F64)
    a, b = math.log1p(math.exp(0.3)), 0.5 + math.log1p(math.exp(-0.8))
    got = plain.xielu(z, p, q)
    assert torch.allclose(got[4], torch.tensor(a * 4 + 1.0, dtype=F64))
    assert torch.allclose(got[0], torch.tensor(b * (math.exp(-3.0) - 1 + 3.0) - 1.5, dtype=F64))
    assert got[2] == 0 and torch.allclose(got[[1, 3]] / z[[1, 3]], torch.full((2,), 0.5, dtype=F64), atol=1e-6)


def test_a_layers_update_gates_then_normalises_then_scales():
    width, eps = 6, 1e-6
    w = {"norm1": 1 + values(width, seed=1) * 0.1, "norm1b": 1 + values(width, seed=2) * 0.1, "ls1": values(width, seed=3), "rg1": values(width, width, seed=4),
         "rg1.b": values(width, seed=5)}
    x = values(3, width, seed=6)
    matrix = values(width, width, seed=7)
    got = plain.update(x, w, 1, lambda u: u @ matrix.T, eps)
    u = x / x.pow(2).mean(-1, keepdim=True).add(eps).sqrt() * w["norm1"]
    y = (u @ matrix.T) * torch.sigmoid(u @ w["rg1"].T + w["rg1.b"])
    assert torch.allclose(got, x + w["ls1"] * (y / y.pow(2).mean(-1, keepdim=True).add(eps).sqrt() * w["norm1b"]))
    assert torch.allclose(plain.update(x, w, 1, lambda u: 5.0 * u @ matrix.T, eps), got, atol=1e-5)       # the second norm takes the length out


def test_first_tokens_and_causality():
    from llm_runtime_study_amd.config import config_from_dict, spec_for
    from llm_runtime_study_amd.models import DecoderModel

    raw = configs.ODD
    names = DecoderModel(spec_for(config_from_dict(raw))).tensors()
    weights = {name: configs.lively(name, values(*spec.shape, seed=5 + n) / math.sqrt(spec.shape[-1] if spec.shape else 1)).to(F64)
               for n, (name, spec) in enumerate(names.items())}
    weights = {name: t.abs() if name.endswith((".r1", ".r2")) else t for name, t in weights.items()}
    streams = []
    out = plain.forward(weights, raw, [17, 4, 17, 200, 17], streams)
    assert torch.isfinite(out).all() and len(streams) == len(raw["layers"])
    assert torch.allclose(plain.forward(weights, raw, [17, 4])[:2], out[:2])            # causal
    assert not torch.allclose(out[0], out[2], atol=1e-3)                                 # one token at two places: what came before tells them apart
