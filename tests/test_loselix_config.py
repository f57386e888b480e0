"""Loselix without a GPU: configuration, plan (loops, cache numbers, what enters a pass), contract, and pins of the plain
implementation the GPU tests compare with."""

import copy
import math

import pytest
import torch

import burn_transformers_amd as bt
import plain_loselix as plain
from burn_transformers_amd.config import ConfigError, LoselixConfig, resolve_family
from burn_transformers_amd.weights.contract import WeightError
from burn_transformers_amd.weights.loader import store_from_tensors
from loselix_helpers import ASKS, BASIC, CONFIGS, HOLDS, ODD, planted, prompts_for, random_config, tolerance, weights_for

F64 = torch.float64


def test_configuration_round_trip_and_family():
    for config, _ in CONFIGS.values():
        typed = LoselixConfig.from_dict(config)
        assert LoselixConfig.from_dict(typed.to_dict()) == typed and typed.to_dict() == config
        assert resolve_family(config).name == "loselix"
    for seed in range(30):
        data = random_config(seed)
        assert LoselixConfig.from_dict(data).to_dict() == data
    typed = LoselixConfig.from_dict(BASIC)
    assert [layer.type for layer in typed.layers] == ["attention", "attention_2", "attention_3", "attention", "attention_2"]
    assert typed.layers[0].mixer.rot.dims == 8 and typed.layers[0].mixer.softcap == 30.0 and typed.layers[3].mixer.diff == 0.7
    assert typed.layers[2].mixer.temp_every == 16 and typed.layers[2].mixer.temp_coef == 0.3
    assert typed.runs() == [(0, False), (1, False), (2, False), (3, False), (1, True), (2, False), (3, False), (4, False)]
    odd = LoselixConfig.from_dict(ODD)
    assert odd.runs() == [(0, False), (1, False), (0, True), (1, False), (0, True), (1, False), (2, False), (3, False), (4, False), (5, False)]
    assert odd.layers[2].mlp is None and odd.layers[3].mixer.rot is None and odd.layers[3].mixer.softcap == 0.0
    assert odd.layers[5].mixer.temp_every == 0
    bare = {k: v for k, v in BASIC.items() if k != "loop"}
    assert LoselixConfig.from_dict(bare).runs() == [(i, False) for i in range(5)]


@pytest.mark.parametrize("path,value,field", [
    (("width",), None, "width"), (("norm", "eps"), 0.0, "norm.eps"), (("layers", 0, "type"), "conv", "layers[0].type"),
    (("layers", 0, "mixer", "dim"), 0, "layers[0].mixer.dim"), (("layers", 0, "mixer", "kv_heads"), 3, "layers[0].mixer.kv_heads"),
    (("layers", 0, "mixer", "rot", "dims"), 18, "layers[0].mixer.rot.dims"), (("layers", 0, "mixer", "rot", "base"), -1.0, "layers[0].mixer.rot.base"),
    (("layers", 0, "mixer", "softcap"), -2.0, "layers[0].mixer.softcap"), (("layers", 0, "mixer", "diff"), None, "layers[0].mixer.diff"),
    (("layers", 1, "mixer", "scale"), None, "layers[1].mixer.scale"), (("layers", 2, "mixer", "vdim"), 16, "layers[2].mixer.vdim"),
    (("layers", 2, "mixer", "q_temp", "every"), -1, "layers[2].mixer.q_temp.every"),
    (("layers", 2, "mixer", "q_temp", "coef"), None, "layers[2].mixer.q_temp.coef"),
    (("layers", 0, "mlp", "kind"), "moe", "layers[0].mlp.kind"), (("layers", 0, "mlp", "ff"), 0, "layers[0].mlp.ff"),
    (("loop", "stop"), 7, "loop.stop"), (("loop", "times"), 0, "loop.times")])
def test_configuration_errors_name_the_field(path, value, field):
    config = copy.deepcopy(BASIC)
    at = config
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError) as error:
        LoselixConfig.from_dict(config)
    assert error.value.field == field


def test_plan_names_the_parts_their_constants_and_a_cache_entry_for_every_run():
    family = resolve_family(BASIC)
    plan = family.plan(LoselixConfig.from_dict(BASIC))
    assert [layer.block for layer in plan.layers] == ["parallel"] * 5 + ["transform"]
    assert [(e.layer, e.cache) for e in plan.schedule] == [(0, 0), (1, 1), (2, 2), (3, 3), (5, None), (1, 4), (2, 5), (3, 6), (4, 7)]
    assert plan.layers[5].parts["transform"].kind == "add_origin" and plan.embedding.params["keep_origin"]
    first, second, third = (layer.parts for layer in plan.layers[:3])
    a = first["mixer"]
    assert a.kind == "differential_attention" and (a.params["softcap"], a.params["diff"], a.params["rot_dims"]) == (30.0, 0.4, 8)
    assert a.tensors["lambda_q1"] == "l0.mix.lq1" and first["norm"].tensors["weight"] == "l0.norm1" and not a.params["head_norm"]
    b = second["mixer"]
    assert b.kind == "rotary_attention" and b.params["gate"] == "head" and b.tensors["gate_weight"] == "l1.mix.g" and "weights" not in b.params
    c = third["mixer"]
    assert (c.params["values"], c.params["weights"], c.params["gate"], c.params["norm_span"]) == ("keys", "sigmoid", "channel", "whole")
    assert c.params["temperature"] == {"coef": 0.3, "every": 16} and "rot_dims" not in c.params and "v_weight" not in c.tensors
    assert c.tensors["score_bias"] == "l2.mix.pb" and first["ff"].params["activation"] == "squared_relu"
    single = family.plan(LoselixConfig.from_dict(dict(BASIC, loop={"start": 0, "stop": 2, "times": 1})))
    assert [e.cache for e in single.schedule] == list(range(5)) and not single.embedding.params["keep_origin"]
    odd = family.plan(LoselixConfig.from_dict(ODD))
    assert [e.cache for e in odd.schedule if e.cache is not None] == list(range(10)) and "ff" not in odd.layers[2].parts
    assert sum(e.cache is None for e in odd.schedule) == 2


def test_contract_and_random_weights_agree():
    for config, seed in CONFIGS.values():
        family = resolve_family(config)
        typed, tensors = bt.random_tensors(config, seed)
        contract = family.contract(typed)
        assert {spec.name for spec in contract.tensors} == set(tensors)
        assert all(tuple(tensors[spec.name].shape) == tuple(spec.shape) for spec in contract.tensors)
    typed = LoselixConfig.from_dict(BASIC)
    specs = {spec.name: spec for spec in resolve_family(BASIC).contract(typed).tensors}
    assert specs["l0.mix.q"].shape == (128, 64) and specs["l0.mix.k"].shape == (64, 64) and specs["l0.mix.lk2"].shape == (16,)
    assert specs["l1.mix.g"].shape == (4, 64) and specs["l2.mix.g"].shape == (128, 64) and specs["l2.mix.pb"].shape == (4,)
    assert specs["l2.mix.k.norm"].shape == (64,) and "l2.mix.v" not in specs
    _, tensors = bt.random_tensors(BASIC, 1)
    tensors["l1.mix.g"] = tensors["l1.mix.g"][:3]
    with pytest.raises(WeightError):
        store_from_tensors(tensors, resolve_family(BASIC).contract(typed), torch.float32, "cpu")


def test_plain_mechanisms_are_pinned():
    """The plain implementation on inputs whose answers are known by hand."""
    assert torch.equal(plain.squared_relu(torch.tensor([-2.0, 0.0, 3.0])), torch.tensor([0.0, 0.0, 9.0]))
    assert torch.allclose(plain.unit_rms(torch.tensor([[3.0, 4.0]], dtype=F64), 0.0), torch.tensor([[3.0, 4.0]], dtype=F64) / math.sqrt(12.5))
    # channel i turns with channel i + dims / 2; channels behind dims stay; a quarter turn
    v = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=F64)
    turned = plain.turn(v, torch.tensor([math.pi / 2.0]), {"dims": 4, "base": 1.0})
    assert torch.allclose(turned, torch.tensor([[[-3.0, -4.0, 1.0, 2.0, 5.0]]], dtype=F64))
    # a small score passes the cap, a large one stops at it
    assert float(plain.softcap(torch.tensor(0.01, dtype=F64), 30.0)) == pytest.approx(0.01, rel=1e-6)
    assert float(plain.softcap(torch.tensor(900.0, dtype=F64), 30.0)) == pytest.approx(30.0)
    # sigmoid weights: a key that is not seen has none, the others need not add up to one
    seen = torch.tensor([[True, True, False]])
    got = plain.sigmoid_over(torch.tensor([[1.0, -1.0, 7.0]], dtype=F64), seen, torch.tensor(1.0, dtype=F64))
    assert torch.allclose(got, torch.tensor([[1.0 / (1.0 + math.exp(-2.0)), 0.5, 0.0]], dtype=F64))
    # the temperature steps up where p + 1 reaches a multiple
    steps = plain.temperature(torch.tensor([0, 6, 7, 14, 15]), 0.5, 8)
    assert torch.allclose(steps, 1.0 + 0.5 * torch.log(torch.tensor([1.0, 1.0, 2.0, 2.0, 3.0], dtype=F64)))
    # lambda
    w = {"m.lq1": torch.tensor([1.0, 2.0]), "m.lk1": torch.tensor([0.5, 0.25]), "m.lq2": torch.tensor([2.0, 0.0]), "m.lk2": torch.tensor([-1.0, 3.0])}
    assert plain.difference_weight(w, "m.", 0.3) == pytest.approx(math.e - math.exp(-2.0) + 0.3)


def test_plain_differential_attention_of_one_token():
    """One key: both maps give its value, so the head's row is its direction times (1 - diff), whatever lambda."""
    config, weights = CONFIGS["differential"][0], {k: v.double() for k, v in weights_for("differential").items()}
    sizes = config["layers"][0]["mixer"]
    h = torch.randn(1, 64, generator=torch.Generator().manual_seed(0), dtype=F64)
    v = (h @ weights["l0.mix.v"].T).view(2, 64)
    lam = plain.difference_weight(weights, "l0.mix.", sizes["diff"])
    row = plain.unit_rms(v * (1.0 - lam), 1e-5) * (1.0 - sizes["diff"])
    want = row.repeat_interleave(2, 0).reshape(1, -1) @ weights["l0.mix.o"].T
    assert torch.allclose(plain.differential_attention(h, weights, "l0.mix.", sizes, 1e-5), want, rtol=1e-12, atol=1e-12)


def test_plain_passes_start_from_the_embedding_again():
    config, weights = CONFIGS["basic"][0], weights_for("basic")
    ids = prompts_for("basic", [9])[0]
    looped, straight = [], []
    plain.forward(ids, weights, config, streams=looped)
    plain.forward(ids, weights, dict(config, loop=None), streams=straight)
    assert len(looped) == 8 and len(straight) == 5
    for run in range(4):
        assert torch.equal(looped[run], straight[run])
    # the second pass begins with x + x0
    w = {k: v.to(F64) for k, v in weights.items()}
    x = looped[3] + w["embed"][torch.tensor(ids)]
    h = plain.unit_rms(x, 1e-5) * w["l1.norm1"]
    x = x + plain.head_gated_attention(h, w, "l1.mix.", config["layers"][1]["mixer"], 1e-5) + plain.feed_forward(h, w, "l1.mlp.")
    assert torch.allclose(x, looped[4], rtol=1e-12, atol=1e-12)


@pytest.mark.parametrize("kind", ["differential", "head_gated", "sigmoid"])
def test_the_planted_key_moves_the_logits(kind):
    """The premise of the far-key tests: with the token that holds the key at the start and the one that asks at the end
    of 300 tokens, another token in the first place moves the last logits by far more than any bound on rounding."""
    config, weights = planted(kind)
    ids = torch.randint(10, config["vocab"], (300,), generator=torch.Generator().manual_seed(1)).tolist()
    ids[0], ids[-1] = HOLDS, ASKS
    base = plain.forward(ids, weights, config)[-1]
    moved = plain.forward([11] + ids[1:], weights, config)[-1]
    assert float((base - moved).abs().max()) > 4 * tolerance("bfloat16", base)
