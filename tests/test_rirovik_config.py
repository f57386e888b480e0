"""Rirovik without a GPU: configuration, plan (borrowed latents), contract, what a shared cache entry has to keep, the
cache ledger with kept first positions, and pins of the plain implementation the GPU tests compare with."""

import copy
import math

import pytest
import torch

import burn_transformers_amd as bt
import plain_rirovik as plain
from burn_transformers_amd.cache.ledger import BLOCK, RELEASED, CacheLedger
from burn_transformers_amd.cache.storage import KVSpec
from burn_transformers_amd.config import ConfigError, RirovikConfig, resolve_family
from burn_transformers_amd.engine.plan import ScheduleEntry
from burn_transformers_amd.parts.attention import keys_in_reach
from burn_transformers_amd.weights.contract import WeightError
from burn_transformers_amd.weights.loader import store_from_tensors
from rirovik_helpers import BASIC, CONFIGS, ODD, config_for, prompts_for, random_config, weights_for

F64 = torch.float64


def test_configuration_round_trip_and_family():
    for name, (config, _) in CONFIGS.items():
        for data in (config, config_for(name, "bfloat16")):
            typed = RirovikConfig.from_dict(data)
            assert RirovikConfig.from_dict(typed.to_dict()) == typed and typed.to_dict() == data
            assert resolve_family(data).name == "rirovik"
    for seed in range(40):
        data = random_config(seed)
        assert RirovikConfig.from_dict(data).to_dict() == data
    typed = RirovikConfig.from_dict(BASIC)
    assert [layer.type for layer in typed.layers] == ["attention", "latent_attention", "latent_attention", "latent_attention_2", "latent_attention_2"]
    assert (typed.layers[0].mixer.mask.size, typed.layers[0].mixer.mask.keep_first) == (24, 5)
    assert typed.layers[1].mixer.mask.keep_first == 0 and typed.layers[3].mixer.mask is None
    assert [getattr(layer.mixer, "kv_from", None) for layer in typed.layers] == [None, None, 1, None, 1]
    assert typed.layers[1].mixer.rot_base == 2000.0 and typed.layers[1].mlp.shared_ff == 0 and typed.layers[0].mlp.shared_ff == 40
    odd = RirovikConfig.from_dict(ODD)
    assert odd.layers[2].mlp is None and odd.layers[2].mixer.rot_dim == 0 and odd.layers[4].mixer.mask is None


@pytest.mark.parametrize("path,value,field", [
    (("width",), None, "width"), (("norm", "eps"), 0.0, "norm.eps"), (("embedding", "scale"), "x", "embedding.scale"),
    (("layers", 0, "type"), "conv", "layers[0].type"), (("layers", 0, "mixer", "dim"), 0, "layers[0].mixer.dim"),
    (("layers", 0, "mixer", "kv_heads"), 3, "layers[0].mixer.kv_heads"), (("layers", 0, "mixer", "mask", "size"), 0, "layers[0].mixer.mask.size"),
    (("layers", 0, "mixer", "mask", "size"), None, "layers[0].mixer.mask.size"),
    (("layers", 0, "mixer", "mask", "keep_first"), -1, "layers[0].mixer.mask.keep_first"), (("layers", 0, "mixer", "scale"), None, "layers[0].mixer.scale"),
    (("layers", 1, "mixer", "rot_dim"), 6, "layers[1].mixer.rot.dims"), (("layers", 1, "mixer", "kv_rank"), None, "layers[1].mixer.kv_rank"),
    (("layers", 1, "mixer", "rot"), None, "layers[1].mixer.rot"), (("layers", 2, "mixer", "kv_from"), 2, "layers[2].mixer.kv_from"),
    (("layers", 2, "mixer", "kv_from"), 0, "layers[2].mixer.kv_from"), (("layers", 4, "mixer", "kv_from"), 2, "layers[4].mixer.kv_from"),
    (("layers", 2, "mixer", "kv_from"), -1, "layers[2].mixer.kv_from"), (("layers", 2, "mixer", "kv_rank"), 48, "layers[2].mixer.kv_rank"),
    (("layers", 2, "mixer", "rot", "base"), 3.0, "layers[2].mixer.rot.base"),
    (("layers", 1, "mlp", "router", "top"), 9, "layers[1].mlp.router.top"), (("layers", 1, "mlp", "expert", "ff"), 0, "layers[1].mlp.expert.ff"),
    (("layers", 0, "mlp", "kind"), "dense", "layers[0].mlp.kind")])
def test_configuration_errors_name_the_field(path, value, field):
    config = copy.deepcopy(BASIC)
    at = config
    for key in path[:-1]:
        at = at[key]
    at[path[-1]] = value
    with pytest.raises(ConfigError) as error:
        RirovikConfig.from_dict(config)
    assert error.value.field == field


def test_plan_names_the_parts_their_constants_and_whose_cache_entry_a_run_reads():
    family = resolve_family(BASIC)
    plan = family.plan(RirovikConfig.from_dict(BASIC))
    assert [layer.block for layer in plan.layers] == ["sandwich_norm"] * 5
    assert plan.schedule == [ScheduleEntry(0, 0, True), ScheduleEntry(1, 1, True), ScheduleEntry(2, 1, False), ScheduleEntry(3, 2, True),
                             ScheduleEntry(4, 1, False)]
    parts = [layer.parts for layer in plan.layers]
    for index, p in enumerate(parts):
        for role, leaf in (("mixer_norm", "norm1"), ("mixer_post", "norm1b"), ("ff_norm", "norm2"), ("ff_post", "norm2b")):
            assert p[role].kind == "rms_norm" and p[role].params["offset"] == 1.0 and p[role].tensors["weight"] == f"l{index}.{leaf}"
    a = parts[0]["mixer"]
    assert a.kind == "rotary_attention" and (a.params["window"], a.params["keep"], a.params["rot_dims"]) == (24, 5, 0)
    assert (a.params["head_norm"], a.params["norm_scale"], a.params["gate"]) == (True, False, "channel")
    assert a.tensors["q_bias"] == "l0.mix.q.b" and a.tensors["gate_weight"] == "l0.mix.g" and "q_norm" not in a.tensors
    m = parts[1]["mixer"]
    assert m.kind == "latent_attention" and (m.params["window"], m.params["keep"], m.params["gate"], m.params["borrows"]) == (20, 0, "head", False)
    assert m.params["rot_pairing"] == "neighbours" and m.tensors["gate"] == "l1.mix.g" and m.tensors["down_kv"] == "l1.mix.dkv"
    b = parts[2]["mixer"]
    assert b.params["borrows"] and "down_kv" not in b.tensors and "kv_norm" not in b.tensors and b.tensors["up_k"] == "l2.mix.uk"
    assert "gate" not in parts[3]["mixer"].tensors and parts[3]["mixer"].params["window"] == 0
    e = parts[0]["ff"]
    assert (e.params["score"], e.params["normalize"], e.params["unit"], e.params["shared_ff"], e.params["top"]) == ("chosen", True, "squared_relu", 40, 3)
    assert e.tensors["router_bias"] == "l0.mlp.router.b" and "shared_up" not in parts[1]["ff"].tensors
    assert plan.embedding.params["scale"] == 2.0 and plan.readout.tensors["weight"] == "head"
    late = family.plan(RirovikConfig.from_dict(ODD)).layers
    assert set(late[2].parts) == {"mixer_norm", "mixer", "mixer_post"}


def test_contract_and_random_weights_agree():
    for config, seed in CONFIGS.values():
        family = resolve_family(config)
        typed, tensors = bt.random_tensors(config, seed)
        contract = family.contract(typed)
        assert {spec.name for spec in contract.tensors} == set(tensors)
        assert all(tuple(tensors[spec.name].shape) == tuple(spec.shape) for spec in contract.tensors)
    typed = RirovikConfig.from_dict(BASIC)
    specs = {spec.name: spec for spec in resolve_family(BASIC).contract(typed).tensors}
    assert specs["l0.mix.q.b"].shape == (64,) and specs["l0.mix.g"].shape == (128, 64) and specs["l0.mix.o"].shape == (64, 128)
    assert specs["l1.mix.g"].shape == (3, 64) and specs["l1.mix.dkv"].shape == (40, 64) and specs["l1.mix.uq"].shape == (72, 40)
    assert specs["l2.mix.uk"].shape == (48, 32) and "l2.mix.dkv" not in specs and "l2.mix.dkv.norm" not in specs and "l3.mix.g" not in specs
    assert specs["l0.mlp.router"].layout == "vector" and specs["l0.mlp.router.b"].shape == (6,) and "l1.mlp.shared.up" not in specs
    _, tensors = bt.random_tensors(BASIC, 1)
    tensors["l2.mix.dkv"] = torch.zeros(40, 64)
    with pytest.raises(WeightError):
        store_from_tensors(tensors, resolve_family(BASIC).contract(typed), torch.float32, "cpu")


def test_what_an_entry_keeps_that_several_mixers_read():
    windowed, wider, whole = KVSpec(1, 32, 20), KVSpec(1, 32, 33, keep=4), KVSpec(1, 32)
    assert windowed.joined(windowed) == windowed
    assert windowed.joined(wider) == wider.joined(windowed) == KVSpec(1, 32, 33, keep=4)
    assert windowed.joined(whole) == whole.joined(wider) == whole
    assert KVSpec(2, 16, 0, 50).joined(KVSpec(2, 16, 0, 50, 3)) == KVSpec(2, 16, 0, 50, 3)
    assert KVSpec(2, 16, 0, 50).joined(KVSpec(2, 16, 0, 60)) == KVSpec(2, 16, 30).joined(KVSpec(2, 16, 0, 60)) == KVSpec(2, 16)
    with pytest.raises(ValueError):
        windowed.joined(KVSpec(1, 48, 20))


@pytest.mark.parametrize("window,keep", [(70, 5), (70, 64), (70, 65), (30, 130), (1, 1), (64, 0)])
def test_ledger_keeps_the_blocks_of_the_first_positions(window, keep):
    ledger = CacheLedger(2, 64, 4, 32, windows=[0, window], keeps=[0, keep])
    slot = ledger.acquire()
    for length in (1, 63, 64, 65, 130, 193, 200, 500, 501):
        ledger.check_growth({slot: length})
        ledger.reserve(slot, length)
        ledger.commit(slot, length)
        ledger.check()
        held = ledger.held_blocks[1][slot]
        # the next token (position ``length``) reads positions length - window + 1 .. and those below keep
        for index, block in enumerate(held):
            positions = range(index * BLOCK, index * BLOCK + BLOCK)
            needed = any(p < keep or p >= length - window + 1 for p in positions)
            assert (block != RELEASED) == needed, (length, index)
        assert RELEASED not in ledger.held_blocks[0][slot]
    ledger.release(slot)
    ledger.check()
    with pytest.raises(ValueError):
        CacheLedger(2, 8, 2, 8, keeps=[0])


def test_the_most_keys_a_query_sees():
    assert keys_in_reach(5000, 0, 0, 10) == 5000
    assert keys_in_reach(5000, 100, 0, 0) == 132 and keys_in_reach(5000, 100, 0, 33) == 196 and keys_in_reach(90, 100, 0, 33) == 90


def test_plain_mechanisms_are_pinned():
    """The plain implementation on inputs whose answers are known by hand."""
    # the layers' norm: the stored scale is the distance from one
    x = torch.tensor([[3.0, 4.0]], dtype=F64)
    assert torch.allclose(plain.layer_norm(x, torch.tensor([0.0, 1.0], dtype=F64), 0.0), torch.tensor([[3.0, 8.0]], dtype=F64) / math.sqrt(12.5))
    # neighbours turn together; a quarter turn of every pair
    v = torch.tensor([[[1.0, 2.0, 3.0, 4.0]]], dtype=F64)
    assert torch.allclose(plain.turn(v, torch.tensor([math.pi / 2.0]), {"dims": 4, "base": 1.0}), torch.tensor([[[-2.0, 1.0, -4.0, 3.0]]], dtype=F64))
    assert torch.equal(plain.squared_relu(torch.tensor([-2.0, 0.0, 3.0])), torch.tensor([0.0, 0.0, 9.0]))
    # a window of 2 that keeps the first token
    seen = plain.visible(torch.arange(4), {"size": 2, "keep_first": 1})
    assert seen.tolist() == [[True, False, False, False], [True, True, False, False], [True, True, True, False], [True, False, True, True]]
    assert plain.visible(torch.arange(3), None).tolist() == torch.tril(torch.ones(3, 3)).bool().tolist()
    # the largest logits, a softmax over those alone
    chosen, weights = plain.choice(torch.tensor([1.0, 3.0, 2.0, -5.0], dtype=F64), 2)
    assert chosen == [1, 2] and torch.allclose(weights, torch.softmax(torch.tensor([3.0, 2.0], dtype=F64), 0))


def test_plain_experts_by_hand():
    """Two of three experts, chosen by logits with a bias that turns the choice; the shared expert on top."""
    w = {"m.router": torch.tensor([[1.0, 0.0], [0.0, 1.0], [-1.0, -1.0]], dtype=F64), "m.router.b": torch.tensor([0.0, 0.0, 6.0], dtype=F64)}
    for e in range(3):
        w[f"m.e{e}.up"], w[f"m.e{e}.down"] = torch.eye(2, dtype=F64) * (e + 1), torch.eye(2, dtype=F64)
    w["m.shared.up"], w["m.shared.down"] = torch.eye(2, dtype=F64), 2.0 * torch.eye(2, dtype=F64)
    h = torch.tensor([[2.0, -1.0]], dtype=F64)
    mlp = {"kind": "moe", "expert": {"ff": 2}, "router": {"experts": 3, "top": 2}, "shared": {"ff": 2}}
    s = torch.softmax(torch.tensor([2.0, 5.0], dtype=F64), 0)                # logits 2, -1, 5: experts 0 and 2
    square = torch.tensor([[4.0, 0.0]], dtype=F64)
    assert torch.allclose(plain.experts(h, w, "m.", mlp), s[0] * square + s[1] * 9.0 * square + 2.0 * square, rtol=1e-14)
    assert torch.allclose(plain.experts(h, w, "m.", dict(mlp, shared=None)), s[0] * square + s[1] * 9.0 * square, rtol=1e-14)


def test_plain_windows_kept_tokens_and_borrowed_latents():
    # a window one shorter changes exactly the position that loses its first key, and not where the kept tokens hold it
    config, weights = CONFIGS["attention"][0], weights_for("attention")
    ids = prompts_for("attention", [90])[0]
    base = plain.forward(ids, weights, config)

    def masked(size, keep):
        mixer = dict(config["layers"][0]["mixer"], mask={"size": size, "keep_first": keep})
        return plain.forward(ids, weights, dict(config, layers=[dict(config["layers"][0], mixer=mixer)]))
    shorter = masked(39, 3)                  # windows 40 and 39, three kept: positions up to 41 see everything either way
    assert float((shorter[:42] - base[:42]).abs().max()) < 1e-12 and float((shorter[42] - base[42]).abs().max()) > 1e-6
    fewer = masked(40, 2)
    assert float((fewer[:42] - base[:42]).abs().max()) < 1e-12 and float((fewer[42] - base[42]).abs().max()) > 1e-6
    # a borrowed latent is its owner's: the owner's W_dkv moves the borrower's output even with the owner's own output cut off
    config, weights = CONFIGS["borrowed"][0], dict(weights_for("borrowed"))
    ids = prompts_for("borrowed", [30])[0]
    weights["l0.mix.o"] = torch.zeros_like(weights["l0.mix.o"])
    base = plain.forward(ids, weights, config)
    weights["l0.mix.dkv"] = weights["l0.mix.dkv"].flip(1)
    assert float((plain.forward(ids, weights, config) - base).abs().max()) > 1e-3
