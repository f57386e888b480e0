"""Loselix through the engine against the plain implementation: every mechanism alone, and every way of cutting,
batching and reusing that must not change the logits."""

import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

pytestmark = pytest.mark.gpu

import burn_transformers_amd as bt  # noqa: E402
import plain_loselix as plain  # noqa: E402
from burn_transformers_amd.kernels import library as K  # noqa: E402
from loselix_helpers import (ASKS, CONFIGS, HOLDS, engine_for, model_for, model_from, plain_logits, planted, prompts_for,  # noqa: E402
                             random_config, tolerance, weights_for)

DTYPES = ["float32", "bfloat16"]
SHARPEN = 4.0        # factor on the queries where attention is to put its weight on few keys


def check(got, want, dtype, what):
    """float32: every row within the bound.  bfloat16: a row in forty (at least two) may pass it: the norm of a head's
    difference divides by the difference's own size, so where the two maps nearly cancel, rounding to 8 bits decides
    its direction."""
    got = got.detach().cpu().double()
    assert torch.isfinite(got).all(), what
    rows = (got - want).abs().max(dim=1).values
    bound = tolerance(dtype, want)
    over = int((rows > bound).sum())
    allowed = 0 if dtype == "float32" else max(2, rows.numel() // 40)
    assert over <= allowed, f"{what}: {over} rows over {bound}, max abs error {float(rows.max())}"


def whole(engine, ids):
    slot = engine.open()
    logits = engine.step([(slot, ids)], want=[list(range(len(ids)))]).clone()
    engine.close(slot)
    return logits


def decoded(engine, ids, head):
    """The first ``head`` tokens in one step, the others one by one."""
    slot = engine.open()
    rows = [engine.step([(slot, ids[:head])], want=[list(range(head))]).clone()]
    rows += [engine.step([(slot, [token])]).clone() for token in ids[head:]]
    engine.close(slot)
    return torch.cat(rows)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,lengths", [("differential", [1, 2, 9, 63, 64, 65, 130, 300]), ("head_gated", [1, 2, 9, 63, 64, 65, 130, 300]),
                                          ("sigmoid", [1, 2, 15, 16, 17, 64, 65, 300]), ("basic", [1, 2, 15, 16, 17, 40, 64, 65, 130, 530]),
                                          ("odd", [1, 2, 6, 7, 8, 64, 101, 210]), ("aligned", [1, 8, 9, 33, 64, 65, 257]),
                                          ("many_heads", [1, 20, 100]), ("wide_heads", [1, 31, 90]), ("unaligned", [1, 2, 10, 70])])
def test_each_mechanism_and_each_request_whole(name, dtype, lengths):
    engine = engine_for(name, dtype)
    for ids in prompts_for(name, lengths):
        check(whole(engine, ids), plain_logits(name, ids), dtype, f"{name} whole {len(ids)}")
    engine.cache.ledger.check()


@pytest.mark.parametrize("name", ["basic", "odd"])
def test_residual_stream_after_every_run_of_a_layer(name):
    """The stream itself, run by run (the looped layers several times), in float32."""
    model = model_for(name, "float32")
    engine = bt.Engine(model, max_tokens=256, graphs=False, programs=False)
    ids = prompts_for(name, [29], seed=4)[0]
    want = []
    plain.forward(ids, weights_for(name), CONFIGS[name][0], streams=want)
    caught, restore = [], []
    for block in model.blocks:
        if "mixer" not in block.parts:
            continue
        restore.append(block)

        def run(stream, step, memory, forward=block.forward):
            forward(stream, step, memory)
            stream.flush()
            caught.append(stream.x.detach().cpu().double().clone())
        block.forward = run
    try:
        slot = engine.open()
        engine.step([(slot, ids)])
        engine.close(slot)
    finally:
        for block in restore:
            del block.forward
    assert len(caught) == len(want)
    for number, (got, reference) in enumerate(zip(caught, want)):
        assert float((got - reference).abs().max()) <= 2e-5 + 2e-5 * float(reference.abs().max()), f"run {number}"


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,length,tail", [("basic", 110, 50), ("odd", 80, 20), ("differential", 140, 80), ("head_gated", 140, 80),
                                              ("sigmoid", 140, 80), ("aligned", 80, 20), ("many_heads", 90, 30), ("wide_heads", 80, 20),
                                              ("unaligned", 30, 20)])
def test_prompt_then_token_by_token(name, dtype, length, tail):
    """The last tokens one by one through the cache give what the whole prompt gives; the tails pass block borders
    and steps of the temperature."""
    engine = engine_for(name, dtype)
    ids = prompts_for(name, [length], seed=3)[0]
    check(decoded(engine, ids, length - tail), plain_logits(name, ids), dtype, f"{name} decode")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["basic", "odd"])
def test_from_the_first_token_one_by_one(name, dtype):
    engine = engine_for(name, dtype)
    ids = prompts_for(name, [70], seed=9)[0]
    check(decoded(engine, ids, 1), plain_logits(name, ids), dtype, f"{name} from the first token")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name,portion", [("basic", 2), ("basic", 3), ("basic", 64), ("basic", 65), ("odd", 2), ("odd", 7), ("odd", 50),
                                          ("aligned", 12), ("long", 193)])
def test_prompt_in_portions(name, dtype, portion):
    engine = engine_for(name, dtype)
    ids = prompts_for(name, [600 if name == "long" else 151], seed=5)[0]
    slot = engine.open()
    rows = []
    for at in range(0, len(ids), portion):
        part = ids[at:at + portion]
        rows.append(engine.step([(slot, part)], want=[list(range(len(part)))]).clone())
    check(torch.cat(rows), plain_logits(name, ids), dtype, f"{name} in portions of {portion}")
    engine.close(slot)
    engine.cache.ledger.check()


def batch_then_decode(engine, prompts, extra):
    """The prompts in one step, then one token of every request that still has some in each further step."""
    slots = [engine.open() for _ in prompts]
    got = [[] for _ in prompts]
    logits = engine.step(list(zip(slots, prompts)), want=[list(range(len(p))) for p in prompts])
    at = 0
    for i, p in enumerate(prompts):
        got[i].append(logits[at:at + len(p)].clone())
        at += len(p)
    for t in range(max(len(e) for e in extra)):
        live = [i for i in range(len(prompts)) if t < len(extra[i])]
        logits = engine.step([(slots[i], [extra[i][t]]) for i in live])
        for row, i in enumerate(live):
            got[i].append(logits[row:row + 1].clone())
        for i in range(len(prompts)):
            if t + 1 == len(extra[i]):
                engine.close(slots[i])
    return [torch.cat(rows) for rows in got]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["basic", "odd", "unaligned"])
def test_unequal_batch_decoded_together_then_slots_and_blocks_reused(name, dtype):
    """Requests of unequal length in one step, decoded together while the shorter ones end; then a
    second batch in the slots and blocks the first gave back."""
    engine = engine_for(name, dtype, max_tokens=1024)
    for number, lengths in enumerate([[1, 70, 33, 129], [64, 5, 90]]):
        prompts = prompts_for(name, lengths, seed=20 + number)
        extra = [prompts_for(name, [t], seed=30 + i)[0] for i, t in enumerate([12, 5, 9, 3][:len(prompts)])]
        for i, got in enumerate(batch_then_decode(engine, prompts, extra)):
            check(got, plain_logits(name, prompts[i] + extra[i]), dtype, f"{name} batch {number} request {i}")
        engine.cache.ledger.check()
    assert not engine.cache.ledger.live_slots()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["basic", "aligned"])
def test_a_batch_large_enough_for_chunk_major_operands(name, dtype):
    """Twelve requests decoded together: the products' operands are then kept chunk-major where the sizes allow."""
    engine = engine_for(name, dtype, max_tokens=2048)
    prompts = prompts_for(name, [3, 1, 17, 64, 65, 20, 9, 40, 2, 30, 7, 12], seed=50)
    extra = [prompts_for(name, [t], seed=60 + i)[0] for i, t in enumerate([6, 5, 6, 6, 4, 6, 6, 3, 6, 6, 6, 6])]
    for i, got in enumerate(batch_then_decode(engine, prompts, extra)):
        check(got, plain_logits(name, prompts[i] + extra[i]), dtype, f"{name} request {i} of twelve")


@pytest.mark.parametrize("dtype", DTYPES)
def test_sharp_attention_over_many_blocks_whole_and_decoded(dtype):
    """Queries sharpened so that weight lies on few keys, a context of several blocks."""
    name = "long"
    ids = prompts_for(name, [400], seed=11)[0]
    want = plain_logits(name, ids, SHARPEN if dtype == "float32" else 2.0)
    engine = engine_for(name, dtype, sharpen=SHARPEN if dtype == "float32" else 2.0)
    check(whole(engine, ids), want, dtype, "long whole")
    check(decoded(engine, ids, 370), want, dtype, "long decoded")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["differential", "head_gated", "sigmoid"])
def test_one_far_key_with_nearly_all_the_weight(kind, dtype):
    """One key stands out: at the sequence's start, around block borders, far back and near; asked for in a prompt's
    portion and by a decoded token."""
    config, weights = planted(kind)
    engine = bt.Engine(model_from(config, weights, dtype), max_tokens=2048)
    gen = torch.Generator().manual_seed(2)
    ids = torch.randint(10, config["vocab"], (520,), generator=gen).tolist()
    ids[-1] = ids[330] = ASKS
    for place in (0, 1, 62, 63, 64, 65, 127, 128, 255, 256, 319, 320, 329):
        tokens = list(ids)
        tokens[place] = HOLDS
        want = plain.forward(tokens, weights, config)
        check(whole(engine, tokens), want, dtype, f"{kind}: the key at {place}, whole")
        asked = decoded(engine, tokens[:331], 330)[-1:]
        check(asked, want[330:331], dtype, f"{kind}: the key at {place}, decoded")
        bound = tolerance(dtype, want)
        for row, got in ((330, asked), (519, whole(engine, tokens)[-1:])):
            assert float((got.cpu().double() - want[row:row + 1]).abs().max()) <= bound, f"{kind}: the key at {place} for {row}"
    late = list(ids)
    late[331] = HOLDS                               # behind the first query: not seen
    base = whole(engine, ids)
    assert torch.equal(whole(engine, late)[330], base[330])
    assert not torch.equal(whole(engine, late)[519], base[519])


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dtype):
    name = "basic"
    engine = engine_for(name, dtype)
    ids = prompts_for(name, [330], seed=12)[0]
    check(decoded(engine, ids, 4), plain_logits(name, ids), dtype, "326 tokens one by one")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["differential", "head_gated", "sigmoid"])
def test_decoding_far_out_in_runs_of_keys(kind, dtype):
    """Contexts beyond 1,024 tokens, where a decode step of one sequence cuts its keys into runs that are joined (heads of
    128); positions with steps of the temperature far out."""
    from loselix_helpers import differential, head_gated, layer, model_config, rotation, sigmoid
    mixer = {"differential": differential(2, 1, 64, 128, 0.2, rotation(32), cap=20.0), "head_gated": head_gated(2, 1, 128, 128, 0.15, rotation(64)),
             "sigmoid": sigmoid(2, 1, 128, 0.12, coef=0.4, every=300)}[kind]
    config = model_config([layer(mixer, 32)], width=64, vocab=61)
    _, tensors = bt.random_tensors(config, 21)
    weights = {k: v.to(torch.bfloat16).float() for k, v in tensors.items()}
    engine = bt.Engine(model_from(config, weights, dtype), max_tokens=2600)
    ids = torch.randint(0, 61, (2408,), generator=torch.Generator().manual_seed(4)).tolist()
    want = plain.forward(ids, weights, config)
    slot = engine.open()
    first = engine.step([(slot, ids[:2395])], want=[[0, 1023, 1024, 2099, 2394]]).clone()
    check(first, want[[0, 1023, 1024, 2099, 2394]], dtype, f"{kind} prompt")
    engine.close(slot)
    slot = engine.open()                   # the same in portions: those behind 1,024 tokens cut their keys into runs too
    for begin, end in ((0, 1500), (1500, 1630), (1630, 1640), (1640, 2200), (2200, 2395)):
        places = [0, (end - begin) // 2, end - begin - 1]
        part = engine.step([(slot, ids[begin:end])], want=[places]).clone()
        check(part, want[[begin + p for p in places]], dtype, f"{kind} portion {begin} to {end}")
    rows = torch.cat([engine.step([(slot, [token])]).clone() for token in ids[2395:]])
    check(rows, want[2395:], dtype, f"{kind} decoded behind 2,395 tokens")
    engine.close(slot)


def test_blocks_that_are_used_again_hold_nothing_of_their_last_owner():
    name = "basic"
    engine = engine_for(name, "float32", max_tokens=512)
    first, second = prompts_for(name, [200, 30], seed=40)
    slot = engine.open()
    engine.step([(slot, first)])
    engine.close(slot)
    again = engine.open()
    assert again == slot
    got = engine.step([(again, second)], want=[list(range(len(second)))]).clone()
    engine.truncate(again, 12)                    # rewound: the second half once more, other tokens
    other = prompts_for(name, [18], seed=41)[0]
    redone = engine.step([(again, other)], want=[list(range(18))]).clone()
    engine.close(again)
    check(got, plain_logits(name, second), "float32", "a slot used again")
    check(redone, plain_logits(name, second[:12] + other)[12:], "float32", "a sequence rewound")


@pytest.mark.parametrize("seed", range(14))
def test_configurations_drawn_at_random(seed):
    """Layers, sizes, loops and constants drawn from a seed: three unequal prompts in one step, then decoded together
    while the shorter requests end; float32, and bfloat16 for every other seed."""
    config = random_config(seed)
    _, tensors = bt.random_tensors(config, seed)
    weights = {k: v.to(torch.bfloat16).float() for k, v in tensors.items()}
    gen = torch.Generator().manual_seed(seed)
    prompts = [torch.randint(0, config["vocab"], (n,), generator=gen).tolist() for n in (3, 70, 200)]
    extra = [torch.randint(0, config["vocab"], (t,), generator=gen).tolist() for t in (4, 9, 6)]
    want = [plain.forward(p + e, weights, config) for p, e in zip(prompts, extra)]
    for dtype in DTYPES[:1 + seed % 2]:
        engine = bt.Engine(model_from(config, weights, dtype), max_tokens=1024)
        for i, got in enumerate(batch_then_decode(engine, prompts, extra)):
            check(got, want[i], dtype, f"seed {seed} request {i} {dtype}: {config}")


@pytest.mark.parametrize("name", ["basic", "aligned"])
@pytest.mark.parametrize("graphs,programs", [(False, False), (False, True), ("always", True)])
def test_launch_lists_and_graphs_give_the_same_bits(name, graphs, programs):
    prompts = prompts_for(name, [70] + [15] * 9, seed=13)
    rows = {}
    for key, options in (("direct", dict(graphs=False, programs=False)), ("other", dict(graphs=graphs, programs=programs))):
        engine = engine_for(name, "bfloat16", **options)
        got = []
        for _ in range(3):          # a shape comes again: recorded, then replayed
            slots = [engine.open() for _ in prompts]
            got.append(engine.step([(s, p[:12]) for s, p in zip(slots, prompts)], want=[[11]] * len(slots)).clone())
            for t in range(12, 15):
                got.append(engine.step([(s, [p[t]]) for s, p in zip(slots, prompts)]).clone())
            for slot in slots[1:]:
                engine.close(slot)
            got += [engine.step([(slots[0], [token])]).clone() for token in prompts[0][15:]]
            engine.close(slots[0])
        rows[key] = torch.cat(got)
    assert torch.equal(rows["direct"], rows["other"])


@pytest.mark.parametrize("count", [1, 3, 12, 70])
def test_joined_and_carried_products_give_what_separate_ones_give(count):
    """The block with every product on its own (parts built apart from a block) against the joined form, float32."""
    name = "aligned"
    joined = model_for(name, "float32")
    apart = model_from(CONFIGS[name][0], weights_for(name), "float32")
    store = apart.store
    for index, block in enumerate(apart.blocks):
        if "ff" not in block.parts:
            continue
        from burn_transformers_amd.engine.model import build_part
        plan = apart.plan.layers[index]
        block.parts = {role: build_part(type(block).ROLES[role], spec, store) for role, spec in plan.parts.items()}
        block.output, block.carries = None, False
    ids = prompts_for(name, [count], seed=70)[0]
    got = [whole(bt.Engine(model, max_tokens=512), ids) for model in (joined, apart)]
    assert float((got[0] - got[1]).abs().max()) <= 2e-5 * float(got[1].abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_entry_point(dtype):
    name = "basic"
    config = CONFIGS[name][0]
    prompts = prompts_for(name, [5, 40, 1, 27], seed=14)
    engine = engine_for(name, dtype)
    got = bt.generate(engine, prompts, bt.GenerationConfig(max_new_tokens=10), prefill_chunk=16)
    for prompt, sequence in zip(prompts, got):
        ids = list(prompt)
        for token in sequence.token_ids:
            logits = plain.forward(ids, weights_for(name), config)[-1]
            best = int(logits.argmax())
            if dtype == "float32":
                assert token == best
            else:                    # 8-bit operands may take a token whose logit is within rounding of the best
                assert float(logits[best] - logits[token]) <= tolerance(dtype, logits)
            ids.append(token)
    assert not engine.cache.ledger.live_slots()


def test_folder_round_trip_and_replay(tmp_path):
    """A folder written with random weights, loaded by what config.json names, replayed step by step."""
    from burn_transformers_amd.engine.replay import Replay, cache_tokens
    config = CONFIGS["odd"][0]
    folder = tmp_path / "model"
    weights = bt.write_random_model(str(folder), config, seed=3)
    assert json.load(open(folder / "config.json"))["architecture"] == "Loselix"
    model = bt.load_model(str(folder), dtype="float32")
    replay = Replay(bt.Engine(model, max_tokens=cache_tokens(300)), str(tmp_path / "out"))
    a, b = prompts_for("odd", [45, 9], seed=15)
    replay.run([json.dumps({"step": 0, "entries": [{"id": "a", "tokens": a[:40], "want": [0, 39]},
                                                   {"id": "b", "tokens": b[:6], "want": [5]}], "end": []}),
                json.dumps({"step": 1, "entries": [{"id": "a", "tokens": a[40:41], "want": [0]},
                                                   {"id": "b", "tokens": b[6:7], "want": []}], "end": ["b"]}),
                json.dumps({"step": 2, "entries": [{"id": "a", "tokens": a[41:42], "want": [0]}], "end": ["a"]})],
               out=open(tmp_path / "log", "w"))
    want_a, want_b = plain.forward(a, weights, config), plain.forward(b, weights, config)
    first = torch.from_numpy(np.fromfile(tmp_path / "out" / "0.f32", dtype="<f4").reshape(3, -1)).double()
    check(first, torch.stack([want_a[0], want_a[39], want_b[5]]), "float32", "replayed step 0")
    for step, row in ((1, 40), (2, 41)):
        got = torch.from_numpy(np.fromfile(tmp_path / "out" / f"{step}.f32", dtype="<f4").reshape(1, -1)).double()
        check(got, want_a[row:row + 1], "float32", f"replayed step {step}")


def test_command_line(capsys, tmp_path):
    """The command line takes the family by config.json: random weights written from a configuration,
    then greedy tokens for two prompts, then sampled ones with the prompts fed in portions."""
    from burn_transformers_amd.cli import main
    config, seed = CONFIGS["basic"]
    cfg_path = tmp_path / "cfg.json"
    cfg_path.write_text(json.dumps(config))
    prompts = prompts_for("basic", [6, 30], seed=60)
    text = ";".join(",".join(str(t) for t in p) for p in prompts)
    assert main([str(tmp_path / "made"), text, "5", "--dtype", "float32", "--json", "--random-weights", str(cfg_path),
                 "--weights-seed", str(seed)]) == 0
    lines = [json.loads(line) for line in capsys.readouterr().out.strip().splitlines()]
    weights = weights_for("basic")
    assert [line["token_ids"] for line in lines] == [plain.greedy(p, weights, config, 5) for p in prompts]
    assert main([str(tmp_path / "made"), text, "4", "--temperature", "0.7", "--seed", "5", "--prefill-chunk-size", "4"]) == 0


def test_trace_runner_as_a_program(tmp_path):
    """bin/trace_run in a process of its own, in both number formats: a batch of two prompts, then
    both decoded together, one of them ending first."""
    config, weights = CONFIGS["basic"][0], weights_for("basic")
    os.makedirs(tmp_path / "model")
    (tmp_path / "model" / "config.json").write_text(json.dumps(config))
    bt.write_safetensors(str(tmp_path / "model" / "model.safetensors"), {k: v.to(torch.bfloat16) for k, v in weights.items()})
    a, b = prompts_for("basic", [70, 12], seed=22)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": a[:66], "want": [65]}, {"id": "y", "tokens": b[:10], "want": [0, 9]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": a[66:67], "want": [0]}, {"id": "y", "tokens": b[10:11], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": a[67:68], "want": [0]}, {"id": "y", "tokens": b[11:12], "want": [0]}], "end": ["y"]},
             {"step": 3, "entries": [{"id": "x", "tokens": a[68:69], "want": [0]}], "end": ["x"]}]
    want_a, want_b = plain.forward(a, weights, config), plain.forward(b, weights, config)
    expected = {0: [want_a[65], want_b[0], want_b[9]], 1: [want_a[66]], 2: [want_a[67], want_b[11]], 3: [want_a[68]]}
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    for dtype in DTYPES:
        out = tmp_path / ("out_" + dtype)
        done = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", str(tmp_path / "model"),
                               "--dtype", dtype, "--out", str(out), "--max-tokens", "100"],
                              input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=300)
        assert done.returncode == 0, done.stderr[-2000:]
        assert [line for line in done.stdout.splitlines() if line.startswith("done")] == [f"done {i}" for i in range(4)]
        for step, rows in expected.items():
            got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(len(rows), -1)).double()
            assert float((got - torch.stack(rows)).abs().max()) <= tolerance(dtype, want_a), (dtype, step)


def test_heads_and_widths_beyond_the_kernels_are_refused_when_the_model_is_built():
    from loselix_helpers import head_gated, layer, model_config
    config = model_config([layer(head_gated(1, 1, 320, 16, 0.1), 16)], width=32, vocab=31)
    _, tensors = bt.random_tensors(config, 0)
    with pytest.raises(ValueError, match="beyond 256"):
        bt.model_from_tensors(config, tensors, "bfloat16", "cuda:0")
    assert K.ACTIVATIONS["squared_relu"] == 2
