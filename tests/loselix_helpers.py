"""Tiny Loselix configurations and helpers shared by the tests of that family."""

import random

import torch

import burn_transformers_amd as bt
import plain_loselix as plain


def rotation(dims, base=10000.0):
    return {"dims": dims, "base": base} if dims else None


def differential(heads, kv_heads, dim, vdim, scale, rot=None, cap=30.0, diff=0.4):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot, "softcap": cap,
                         "diff": diff}


def head_gated(heads, kv_heads, dim, vdim, scale, rot=None):
    return "attention_2", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}


def sigmoid(heads, kv_heads, dim, scale, coef=0.2, every=16):
    return "attention_3", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": scale,
                           "q_temp": {"coef": coef, "every": every}}


def layer(mixer, ff=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model_config(layers, width=64, vocab=211, eps=1e-5, loop=None):
    return {"architecture": "Loselix", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "loop": dict(zip(("start", "stop", "times"), loop)) if loop else None, "layers": layers}


# all three mixers; the middle three layers run twice; values of twice a map's size, as wide as it and wider
BASIC = model_config([layer(differential(4, 2, 16, 32, 0.25, rotation(8, 500.0)), 96),
                      layer(head_gated(4, 1, 32, 48, 0.18, rotation(32)), 64),
                      layer(sigmoid(4, 2, 32, 0.2, coef=0.3, every=16), 80),
                      layer(differential(2, 1, 32, 16, 0.2, rotation(16, 2000.0), cap=20.0, diff=0.7), 64),
                      layer(head_gated(2, 2, 16, 16, 0.3, rotation(8)), 128)], loop=(1, 4, 2))
# sizes the kernels do not divide, values of one, the loop over the first layers, a layer without a feed-forward, no
# rotation, no cap, no temperature, a step of the temperature at every position, one query head a map
ODD = model_config([layer(sigmoid(3, 1, 20, 0.25, coef=-0.1, every=1), 50),
                    layer(differential(3, 3, 6, 5, 0.4, rotation(2, 100.0), cap=5.0, diff=0.1), 22),
                    layer(head_gated(5, 1, 24, 10, 0.2, rotation(24, 100.0))),
                    layer(differential(1, 1, 10, 40, 0.3, None, cap=None, diff=0.0), 9),
                    layer(head_gated(1, 1, 8, 7, 0.4), 30),
                    layer(("attention_3", dict(sigmoid(2, 2, 9, 0.3)[1], q_temp=None)))], width=40, vocab=97, eps=1e-3, loop=(0, 2, 3))
# each mixer alone, in a model of one layer
DIFFERENTIAL_ONLY = model_config([layer(differential(4, 2, 32, 64, 0.2, rotation(16, 1000.0)), 96)], vocab=101)
HEAD_GATED_ONLY = model_config([layer(head_gated(4, 2, 64, 64, 0.12, rotation(32, 1000.0)), 96)], vocab=101)
SIGMOID_ONLY = model_config([layer(sigmoid(4, 2, 48, 0.15), 96)], vocab=101)
# heads of 128 over several blocks of the cache, the whole model in one loop
LONG = model_config([layer(differential(2, 1, 64, 128, 0.11, rotation(32, 300000.0), cap=40.0, diff=0.3), 64),
                     layer(head_gated(3, 1, 128, 96, 0.09, rotation(64, 300000.0)), 64),
                     layer(sigmoid(2, 1, 128, 0.09, coef=0.25, every=100), 64)], width=96, vocab=151, loop=(0, 3, 2))
# operands that are chunk-major in steps of 9 to 64 rows, the loop over the last layer
ALIGNED = model_config([layer(differential(4, 2, 32, 64, 0.2, rotation(32)), 128), layer(head_gated(2, 1, 64, 64, 0.12, rotation(64)), 160),
                        layer(sigmoid(4, 4, 32, 0.2, every=7), 64)], width=128, vocab=131, loop=(2, 3, 3))
# more query heads (and maps) on a cached head than a decode tile takes
MANY_HEADS = model_config([layer(differential(10, 1, 8, 16, 0.3, rotation(4)), 48), layer(head_gated(20, 1, 16, 16, 0.25, rotation(16)), 40),
                           layer(sigmoid(18, 1, 16, 0.25), 24)], width=48, vocab=71)
# heads wider than any MFMA attention kernel's
WIDE_HEADS = model_config([layer(differential(2, 1, 96, 40, 0.1, rotation(50, 1000.0)), 40), layer(head_gated(2, 1, 144, 20, 0.08, rotation(100, 1000.0)), 24),
                           layer(sigmoid(2, 2, 160, 0.07), 16), layer(differential(1, 1, 20, 200, 0.2, rotation(20)), 24)], width=32, vocab=53)
# nothing a multiple of four
UNALIGNED = model_config([layer(sigmoid(3, 1, 7, 0.3, every=5), 11), layer(differential(3, 1, 6, 9, 0.3, rotation(6), cap=10.0), 21),
                          layer(head_gated(3, 3, 10, 13, 0.3, rotation(10)), 13)], width=42, vocab=53, loop=(1, 2, 2))
CONFIGS = {"basic": (BASIC, 1), "odd": (ODD, 2), "differential": (DIFFERENTIAL_ONLY, 3), "head_gated": (HEAD_GATED_ONLY, 4),
           "sigmoid": (SIGMOID_ONLY, 5), "long": (LONG, 6), "aligned": (ALIGNED, 7), "many_heads": (MANY_HEADS, 8),
           "wide_heads": (WIDE_HEADS, 9), "unaligned": (UNALIGNED, 10)}

_weights, _models = {}, {}


def weights_for(name, sharpen=1.0):
    """float32 weights as a load will see them (rounded to bfloat16).  ``sharpen`` multiplies what sets how sharply a
    query picks its keys (the query projections, or the scales behind them), so that a lost key shows."""
    key = (name, sharpen)
    if key not in _weights:
        config, seed = CONFIGS[name]
        _, tensors = bt.random_tensors(config, seed)
        if sharpen != 1.0:
            normed = {k.removesuffix(".norm") for k in tensors if k.endswith(".mix.q.norm")}
            tensors = {k: (v * sharpen if k.endswith(".mix.q.norm") or (k.endswith(".mix.q") and k not in normed) else v)
                       for k, v in tensors.items()}
        _weights[key] = {k: v.to(torch.bfloat16).float() for k, v in tensors.items()}
    return _weights[key]


def model_from(config, weights, dtype):
    return bt.model_from_tensors(config, {k: v.to(torch.bfloat16) for k, v in weights.items()}, dtype, "cuda:0")


def model_for(name, dtype, sharpen=1.0):
    key = (name, dtype, sharpen)
    if key not in _models:
        _models[key] = model_from(CONFIGS[name][0], weights_for(name, sharpen), dtype)
    return _models[key]


def engine_for(name, dtype, max_tokens=4096, sharpen=1.0, **options):
    return bt.Engine(model_for(name, dtype, sharpen), max_tokens=max_tokens, **options)


_plain = {}


def plain_logits(name, ids, sharpen=1.0):
    key = (name, tuple(ids), sharpen)
    if key not in _plain:
        _plain[key] = plain.forward(ids, weights_for(name, sharpen), CONFIGS[name][0])
    return _plain[key]


def prompts_for(name, lengths, seed=0):
    gen = torch.Generator().manual_seed(seed)
    return [torch.randint(0, CONFIGS[name][0]["vocab"], (n,), generator=gen).tolist() for n in lengths]


def tolerance(dtype, reference):
    """Largest allowed absolute error of logits: float32 differs from float64 by the rounding of sums;
    bfloat16 rounds the operands of every product to 8 bits."""
    scale = float(reference.abs().max())
    return 2e-5 + 3e-5 * scale if dtype == "float32" else 3e-2 * scale


# --- a far key that carries nearly all the weight ------------------------------------------------

ASKS, HOLDS = 5, 9         # tokens: a query for the key of the other


def planted(kind, dtype_seed=11):
    """(config, weights) of a one-layer model in which token ``ASKS`` as a query has ONE large score, with the key of token
    ``HOLDS``, wherever that lies, and in which token ``HOLDS`` has a value row like no other token's.  The score lies in
    a channel that is not turned, so that no distance changes it."""
    mixer = {"differential": differential(2, 1, 32, 64, 0.2, rotation(16, 1000.0), cap=30.0, diff=0.3),
             "head_gated": head_gated(2, 1, 48, 48, 0.15, rotation(16, 1000.0)),
             "sigmoid": sigmoid(2, 1, 48, 0.15, coef=0.1, every=64)}[kind]
    config = model_config([layer(mixer, 32)], width=64, vocab=83)
    _, tensors = bt.random_tensors(config, dtype_seed)
    width, m = config["width"], mixer[1]
    # the first two channels of the stream belong to the two tokens alone
    tensors["embed"][:, :2] = 0.0
    tensors["embed"][ASKS], tensors["embed"][HOLDS] = 0.0, 0.0
    tensors["embed"][ASKS, 0] = tensors["embed"][HOLDS, 1] = width ** 0.5
    tensors["l0.norm1"][:] = 1.0
    for name in ("q", "k"):
        weight = tensors["l0.mix." + name]
        weight[:, 0] = weight[:, 1] = 0.0
        parts = weight.view(-1, m["dim"], width)                # a row block per head, or per map of a head
        parts[0, m["dim"] - 1, 0 if name == "q" else 1] = {"differential": 3.0, "head_gated": 3.0, "sigmoid": 1.0}[kind]
    return config, {k: v.to(torch.bfloat16).float() for k, v in tensors.items()}


def random_config(seed):
    """A configuration drawn from a seed: two to five layers of any kind in any order, with a feed-forward or none, a
    loop or none, sizes and constants from short lists."""
    rng = random.Random(seed)
    width = rng.choice([64, 96, 128, 160, 256])
    layers = []
    for _ in range(rng.randint(2, 5)):
        kv = rng.choice([1, 2, 3])
        heads = kv * rng.choice([1, 2, 3, 4])
        kind = rng.randrange(3)
        factor = rng.choice([0.7, 1.0, 1.4])
        if kind == 0:
            dim = rng.choice([8, 16, 32, 40, 64])
            mixer = differential(heads, kv, dim, rng.choice([16, 32, 48, 64, 128]), dim ** -0.5 * factor,
                                 rotation(rng.choice([0, dim // 4 * 2, dim]), rng.choice([100.0, 10000.0, 500000.0])),
                                 cap=rng.choice([5.0, 20.0, 50.0]), diff=rng.choice([0.0, 0.2, 0.5, 0.8]))
        elif kind == 1:
            dim = rng.choice([16, 32, 48, 64, 80, 128])
            mixer = head_gated(heads, kv, dim, rng.choice([16, 32, 48, 64, 128]), dim ** -0.5 * factor,
                               rotation(rng.choice([0, dim // 4 * 2, dim]), rng.choice([100.0, 10000.0, 500000.0])))
        else:
            dim = rng.choice([16, 32, 48, 64, 96, 128])
            mixer = sigmoid(heads, kv, dim, dim ** -0.5 * factor, coef=rng.choice([0.1, 0.3, 0.5]), every=rng.choice([3, 32, 64, 100]))
        layers.append(layer(mixer, rng.choice([None, 64, 100, 200, 256])))
    loop = None
    if rng.random() < 0.7:
        start = rng.randrange(len(layers))
        loop = (start, rng.randint(start + 1, len(layers)), rng.randint(1, 3))
    return model_config(layers, width=width, vocab=rng.choice([97, 320, 1000]), eps=rng.choice([1e-5, 1e-6]), loop=loop)
