"""Tiny Rirovik configurations and helpers shared by the tests of that family."""

import torch

import burn_transformers_amd as bt
import plain_rirovik as plain


def mask_of(window, keep):
    if not window:
        return None
    return {"size": window, "keep_first": keep} if keep else {"size": window}


def attention(heads, kv_heads, dim, vdim, scale, window=None, keep=0):
    return "attention", {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "mask": mask_of(window, keep)}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=10000.0, window=None, keep=0, kv_from=None, gated=True):
    sizes = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "scale": scale,
             "rot": {"base": base, "dims": rot_dim} if rot_dim else None, "mask": mask_of(window, keep)}
    if kv_from is not None:
        sizes["kv_from"] = kv_from
    return "latent_attention" if gated else "latent_attention_2", sizes


def moe(experts, ff, top, shared=None):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}, "shared": {"ff": shared} if shared else None}


def layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def model_config(layers, width=64, vocab=211, eps=1e-5, scale=2.0):
    return {"architecture": "Rirovik", "vocab": vocab, "width": width, "embedding": {"scale": scale}, "norm": {"eps": eps}, "layers": layers}


# all three mixers, a latent that two later layers borrow (one sees further back than its owner), kept first tokens that are no
# multiple of a tile, values wider than keys
BASIC = model_config([layer(attention(4, 2, 16, 32, 0.7, window=24, keep=5), moe(6, 24, 3, shared=40)),
                      layer(latent(3, 16, 8, 24, 40, 32, 0.3, base=2000.0, window=20), moe(4, 16, 2)),
                      layer(latent(2, 24, 8, 16, 24, 32, 0.3, base=2000.0, window=33, kv_from=1), moe(5, 16, 2, shared=24)),
                      layer(latent(4, 32, 16, 16, 48, 48, 0.2, base=500.0, gated=False), moe(4, 32, 1, shared=16)),
                      layer(latent(2, 16, 8, 16, 24, 32, 0.3, base=2000.0, kv_from=1, gated=False), moe(3, 16, 2))])
# sizes the kernels do not divide, no turned part, one expert a token, every expert chosen, no shared expert, a layer without a
# feed-forward, no mask, more kept tokens than the window holds, a window on borrowed keys that are kept for a whole context
ODD = model_config([layer(attention(3, 1, 10, 6, 0.9, window=7, keep=9), moe(5, 12, 1)),
                    layer(latent(5, 24, 6, 10, 18, 44, 0.25, base=100.0, gated=False), moe(3, 20, 3, shared=9)),
                    layer(latent(2, 12, 0, 20, 30, 20, 0.4, window=11)),
                    layer(latent(3, 20, 6, 14, 12, 44, 0.25, base=100.0, window=13, kv_from=1), moe(2, 22, 2)),
                    layer(attention(2, 2, 24, 10, 0.5), moe(7, 10, 4, shared=30))], width=40, vocab=97, eps=1e-3, scale=0.5)
# each mechanism alone, in a model of one or two layers
ATTENTION_ONLY = model_config([layer(attention(6, 2, 32, 32, 0.6, window=40, keep=3))], vocab=101)
LATENT_ONLY = model_config([layer(latent(4, 32, 16, 24, 48, 64, 0.2, base=5000.0, window=33))], vocab=101)
FULL_LATENT_ONLY = model_config([layer(latent(4, 32, 16, 24, 48, 64, 0.2, base=5000.0, gated=False))], vocab=101)
BORROWED = model_config([layer(latent(2, 16, 8, 16, 24, 40, 0.3, window=17)), layer(latent(6, 32, 8, 24, 48, 40, 0.3, window=50, kv_from=0)),
                         layer(latent(3, 16, 8, 16, 20, 40, 0.3, kv_from=0, gated=False))], vocab=101)
EXPERTS_ONLY = model_config([layer(attention(1, 1, 8, 8, 0.5), moe(8, 16, 2, shared=24))], width=32, vocab=61)
# windows and kept tokens that span several blocks of the cache, heads of 128, a latent wider than any MFMA attention kernel's head
LONG = model_config([layer(attention(2, 1, 128, 64, 2.0, window=200, keep=70), moe(4, 32, 2, shared=16)),
                     layer(latent(2, 64, 32, 48, 64, 112, 0.1, base=30000.0, window=150)),
                     layer(latent(2, 64, 32, 48, 64, 96, 0.1, base=30000.0, gated=False), moe(3, 16, 2)),
                     layer(latent(4, 32, 32, 32, 64, 112, 0.1, base=30000.0, window=210, kv_from=1))], width=96, vocab=151)
# more query heads on a cached head than a decode tile takes, on keys of its own and on borrowed ones
MANY_HEADS = model_config([layer(latent(4, 32, 32, 32, 48, 96, 0.2, window=70), moe(3, 16, 2)),
                           layer(latent(20, 8, 32, 8, 24, 96, 0.3, window=48, kv_from=0)),
                           layer(attention(20, 1, 16, 16, 0.8, window=48, keep=2)),
                           layer(latent(18, 16, 8, 8, 24, 40, 0.3, gated=False))], width=48, vocab=71)
# heads wider than any MFMA attention kernel's
WIDE_HEADS = model_config([layer(attention(2, 1, 144, 20, 2.0, window=30, keep=4)),
                           layer(latent(2, 40, 64, 144, 72, 250, 0.1, window=64)),
                           layer(latent(3, 20, 64, 30, 40, 250, 0.1, kv_from=1, gated=False))], width=32, vocab=53)
# nothing a multiple of eight
UNALIGNED = model_config([layer(attention(2, 1, 12, 20, 0.9, window=9, keep=1), moe(3, 10, 2, shared=7)),
                          layer(latent(3, 10, 6, 5, 7, 9, 0.3, window=11), moe(3, 5, 1)),
                          layer(latent(5, 7, 6, 3, 11, 9, 0.3, window=6, kv_from=1), moe(2, 3, 1, shared=1))], width=36, vocab=53)
# one of everything
ONES = model_config([layer(attention(1, 1, 1, 1, 1.0, window=1, keep=1), moe(1, 1, 1, shared=1)),
                     layer(latent(1, 1, 2, 1, 1, 1, 1.0, base=7.0, window=1), moe(1, 1, 1)),
                     layer(latent(1, 1, 2, 1, 1, 1, 1.0, base=7.0, window=2, kv_from=1))], width=24, vocab=19)
CONFIGS = {"basic": (BASIC, 1), "odd": (ODD, 2), "attention": (ATTENTION_ONLY, 3), "latent": (LATENT_ONLY, 4),
           "full_latent": (FULL_LATENT_ONLY, 5), "borrowed": (BORROWED, 6), "experts": (EXPERTS_ONLY, 7), "long": (LONG, 8),
           "many_heads": (MANY_HEADS, 9), "wide_heads": (WIDE_HEADS, 10), "unaligned": (UNALIGNED, 11), "ones": (ONES, 12)}

_weights, _models = {}, {}


def every_expert(config):
    """The configuration with every token using every expert."""
    layers = []
    for entry in config["layers"]:
        if entry["mlp"]:
            entry = dict(entry, mlp=dict(entry["mlp"], router=dict(entry["mlp"]["router"], top=entry["mlp"]["router"]["experts"])))
        layers.append(entry)
    return dict(config, layers=layers)


def config_for(name, dtype="float32"):
    """The configuration a run uses.  bfloat16 runs let every token use every expert: with operands rounded to 8 bits a
    near tie between two experts' logits falls the other way now and then, the token's whole feed-forward output is then
    another, and no bound on rounding holds.  The choice itself is made in the float32 runs, which go through the same
    kernels."""
    config = CONFIGS[name][0]
    return every_expert(config) if dtype == "bfloat16" else config


def sharpened(tensors, factor):
    """Latent attention whose weight lies on few keys, so that a lost key shows: the scales of the query latents' norms
    times ``factor`` (attention's own queries are unit heads; its configurations here have large scales instead)."""
    return {k: (v * factor if k.endswith(".mix.dq.norm") else v) for k, v in tensors.items()}


def weights_for(name, sharpen=1.0):
    """float32 weights as a load will see them (rounded to bfloat16)."""
    key = (name, sharpen)
    if key not in _weights:
        config, seed = CONFIGS[name]
        _, tensors = bt.random_tensors(config, seed)
        _weights[key] = {k: v.to(torch.bfloat16).float() for k, v in sharpened(tensors, sharpen).items()}
    return _weights[key]


def model_for(name, dtype, sharpen=1.0):
    key = (name, dtype, sharpen)
    if key not in _models:
        stored = {k: v.to(torch.bfloat16) for k, v in weights_for(name, sharpen).items()}
        _models[key] = bt.model_from_tensors(config_for(name, dtype), stored, dtype, "cuda:0")
    return _models[key]


def engine_for(name, dtype, max_tokens=4096, sharpen=1.0, **options):
    return bt.Engine(model_for(name, dtype, sharpen), max_tokens=max_tokens, **options)


def plain_logits(name, ids, sharpen=1.0, dtype="float32"):
    return plain.forward(ids, weights_for(name, sharpen), config_for(name, dtype))


def prompts_for(name, lengths, seed=0):
    gen = torch.Generator().manual_seed(seed)
    return [torch.randint(0, CONFIGS[name][0]["vocab"], (n,), generator=gen).tolist() for n in lengths]


def tolerance(dtype, reference):
    """Largest allowed absolute error of logits: float32 differs from float64 by the rounding of sums;
    bfloat16 rounds the operands of every product to 8 bits."""
    scale = float(reference.abs().max())
    return 2e-5 + 3e-5 * scale if dtype == "float32" else 4e-2 * scale


def random_config(seed):
    """A configuration drawn from a seed: two to six layers of any kind in any order, with a feed-forward or none, sizes,
    windows, kept tokens, borrowed latents and constants from short lists."""
    import random
    rng = random.Random(seed)
    width = rng.choice([64, 96, 128, 160, 256])

    def window():
        return rng.choice([1, 5, 32, 64, 96, 100, 160]) if rng.random() < 0.75 else None

    layers = []
    for _ in range(rng.randint(2, 6)):
        owners = [i for i, e in enumerate(layers) if e["type"] != "attention" and "kv_from" not in e["mixer"]]
        kind = rng.random()
        if kind < 0.4:
            kv, dim = rng.choice([1, 2, 4]), rng.choice([16, 32, 48, 64, 80, 128])
            mixer = attention(kv * rng.choice([1, 2, 3, 4, 8]), kv, dim, rng.choice([16, 32, 48, 64, 128]), dim ** -0.5 * rng.choice([0.5, 1.0, 3.0]),
                              window=window(), keep=rng.choice([0, 1, 4, 30, 64, 70, 130]))
        else:
            heads, dim, vdim, q_rank = rng.choice([1, 2, 4, 6]), rng.choice([16, 32, 64, 96]), rng.choice([16, 32, 48, 80]), rng.choice([24, 64, 96])
            gated, scale = rng.random() < 0.6, rng.choice([0.1, 0.2, 0.4])
            see = window() if gated else None
            if owners and rng.random() < 0.5:
                source = rng.choice(owners)
                of = layers[source]["mixer"]
                mixer = latent(heads, dim, of["rot_dim"], vdim, q_rank, of["kv_rank"], scale, base=of["rot"]["base"] if of["rot"] else 10000.0,
                               window=see, kv_from=source, gated=gated)
            else:
                mixer = latent(heads, dim, rng.choice([0, 8, 16, 32, 64]), vdim, q_rank, rng.choice([32, 64, 96, 128, 192]), scale,
                               base=rng.choice([100.0, 30000.0]), window=see, gated=gated)
        mlp = None
        if rng.random() < 0.8:
            count = rng.choice([1, 2, 4, 8, 12])
            mlp = moe(count, rng.choice([32, 64]), rng.randint(1, count), shared=rng.choice([None, 32, 100]))
        layers.append(layer(mixer, mlp))
    return model_config(layers, width=width, vocab=rng.choice([97, 320, 1000]), eps=rng.choice([1e-5, 1e-6]), scale=rng.choice([1.0, 3.0, 8.0]))
