"""Rirovik as a family: its plan, its checkpoint contract and its random initialisation.

This is the only file that knows Rirovik's wiring and tensor names.
  plan      token table times a scale; layers of the kinds config.json lists, each a ``sandwich_norm`` block:
            x += norm1b(mixer(norm1(x))), then, where the layer has a feed-forward, x += norm2b(ff(norm2(x))); the
            norms are RMS norms whose scales are stored as their distance from one.  Mixers: ``rotary_attention``
            without a rotation (config type attention: biased projections, unit query and key heads, a window beside
            which the first tokens stay visible, a gate on every output channel) and ``latent_attention`` (types
            latent_attention, with a window and an output gate per head, and latent_attention_2, with neither: queries
            and keys/values through normalised latents, one turned key part for all heads, neighbouring channels
            turned together).  A latent layer with ``kv_from`` has no latent of its own: its run reads the cache entry
            of the layer it names.  Feed-forward: ``routed_experts`` whose router has a bias, chooses by its logits and
            weighs by the softmax over the chosen ones; ungated units with the square of relu; an expert every token
            uses.  Final norm, readout with a table of its own.
  contract  tensor names ('l<i>.mix.*', 'l<i>.mlp.*', 'l<i>.norm1' ...), shapes
  init      random weights for tests and benchmarks
"""

import math

import torch

from ..config.registry import Family, register_family
from ..config.rirovik import RirovikConfig
from ..engine.plan import LayerPlan, ModelPlan, PartSpec, ScheduleEntry
from ..weights.contract import Contract, TensorSpec


def _attention_tensors(layer, width):
    """[(name below '<layer>.mix.', shape, layout, role in the part)]"""
    m = layer.mixer
    names = []
    for name, rows in (("q", m.heads * m.dim), ("k", m.kv_heads * m.dim), ("v", m.kv_heads * m.vdim)):
        names += [(name, (rows, width), "out_in", name + "_weight"), (name + ".b", (rows,), "vector", name + "_bias")]
    inner = m.heads * m.vdim
    return names + [("g", (inner, width), "out_in", "gate_weight"), ("o", (width, inner), "out_in", "out_weight")]


def _latent_tensors(layer, width):
    m = layer.mixer
    names = [("dq", (m.q_rank, width), "out_in", "down_q"), ("dq.norm", (m.q_rank,), "vector", "q_norm"),
             ("uq", (m.heads * (m.dim + m.rot_dim), m.q_rank), "out_in", "up_q")]
    if m.kv_from is None:
        names += [("dkv", (m.kv_rank + m.rot_dim, width), "out_in", "down_kv"), ("dkv.norm", (m.kv_rank,), "vector", "kv_norm")]
    names += [("uk", (m.heads * m.dim, m.kv_rank), "out_in", "up_k"), ("uv", (m.heads * m.vdim, m.kv_rank), "out_in", "up_v")]
    if layer.gated:
        names.append(("g", (m.heads, width), "out_in", "gate"))
    return names + [("o", (width, m.heads * m.vdim), "out_in", "out_weight")]


def _mixer_tensors(layer, index, width):
    """[(checkpoint name, shape, layout, role in the layer's mixer part)]"""
    tensors = (_attention_tensors if layer.type == "attention" else _latent_tensors)(layer, width)
    return [(f"l{index}.mix.{name}", shape, layout, role) for name, shape, layout, role in tensors]


def _mlp_tensors(mlp, index, width):
    p = f"l{index}.mlp."
    names = []
    for e in range(mlp.experts):
        names += [(f"{p}e{e}.up", (mlp.ff, width), "out_in", f"up_{e}"), (f"{p}e{e}.down", (width, mlp.ff), "out_in", f"down_{e}")]
    names += [(p + "router", (mlp.experts, width), "vector", "router"),             # routers are 32-bit: held widened
              (p + "router.b", (mlp.experts,), "vector", "router_bias")]
    if mlp.shared_ff:
        names += [(p + "shared.up", (mlp.shared_ff, width), "out_in", "shared_up"),
                  (p + "shared.down", (width, mlp.shared_ff), "out_in", "shared_down")]
    return names


def _mixer_spec(layer, index, config):
    m = layer.mixer
    tensors = {role: name for name, _, _, role in _mixer_tensors(layer, index, config.width)}
    params = {"width": config.width, "heads": m.heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale, "eps": config.norm_eps,
              "window": m.mask.size if m.mask else 0, "keep": m.mask.keep_first if m.mask else 0}
    if layer.type == "attention":
        return PartSpec("rotary_attention", {**params, "kv_heads": m.kv_heads, "head_norm": True, "norm_scale": False, "rot_dims": 0,
                                             "gate": "channel"}, tensors)
    params.update(q_rank=m.q_rank, kv_rank=m.kv_rank, rot_dim=m.rot_dim, rot_base=m.rot_base, rot_pairing="neighbours",
                  gate="head", borrows=m.kv_from is not None)
    return PartSpec("latent_attention", params, tensors)


def _mlp_spec(mlp, index, config):
    tensors = {role: name for name, _, _, role in _mlp_tensors(mlp, index, config.width)}
    return PartSpec("routed_experts",
                    {"width": config.width, "experts": mlp.experts, "ff": mlp.ff, "top": mlp.top, "shared_ff": mlp.shared_ff,
                     "score": "chosen", "normalize": True, "unit": "squared_relu"}, tensors)


def plan(config: RirovikConfig) -> ModelPlan:
    width = config.width

    def norm(name):
        return PartSpec("rms_norm", {"width": width, "eps": config.norm_eps, "offset": 1.0}, {"weight": name})

    layers, schedule, entries = [], [], {}
    for index, layer in enumerate(config.layers):
        p = f"l{index}."
        parts = {"mixer_norm": norm(p + "norm1"), "mixer": _mixer_spec(layer, index, config), "mixer_post": norm(p + "norm1b")}
        if layer.mlp is not None:
            parts.update(ff_norm=norm(p + "norm2"), ff=_mlp_spec(layer.mlp, index, config), ff_post=norm(p + "norm2b"))
        layers.append(LayerPlan("sandwich_norm", parts))
        source = getattr(layer.mixer, "kv_from", None)
        if source is None:
            entries[index] = len(entries)
        schedule.append(ScheduleEntry(layer=index, cache=entries[index if source is None else source], writes=source is None))
    return ModelPlan(
        width=width, vocab_size=config.vocab, max_positions=2 ** 31 - 1,      # positions are angles: no table bounds them
        embedding=PartSpec("token_only", {"width": width, "vocab_size": config.vocab, "scale": config.embedding_scale},
                           {"tokens": "embed"}),
        layers=layers, schedule=schedule, final_norm=norm("final.norm"),
        readout=PartSpec("linear_readout", {"width": width, "vocab_size": config.vocab}, {"weight": "head"}))


def contract(config: RirovikConfig) -> Contract:
    width = config.width
    tensors = [TensorSpec("embed", (config.vocab, width), "table")]
    for index, layer in enumerate(config.layers):
        p = f"l{index}."
        norms = ("1", "2", "1b", "2b") if layer.mlp is not None else ("1", "1b")
        tensors += [TensorSpec(p + "norm" + n, (width,), "vector") for n in norms]
        tensors += [TensorSpec(name, shape, layout) for name, shape, layout, _ in _mixer_tensors(layer, index, width)]
        if layer.mlp is not None:
            tensors += [TensorSpec(name, shape, layout) for name, shape, layout, _ in _mlp_tensors(layer.mlp, index, width)]
    tensors += [TensorSpec("final.norm", (width,), "vector"), TensorSpec("head", (config.vocab, width), "table")]
    return Contract(tensors=tensors, prefixes=("",), anchor="embed")


def init(config: RirovikConfig, generator):
    """Matrices N(0, 1/in), so routers' logits spread about one; biases and the layers' norm scales around zero (they are
    stored as the distance from one), the latents' scales around one."""

    def normal(shape, std, mean=0.0):
        return torch.randn(shape, generator=generator, dtype=torch.float32) * std + mean

    tensors = {}
    for spec in contract(config).tensors:
        name, shape = spec.name, spec.shape
        leaf = name.rsplit(".", 1)[-1]
        if name == "embed":
            tensors[name] = normal(shape, 1.0)
        elif leaf in ("norm1", "norm2", "norm1b", "norm2b") or name == "final.norm":
            tensors[name] = normal(shape, 0.1)
        elif leaf == "b":
            tensors[name] = normal(shape, 0.3)
        elif len(shape) == 1:                                          # plain scales of the latents' norms
            tensors[name] = normal(shape, 0.1, 1.0)
        else:
            tensors[name] = normal(shape, 1.0 / math.sqrt(shape[-1]))
    return tensors


FAMILY = register_family(Family(
    name="rirovik", architectures=("Rirovik",), model_types=("rirovik",),
    config_class=RirovikConfig, plan=plan, contract=contract, init=init))
