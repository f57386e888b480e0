"""Loselix as a family: its plan, its checkpoint contract and its random initialisation.

This is the only file that knows Loselix's wiring and tensor names.
  plan      token table; layers of the kinds config.json lists, each a ``parallel`` block: with h = norm1(x),
            x += mixer(h) + ff(h) (the feed-forward may be missing); RMS norms.  Mixers: ``differential_attention``
            (config type attention: two maps a head over the same values, capped scores, halves turned together) and
            ``rotary_attention`` in two forms (attention_2: a gate per head; attention_3: norms over the whole query and
            key projections, no rotation, queries that grow with their position, sigmoid weights with a bias per head,
            values that are the projected keys, a gate per channel).  Feed-forward: ``dense`` with the square of relu.
            With ``loop``, layers start .. stop - 1 run ``times`` times with the same tensors and a cache entry per
            run, and before every pass but the first ``add_origin`` adds the embedding's output.  Final norm, readout
            with a table of its own.
  contract  tensor names ('l<i>.mix.*', 'l<i>.mlp.*', 'l<i>.norm1' ...), shapes
  init      random weights for tests and benchmarks
"""

import math

import torch

from ..config.loselix import LoselixConfig
from ..config.registry import Family, register_family
from ..engine.plan import LayerPlan, ModelPlan, PartSpec, ScheduleEntry
from ..weights.contract import Contract, TensorSpec


def _differential_tensors(m, width):
    """[(name below '<layer>.mix.', shape, layout, role in the part)]"""
    return [("q", (m.heads * 2 * m.dim, width), "out_in", "q_weight"), ("k", (m.kv_heads * 2 * m.dim, width), "out_in", "k_weight"),
            ("v", (m.kv_heads * m.vdim, width), "out_in", "v_weight")] + \
        [(name, (m.dim,), "vector", role) for name, role in (("lq1", "lambda_q1"), ("lk1", "lambda_k1"), ("lq2", "lambda_q2"), ("lk2", "lambda_k2"))] + \
        [("o", (width, m.heads * m.vdim), "out_in", "out_weight")]


def _head_gated_tensors(m, width):
    return [("q", (m.heads * m.dim, width), "out_in", "q_weight"), ("k", (m.kv_heads * m.dim, width), "out_in", "k_weight"),
            ("v", (m.kv_heads * m.vdim, width), "out_in", "v_weight"), ("g", (m.heads, width), "out_in", "gate_weight"),
            ("o", (width, m.heads * m.vdim), "out_in", "out_weight")]


def _sigmoid_tensors(m, width):
    q, k = m.heads * m.dim, m.kv_heads * m.dim
    return [("q", (q, width), "out_in", "q_weight"), ("k", (k, width), "out_in", "k_weight"), ("q.norm", (q,), "vector", "q_norm"),
            ("k.norm", (k,), "vector", "k_norm"), ("pb", (m.heads,), "vector", "score_bias"),
            ("g", (m.heads * m.vdim, width), "out_in", "gate_weight"), ("o", (width, m.heads * m.vdim), "out_in", "out_weight")]


_MIXER_TENSORS = {"attention": _differential_tensors, "attention_2": _head_gated_tensors, "attention_3": _sigmoid_tensors}


def _mixer_tensors(layer, index, width):
    """[(checkpoint name, shape, layout, role in the layer's mixer part)]"""
    return [(f"l{index}.mix.{name}", shape, layout, role)
            for name, shape, layout, role in _MIXER_TENSORS[layer.type](layer.mixer, width)]


def _mlp_tensors(mlp, index, width):
    p = f"l{index}.mlp."
    return [(p + "up", (mlp.ff, width), "out_in", "up_weight"), (p + "down", (width, mlp.ff), "out_in", "down_weight")]


def _mixer_spec(layer, index, config):
    m = layer.mixer
    tensors = {role: name for name, _, _, role in _mixer_tensors(layer, index, config.width)}
    params = {"width": config.width, "heads": m.heads, "kv_heads": m.kv_heads, "dim": m.dim, "vdim": m.vdim, "scale": m.scale,
              "eps": config.norm_eps, "head_norm": False}
    rot = getattr(m, "rot", None)
    if rot is not None:
        params.update(rot_dims=rot.dims, rot_base=rot.base, rot_pairing="halves")
    if layer.type == "attention":
        return PartSpec("differential_attention", {**params, "softcap": m.softcap, "diff": m.diff}, tensors)
    if layer.type == "attention_2":
        return PartSpec("rotary_attention", {**params, "gate": "head"}, tensors)
    return PartSpec("rotary_attention",
                    {**params, "head_norm": True, "norm_span": "whole", "values": "keys", "weights": "sigmoid", "gate": "channel",
                     "temperature": {"coef": m.temp_coef, "every": m.temp_every} if m.temp_every else None}, tensors)


def plan(config: LoselixConfig) -> ModelPlan:
    width = config.width

    def norm(name):
        return PartSpec("rms_norm", {"width": width, "eps": config.norm_eps}, {"weight": name})

    layers = []
    for index, layer in enumerate(config.layers):
        parts = {"norm": norm(f"l{index}.norm1"), "mixer": _mixer_spec(layer, index, config)}
        if layer.mlp is not None:
            parts["ff"] = PartSpec("dense", {"width": width, "inner": layer.mlp.ff, "activation": "squared_relu", "padded_rows": True},
                                   {role: name for name, _, _, role in _mlp_tensors(layer.mlp, index, width)})
        layers.append(LayerPlan("parallel", parts))
    runs = config.runs()
    enters_again = any(again for _, again in runs)
    if enters_again:                       # one part for every pass: it holds no tensors
        layers.append(LayerPlan("transform", {"transform": PartSpec("add_origin")}))
    # every run of a layer keeps a cache entry of its own, numbered in the order the runs come
    schedule = []
    for run, (index, again) in enumerate(runs):
        if again:
            schedule.append(ScheduleEntry(layer=len(config.layers), cache=None))
        schedule.append(ScheduleEntry(layer=index, cache=run))
    return ModelPlan(
        width=width, vocab_size=config.vocab, max_positions=2 ** 31 - 1,      # positions are angles: no table bounds them
        embedding=PartSpec("token_only", {"width": width, "vocab_size": config.vocab, "keep_origin": enters_again}, {"tokens": "embed"}),
        layers=layers, schedule=schedule, final_norm=norm("final.norm"),
        readout=PartSpec("linear_readout", {"width": width, "vocab_size": config.vocab}, {"weight": "head"}))


def contract(config: LoselixConfig) -> Contract:
    width = config.width
    tensors = [TensorSpec("embed", (config.vocab, width), "table")]
    for index, layer in enumerate(config.layers):
        tensors.append(TensorSpec(f"l{index}.norm1", (width,), "vector"))
        tensors += [TensorSpec(name, shape, layout) for name, shape, layout, _ in _mixer_tensors(layer, index, width)]
        if layer.mlp is not None:
            tensors += [TensorSpec(name, shape, layout) for name, shape, layout, _ in _mlp_tensors(layer.mlp, index, width)]
    tensors += [TensorSpec("final.norm", (width,), "vector"), TensorSpec("head", (config.vocab, width), "table")]
    return Contract(tensors=tensors, prefixes=("",), anchor="embed")


def init(config: LoselixConfig, generator):
    """Matrices N(0, 1/in), norms' scales around one, the maps' vectors around zero, the sigmoid weights' bias around the
    logarithm of a few hundred keys below zero."""

    def normal(shape, std, mean=0.0):
        return torch.randn(shape, generator=generator, dtype=torch.float32) * std + mean

    tensors = {}
    for spec in contract(config).tensors:
        leaf = spec.name.rsplit(".", 1)[-1]
        if spec.name == "embed":
            tensors[spec.name] = normal(spec.shape, 1.0)
        elif leaf in ("lq1", "lk1", "lq2", "lk2"):
            tensors[spec.name] = normal(spec.shape, 0.1)
        elif leaf == "pb":
            tensors[spec.name] = normal(spec.shape, 0.5, -4.0)
        elif spec.layout == "vector":
            tensors[spec.name] = normal(spec.shape, 0.1, 1.0)
        else:
            tensors[spec.name] = normal(spec.shape, 1.0 / math.sqrt(spec.shape[-1]))
    return tensors


FAMILY = register_family(Family(
    name="loselix", architectures=("Loselix",), model_types=("loselix",),
    config_class=LoselixConfig, plan=plan, contract=contract, init=init))
