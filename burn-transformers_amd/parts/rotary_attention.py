"""Causal self-attention whose queries and keys are normalised per head and turned by their
positions (rotary positions), with grouped heads over the paged cache.

Parameters (all from the plan): width, heads, kv_heads, dim (a query's and a key's head size), vdim
(a value's head size, which may differ), scale (multiplies q.k), eps (of the head norms), head_norm
(whether queries and keys are divided by their root mean square per head, times the scales
``q_norm`` / ``k_norm`` [dim] that all heads share; norm_scale False: without such scales), rot_dims (the first so many channels of every
query and key head are turned, channel i with channel i + rot_dims / 2, by the angle position *
f_i), rot_base (f_i = rot_base^(-2 i / rot_dims)), rot_scaling (None, or factor / low / high /
original: frequencies whose wavelength is beyond original / low are divided by factor, those whose
wavelength is below original / high are kept, and between the two the division is blended in
linearly in original / wavelength; or, with the keys factor / original / fast / slow, the schedule that
blends by a pair's INDEX: with turns(i) the index at which a wave turns that many times in ``original`` positions,
pairs up to turns(fast) are kept, pairs from turns(slow) on are divided by factor, a linear ramp over the index
between, and every sine and cosine is multiplied by 0.1 ln(factor) + 1), rot_pairing ("halves", the default: channel i with channel i + rot_dims / 2;
"neighbours": channel 2 i with channel 2 i + 1), norm_span ("head", the default; "whole": the root mean square
is taken over a token's whole query (key) projection before it is split into heads, and the scales ``q_norm`` /
``k_norm`` are [heads * dim] / [kv_heads * dim]), window, chunk and keep (which earlier keys a query sees, as in
``parts/attention.py``), taps (default 0; with taps > 0 every channel of the query, key and value projections
passes a short causal convolution over its sequence's tokens, tensors ``q_conv`` / ``k_conv`` / ``v_conv``
[channels, taps], the last tap meeting the current token, no bias, no activation, before norms and rotation;
the projections' last taps - 1 outputs are then a state of the sequence beside its keys and values).  Optional
tensors ``q_bias`` / ``k_bias`` / ``v_bias``: added in the projection.  Optional tensor ``sink`` [heads]: a learned logit per head that stands in the softmax's
denominator beside the keys', with no key and no value.  softcap (default 0: none; scores become softcap *
tanh(score / softcap) before the softmax); weights ("softmax", the default; "sigmoid": a visible key weighs
sigmoid(score + b), b the tensor ``score_bias`` [heads], and nothing is normalised over the keys); values
("projected", the default; "keys": the projected keys before norm and rotation, vdim = dim and no ``v_weight``);
temperature (None, or coef / every: queries times 1 + coef * ln(floor((position + 1) / every) + 1)); gate (None;
"head": a head's output times sigmoid of one row of the tensor ``gate_weight`` [heads, width] on the mixer's input;
"channel": every channel times its own, ``gate_weight`` [heads * vdim, width]).  Tensors: q_weight [heads * dim, width], k_weight [kv_heads * dim, width],
v_weight [kv_heads * vdim, width], out_weight [width, heads * vdim], no biases.

One step: ONE product with the projections (the gate's too) laid one behind the other leaves 32-bit sums; a
kernel normalises and turns the heads, writes the queries to a buffer and the keys (turned) and
values straight into the cache at each token's position; the framework's attention kernels read the
cache (and gate what they store); the output projection adds to the stream.  Beside another part that reads the
same rows the first product also carries that part's first projection in small steps (``carry``), and the output
projection may be joined with its last (``last_matrix``).  The cache keeps heads of one size, max(dim, vdim)
rounded up to what the kernels take, with zeros behind a head's own channels; the output
projection's columns are spread the same way, so the zeros meet zeros.
"""

import math

import torch

from ..cache.storage import StateSpec
from ..kernels import library as K
from .attention import CausalSelfAttention
from .base import Mixer, operand_columns, packed_for_stream, pad_columns, pad_rows
from .registry import register


def rotary_frequencies(dims, base, scaling=None):
    """f_i for i < dims / 2 (float64): base^(-2 i / dims), rescaled by ``scaling`` as the module's text says."""
    i = torch.arange(dims // 2, dtype=torch.float64)
    f = float(base) ** (-2.0 * i / dims)
    if scaling and "fast" in scaling:
        factor, original = float(scaling["factor"]), float(scaling["original"])
        # the (fractional) pair index whose wave turns ``turns`` times in ``original`` positions
        index = lambda turns: dims * math.log(original / (2.0 * math.pi * turns)) / (2.0 * math.log(float(base)))
        first = max(math.floor(index(float(scaling["fast"]))), 0)
        last = min(math.ceil(index(float(scaling["slow"]))), dims - 1)
        ramp = torch.clamp((i - first) / max(last - first, 0.001), 0.0, 1.0)
        f = f / factor * ramp + f * (1.0 - ramp)
    elif scaling:
        factor, low, high, original = (float(scaling[k]) for k in ("factor", "low", "high", "original"))
        wavelength = 2.0 * math.pi / f
        blend = (original / wavelength - low) / (high - low)
        between = (1.0 - blend) * f / factor + blend * f
        f = torch.where(wavelength < original / high, f, torch.where(wavelength > original / low, f / factor, between))
    return f


def rotary_amplitude(scaling=None):
    """The factor on every sine and cosine that goes with ``scaling``: 0.1 ln(factor) + 1 for the schedule that
    blends by index, 1 otherwise."""
    return 0.1 * math.log(float(scaling["factor"])) + 1.0 if scaling and "fast" in scaling else 1.0


@register("mixer", "rotary_attention")
class RotaryAttention(CausalSelfAttention):
    takes_deferred_norm = False          # (its first product leaves 32-bit sums; the rows come normalised)
    only_launches_kernels = True
    maps = 1                             # score maps a head: how many queries and key parts it has (see DifferentialAttention)

    def __init__(self, params, tensors):
        Mixer.__init__(self, params, tensors)
        p = params
        self.width, self.heads, self.kv_heads = p["width"], p["heads"], p["kv_heads"]
        self.dim, self.vdim = p["dim"], p["vdim"]
        self.scale, self.eps = float(p["scale"]), float(p.get("eps", 0.0))
        self.window, self.chunk = int(p.get("window") or 0), int(p.get("chunk") or 0)
        self.keep = int(p.get("keep") or 0)
        self.rot_dims = int(p.get("rot_dims") or 0)
        if self.heads % self.kv_heads != 0:
            raise ValueError(f"rotary attention: {self.heads} query heads cannot share {self.kv_heads} key/value heads")
        if self.rot_dims % 2 != 0 or self.rot_dims > self.dim:
            raise ValueError(f"rotary attention: {self.rot_dims} turned channels must be even and at most the head size {self.dim}")
        # columns of the queries, the keys and the values in the first product
        n_qk = (self.heads * self.maps * self.dim, self.kv_heads * self.maps * self.dim)
        self.values_from_keys = {"projected": False, "keys": True}[p.get("values", "projected")]
        n_v = 0 if self.values_from_keys else self.kv_heads * self.vdim
        if self.values_from_keys and (self.vdim != self.dim or self.maps != 1):
            raise ValueError(f"rotary attention: values that are the keys have the keys' size {self.dim}, not {self.vdim}")
        shapes = {"q_weight": (n_qk[0], self.width), "k_weight": (n_qk[1], self.width),
                  "out_weight": (self.width, self.heads * self.vdim)}
        if not self.values_from_keys:
            shapes["v_weight"] = (n_v, self.width)
        self.softcap = float(p.get("softcap") or 0.0)
        self.sigmoid = {"softmax": False, "sigmoid": True}[p.get("weights", "softmax")]
        if self.softcap < 0.0 or (self.sigmoid and self.softcap):
            raise ValueError("rotary attention: a cap on the scores is positive and goes with the softmax")
        if self.sigmoid:
            shapes["score_bias"] = (self.heads,)
        temperature = p.get("temperature")
        self.temperature = (float(temperature["coef"]), int(temperature["every"])) if temperature else None
        self.gate_kind = p.get("gate")
        self.gate_cols = {None: 0, "head": self.heads, "channel": self.heads * self.vdim}[self.gate_kind]
        if self.gate_cols:
            shapes["gate_weight"] = (self.gate_cols, self.width)
        self.neighbours = {"halves": False, "neighbours": True}[p.get("rot_pairing", "halves")]
        self.whole_norm = {"head": False, "whole": True}[p.get("norm_span", "head")]
        scaled = bool(p.get("norm_scale", True))
        if p.get("head_norm", True) and scaled:
            shapes.update(q_norm=(n_qk[0],), k_norm=(n_qk[1],)) if self.whole_norm else \
                shapes.update(q_norm=(self.dim,), k_norm=(self.dim,))
        if "sink" in tensors:
            shapes["sink"] = (self.heads,)
        self.taps = int(p.get("taps") or 0)
        projections = [(name, rows) for name, rows in (("q", n_qk[0]), ("k", n_qk[1]), ("v", n_v)) if rows]
        for name, rows in projections:
            if name + "_bias" in tensors:
                shapes[name + "_bias"] = (rows,)
            if self.taps:
                shapes[name + "_conv"] = (rows, self.taps)
        for role, shape in shapes.items():
            if tuple(tensors[role].shape) != shape:
                raise ValueError(f"rotary attention: {role} is {tuple(tensors[role].shape)}, expected {shape}")
        self.q_norm, self.k_norm = tensors.get("q_norm"), tensors.get("k_norm")
        if p.get("head_norm", True) and not scaled:           # the kernel multiplies by ones, which is exact
            q_scales, k_scales = n_qk if self.whole_norm else (self.dim, self.dim)
            self.q_norm, self.k_norm = (torch.ones(count, dtype=torch.float32, device=tensors["q_weight"].device)
                                        for count in (q_scales, k_scales))
        self.sink = tensors["sink"].float().contiguous() if "sink" in tensors else None
        self.score_bias = tensors["score_bias"].float().contiguous() if self.sigmoid else None
        dtype = tensors["q_weight"].dtype
        bf16 = dtype == torch.bfloat16
        # the cached head: the larger of the two head sizes, in the steps of 16 the MFMA kernels take
        self.head_dim = (max(self.maps * self.dim, self.vdim) + 15) // 16 * 16
        if max(self.dim, self.vdim) > 256:
            raise ValueError(f"rotary attention: heads of {max(self.dim, self.vdim)} are beyond 256, the most any kernel here takes")
        # the MFMA kernels take heads of up to 128 in bfloat16; larger ones run on the plain attention kernel
        self.plain_only = bf16 and self.head_dim > 128
        self.q_heads = self.heads * self.maps                   # queries the attention kernels see
        self.plain_decode = bf16 and self.q_heads // self.kv_heads > 16
        # ... but where all query heads share one cached head and the scores are an ordinary softmax's, both run on the
        # kernel for that
        self.shared_head = (self.plain_only or self.plain_decode) and self.kv_heads == 1 and not self.softcap and not self.sigmoid \
            and not self.wide_output(dtype)
        self.n_q, self.n_kv = self.q_heads * self.head_dim, self.kv_heads * self.head_dim
        self.fused_cols = n_qk[0] + n_qk[1] + n_v               # what a convolution passes over
        self.first_cols = self.fused_cols + self.gate_cols
        first = [tensors[name + "_weight"] for name, _ in projections] + ([tensors["gate_weight"]] if self.gate_cols else [])
        self.qkv_weight = pad_columns(torch.cat(first), operand_columns(self.width, dtype))
        self.out_weight = self.output_matrix(tensors["out_weight"])
        self.out_bias = None
        device = self.qkv_weight.device
        self.inv_freq = rotary_frequencies(self.rot_dims, p["rot_base"], p.get("rot_scaling")).to(torch.float32).to(device) \
            if self.rot_dims else None
        self.amplitude = rotary_amplitude(p.get("rot_scaling")) if self.rot_dims else 1.0
        self.qkv_bias = None
        if any(name + "_bias" in tensors for name in "qkv"):
            self.qkv_bias = torch.cat([tensors[name + "_bias"].float() if name + "_bias" in tensors
                                       else torch.zeros(rows, dtype=torch.float32, device=device)
                                       for name, rows in projections + [("gate", self.gate_cols)]]).contiguous()
        self.conv_weight, self.conv_state = None, 0
        if self.taps:
            self.conv_weight = torch.cat([tensors[name + "_conv"] for name, _ in projections]).float().contiguous()
            self.conv_state = (self.taps - 1) * self.fused_cols
            self.no_state = torch.zeros(1, 1, dtype=torch.float32, device=device)       # what one tap keeps: nothing
        on_gpu = self.qkv_weight.is_cuda
        self.qkv_packed = K.PackedWeight(self.qkv_weight) if on_gpu else None
        self.out_packed = packed_for_stream(self.out_weight) if on_gpu else None
        self.first_matrix, self.first_packed = None, None       # with another part's rows behind its own: see ``carry``

    def output_matrix(self, out):
        """The output projection as it reads heads of head_dim: its columns spread, zeros between them."""
        spread = out.new_zeros(self.width, self.heads, self.head_dim)
        spread[:, :, :self.vdim] = out.view(self.width, self.heads, self.vdim)
        return spread.view(self.width, self.heads * self.head_dim).contiguous()

    def wide_output(self, dtype):
        """Whether the attention kernels store 32-bit rows in a model of this type that keeps bfloat16 ones."""
        return False

    def kernel_modules(self, dtype):
        modules = tuple(super().kernel_modules(dtype))
        if self.softcap or self.sigmoid or self.gate_cols or self.wide_output(dtype):
            variant = "_sigmoid" if self.sigmoid else "_capped" if self.softcap else "_softmax"
            modules = tuple(name + variant for name in modules)
        if dtype == torch.bfloat16 and self.shared_head:
            modules += ("attention_shared",)
        return ("rotary",) + (("state_space",) if self.taps else ()) + modules

    def carry(self, weight, activation):
        if self.qkv_bias is not None or weight.shape[1] != self.qkv_weight.shape[1]:
            return None
        own = (self.first_cols + 3) // 4 * 4                    # (the product's epilogue works on four columns at a time)
        self.first_matrix = torch.cat([pad_rows(self.qkv_weight, own), weight]).contiguous()
        self.qkv_weight, self.first_cols, self.carried_activation = self.first_matrix[:own], own, activation
        if self.first_matrix.is_cuda:                           # small steps run the product of both
            self.qkv_packed, self.first_packed = None, K.PackedWeight(self.first_matrix)
        return self.first_matrix

    def last_matrix(self):
        matrix, self.out_weight, self.out_packed = self.out_weight, None, None
        return matrix

    def chunk_major(self, step, rows):
        return step.decode and step.dtype_is_bf16 and not self.runs_plain(step)

    def runs_plain(self, step):
        """(the bfloat16 decode kernel takes up to 16 query heads on a cached head; beyond, the plain kernel)"""
        return (self.plain_only or (self.plain_decode and step.decode)) and not self.shared_head

    def state_spec(self):
        return StateSpec((self.conv_state,), "float32") if self.conv_state else None

    def forward(self, h, step, memory, stream, carried=None):
        tokens = h.shape[0]
        if not memory.writes:
            raise ValueError("rotary attention: every run keeps a cache entry of its own")
        kv = memory.kv()
        first = fused = step.buffer("rotary.fused", tokens, self.first_cols, "float32")
        if carried is not None:
            K.gemm(h, self.first_matrix, K.epilogue_f32_act(fused, self.first_cols, carried, self.carried_activation),
                   packed=self.first_packed)
        else:
            K.gemm(h, self.qkv_weight, K.epilogue_f32(fused, self.qkv_bias), packed=self.qkv_packed)
        if self.taps:
            mixed_in_time = step.buffer("rotary.conv", tokens, self.fused_cols, "float32")
            K.causal_conv(fused, self.conv_weight, None, mixed_in_time, memory.state() if self.conv_state else self.no_state,
                          step, act="none")
            fused = mixed_in_time
        q = step.buffer("attention.q", tokens, self.n_q, step.dtype)
        K.head_rotary(fused, self.heads, self.kv_heads, self.dim, self.vdim, self.rot_dims, self.inv_freq,
                      self.q_norm, self.k_norm, self.eps, q, step.tok_seq, step.tok_pos, kv, step.dtype,
                      neighbours=self.neighbours, whole_norm=self.whole_norm, amplitude=self.amplitude, maps=self.maps,
                      values_from_keys=self.values_from_keys, temperature=self.temperature)
        gate = first[:, self.fused_cols:] if self.gate_cols else None
        mixed = self.attend(q, gate, kv, step)
        if self.joined is None:
            stream.add_product(step, mixed, self.out_weight, None, packed=self.out_packed)

    def attend(self, q, gate, kv, step):
        """The operand of the output projection."""
        tokens = q.shape[0]
        mixed = self.last_operand(step, "attention.mixed", tokens, self.n_q,
                                  K.Chunked.wanted(tokens) and self.chunk_major(step, tokens))
        self.run_attention(q, mixed, gate, kv, step)
        return mixed

    def run_attention(self, q, out, gate, kv, step):
        plain, partial = self.runs_plain(step), None
        runs, prompt_runs = (1, 1) if plain else (self.decode_runs(step, q.device), self.prompt_runs(step, q.device, self.q_heads))
        if runs > 1:
            partial = step.buffer("attention.partial", step.n_seqs * self.q_heads * runs, self.head_dim + 2, "float32")
        elif prompt_runs > 1:
            partial = step.buffer("attention.partial", q.shape[0] * self.q_heads * prompt_runs, self.head_dim + 2, "float32")
        args = K.attention_args(q, out, kv, step.tok_seq, step.tok_pos, step.seq_off, step.seq_start,
                                self.q_heads, step.n_seqs, step.max_count, self.scale, self.window, partial,
                                runs=prompt_runs if prompt_runs > 1 else None, chunk=self.chunk, keep=self.keep, sink=self.sink, softcap=self.softcap, sigmoid=self.sigmoid,
                                score_bias=self.score_bias, gate=gate, gate_dim=self.vdim if self.gate_kind == "channel" else 0)
        shared = self.shared_head and step.dtype_is_bf16 and (self.plain_only or step.decode)
        K.attention(args, step.dtype, step.decode, impl="plain" if plain else "shared" if shared else "auto")
