"""Causal attention through low-rank latents, with an optional output gate and an optional key part that is
turned by position and shared by all heads.

Parameters: width, heads, dim (query/key size per head), vdim (value size per head), q_rank,
kv_rank, scale (multiplies q.k), eps (of the two latent norms), window (default 0: every earlier key; else the
latest so many positions), keep (default 0: the first so many positions are seen beside the window), gate (how an
optional tensor ``gate`` acts: "channel", the default, or "head"), borrows (default false; true: the mixer has no
down_kv and kv_norm and attends over the latent and the turned key part that ANOTHER layer keeps, of the same kv_rank,
rot_dim and rotation; its run's schedule entry reads that layer's cache entry), rot_dim (default 0), rot_base, rot_scaling, rot_pairing ("neighbours", the default, or
"halves"; frequencies and pairing as in ``parts/rotary_attention.py``).  Tensors, all [out, in]:
down_q [q_rank, width], q_norm [q_rank], up_q [heads*(dim + rot_dim), q_rank] (per head its dim plain rows, then
its rot_dim turned rows), down_kv [kv_rank + rot_dim, width] (the latent's rows, then the shared turned key part's,
which is not normalised), kv_norm [kv_rank], up_k [heads*dim, kv_rank], up_v [heads*vdim, kv_rank], optional
gate [heads*vdim, width] ([heads, width]: one gate a head), out_weight [width, heads*vdim].

With rot_dim > 0 a head's score is q_plain . k_plain + turn(q_turned) . turn(k_shared): the cached head is
[c; turn(k_shared)], its values c with zeros behind, and the absorbed query of head i is
[up_k_i^T up_q_i,plain c_q; turn(up_q_i,turned c_q)], so the same one-head attention serves.

With c_q = rms_norm(down_q h) and c = rms_norm(down_kv h), head i has queries q_i = up_q_i c_q,
keys k_i = up_k_i c and values v_i = up_v_i c.  Both up-projections of c are linear, so
    q_i . k_i(j) = (up_k_i^T up_q_i c_q) . c(j)        and        sum_j p_j v_i(j) = up_v_i sum_j p_j c(j):
attention runs on the latent itself.  Only c is cached, as ONE shared head of size kv_rank whose
keys and values are the same vector, and the heads' queries against it are the grouped-query case
of the attention kernels (all heads of a token read each cached vector once).  The matrix
up_k_i^T up_q_i is formed once when the part is built (in float64, rounded to the products' type).

The same on the way out: out_weight_i up_v_i is formed once as well (``absorbs_values``: no gate, or one per head, and
a matrix that is not much larger for it), so that the output projection reads the attention's own result, gated head by
head where there is a gate.  A gate per channel stands between the two products and keeps them apart.

One step: a fused product [down_q; down_kv; gate] h (32-bit sums) -> the two norms, c straight into
the paged cache (a borrowing mixer: [down_q; gate] h and the one norm) -> absorbed queries (one product; in small steps
their turned parts are rotated in its epilogue, and a borrowing mixer's norm is folded into it) -> attention over the
cache -> per head up_v and sigmoid gate, where they are not absorbed -> output projection (the sublayer's output).
"""

import torch

from ..cache.storage import KVSpec
from ..kernels import library as K
from .attention import CausalSelfAttention, keys_in_reach
from .base import Mixer, compute_units, operand_columns, packed_for_stream, pad_columns, pad_rows
from .registry import register
from .rotary_attention import rotary_amplitude, rotary_frequencies


@register("mixer", "latent_attention")
class LatentAttention(Mixer):
    only_launches_kernels = True

    def __init__(self, params, tensors):
        super().__init__(params, tensors)
        p = params
        self.width, self.heads, self.dim, self.vdim = p["width"], p["heads"], p["dim"], p["vdim"]
        self.q_rank, self.kv_rank = p["q_rank"], p["kv_rank"]
        self.scale, self.eps = float(p["scale"]), float(p["eps"])
        self.window, self.rot_dim = int(p.get("window") or 0), int(p.get("rot_dim") or 0)
        self.keep, self.borrows = int(p.get("keep") or 0), bool(p.get("borrows"))
        self.neighbours = {"halves": False, "neighbours": True}[p.get("rot_pairing", "neighbours")]
        if self.rot_dim % 2 != 0:
            raise ValueError(f"latent attention: {self.rot_dim} turned channels must be even")
        self.gated, self.gate_span = "gate" in tensors, p.get("gate", "channel")
        gate_rows = {"channel": self.heads * self.vdim, "head": self.heads}[self.gate_span] if self.gated else 0
        shapes = {"down_q": (self.q_rank, self.width), "q_norm": (self.q_rank,),
                  "up_q": (self.heads * (self.dim + self.rot_dim), self.q_rank),
                  "down_kv": (self.kv_rank + self.rot_dim, self.width),
                  "kv_norm": (self.kv_rank,), "up_k": (self.heads * self.dim, self.kv_rank),
                  "up_v": (self.heads * self.vdim, self.kv_rank), "out_weight": (self.width, self.heads * self.vdim)}
        if self.gated:
            shapes["gate"] = (gate_rows, self.width)
        if self.borrows:
            del shapes["down_kv"], shapes["kv_norm"]
        for role, shape in shapes.items():
            if tuple(tensors[role].shape) != shape:
                raise ValueError(f"latent attention: {role} is {tuple(tensors[role].shape)}, expected {shape}")
        dtype = tensors["down_q"].dtype
        self.bf16 = dtype == torch.bfloat16
        # the cached head: the latent, padded to what the attention kernels take (zeros that meet zeros)
        self.head_dim = (self.kv_rank + self.rot_dim + 15) // 16 * 16
        if self.head_dim > 768:
            raise ValueError(f"latent attention: a cached head of {self.kv_rank} + {self.rot_dim} is beyond 768, the most any "
                             f"attention kernel here takes")
        # bfloat16: the ordinary kernels take heads of up to 128 and up to 16 query heads per cached head in decode steps, the
        # kernel for one shared head the others.  (float32: the tiled kernel up to 128, the plain one beyond)
        self.shared_only = self.bf16 and self.head_dim > 128
        self.shared_decode = self.bf16 and (self.shared_only or self.heads > 16)
        # segments of the fused first product, each padded so that the next starts where 16-byte loads may
        self.q_cols = operand_columns(self.q_rank, dtype)
        self.kv_offset = (self.q_rank + 3) // 4 * 4
        self.gate_offset = self.kv_offset + (0 if self.borrows else (self.kv_rank + self.rot_dim + 3) // 4 * 4)
        self.fused_cols = (self.gate_offset + gate_rows + 3) // 4 * 4
        self.fused_weight = torch.cat([pad_rows(tensors["down_q"], self.kv_offset)] +
                                      ([pad_rows(tensors["down_kv"], self.gate_offset - self.kv_offset)] if not self.borrows else []) +
                                      ([pad_rows(tensors["gate"], self.fused_cols - self.gate_offset)] if self.gated else []))
        # (the rows it multiplies carry zero columns where the width is no multiple of what 16-byte loads take)
        self.fused_weight = pad_columns(self.fused_weight, operand_columns(self.width, dtype))
        self.q_norm, self.kv_norm = tensors["q_norm"], None if self.borrows else tensors["kv_norm"]
        # absorbed queries: rows i * head_dim .. of W are up_k_i^T up_q_i  ([kv_rank, q_rank]), and behind them
        # the head's turned rows of up_q as they are
        up_q = tensors["up_q"].double().view(self.heads, self.dim + self.rot_dim, self.q_rank)
        up_k = tensors["up_k"].double().view(self.heads, self.dim, self.kv_rank)
        absorbed = torch.einsum("hdr,hdq->hrq", up_k, up_q[:, :self.dim])
        full = absorbed.new_zeros(self.heads, self.head_dim, self.q_cols)
        full[:, :self.kv_rank, :self.q_rank] = absorbed
        full[:, self.kv_rank:self.kv_rank + self.rot_dim, :self.q_rank] = up_q[:, self.dim:]
        device = tensors["down_q"].device
        self.inv_freq, self.amplitude = None, 1.0
        if self.rot_dim:
            self.inv_freq = rotary_frequencies(self.rot_dim, p["rot_base"], p.get("rot_scaling")).to(torch.float32).to(device)
            self.amplitude = rotary_amplitude(p.get("rot_scaling"))
        self.query_weight = full.view(self.heads * self.head_dim, self.q_cols).to(dtype).contiguous()
        self.n_q = self.heads * self.head_dim
        extra = self.heads * (self.head_dim - self.vdim) * self.width * tensors["out_weight"].element_size()
        self.absorbs_values = extra <= self.ABSORBED_BYTES and not (self.gated and self.gate_span == "channel")
        if self.absorbs_values:
            out = tensors["out_weight"].double().view(self.width, self.heads, self.vdim)
            up_v = tensors["up_v"].double().view(self.heads, self.vdim, self.kv_rank)
            full = out.new_zeros(self.width, self.heads, self.head_dim)
            full[:, :, :self.kv_rank] = torch.einsum("whv,hvr->whr", out, up_v)
            self.out_weight = full.view(self.width, self.n_q).to(dtype).contiguous()
        else:
            self.up_v = tensors["up_v"].contiguous()
            self.mixed_cols = operand_columns(self.heads * self.vdim, dtype)
            self.out_weight = pad_columns(tensors["out_weight"], self.mixed_cols)
        # what the query product's epilogue in small steps takes: neighbouring pairs within four columns
        self.turns_in_product = self.rot_dim > 0 and self.neighbours and self.kv_rank % 2 == 0
        # second copies for decode steps, which read the weights and little else
        on_gpu = self.fused_weight.is_cuda
        self.fused_packed = K.PackedWeight(self.fused_weight) if on_gpu else None
        self.query_packed = K.PackedWeight(self.query_weight) if on_gpu else None
        self.out_packed = packed_for_stream(self.out_weight) if on_gpu else None

    def kv_spec(self):
        return KVSpec(1, self.head_dim, self.window, keep=self.keep)

    def kernel_modules(self, dtype):
        names = ["latent"]
        variant = "_softmax" if self.gated and self.absorbs_values else ""        # (the form with an output stage)
        if dtype == torch.bfloat16:
            if self.shared_decode:
                names.append("attention_shared")
            if not self.shared_only:
                names.append(f"attention_bf16_hd{self.head_dim}{variant}")
        elif self.head_dim <= 128:
            names.append("attention_f32" + variant)
        return tuple(names)

    # the planning of a prompt's runs of keys is the ordinary attention's: one cached head, ``heads`` query heads
    kv_heads = 1
    chunk = 0
    plain_only = False

    def prompt_runs(self, step, device):
        if not self.shared_only:
            return CausalSelfAttention.prompt_runs(self, step, device)
        if step.decode:
            return 1
        # tiles of 32 (token, head) rows, a work-group each; a run keeps at least four blocks of keys
        tiles = -(-step.token_capacity * self.heads // 32) + step.n_seqs - 1
        keys = keys_in_reach(step.context_limit, self.window, 0, self.keep)
        return max(1, min(compute_units(device) // tiles, keys // 256, 16))

    def decode_runs(self, step, device):
        """Into how many runs a decode step's keys are cut.  All heads share one cached head, so a
        step has only as many work-groups as sequences unless the keys are cut, and they are cut much
        earlier than where every head brings keys of its own: from ``SPLIT_BYTES`` of a sequence's
        cached vectors on, into runs of at least ``RUN_BYTES``, as many as give every work-group a
        compute unit.  Planned for the step's class of context, like the ordinary attention's."""
        if not step.decode:
            return 1
        keys = keys_in_reach(step.context_limit, self.window, 0, self.keep)
        pair_bytes = keys * self.head_dim * 2 * (2 if step.dtype_is_bf16 else 4)
        if pair_bytes <= self.SPLIT_BYTES:
            return 1
        if not self.shared_decode:
            return max(1, min(compute_units(device) // step.n_seqs, pair_bytes // self.RUN_BYTES, 64))
        # The kernel for one shared head: a run of four blocks of 64 keys, or shorter ones up to eight runs.  Measured at heads
        # of 512 + 64, us a call with 1 / 4 / 8 / 16 / 32 runs (join included): 16 heads, 8 sequences of 544 keys 37 / 24 / 20,
        # of 4,096 230 / 70 / 43 / 34 / 38, 32 sequences of 2,048 119 / 44 / 35 / 44 / 61, one of 8,192 448 / 124 / 67 / 44 /
        # 40; 128 heads, 8 of 4,096 238 / 75 / 54 / 45 / 62, 32 of 2,048 125 / 59 / 71.
        rows = 64 if self.heads >= 64 else 32 if self.heads > 16 and self.head_dim <= 576 else 16      # of a work-group
        blocks = -(-keys // 64)
        return max(1, min(compute_units(device) // (step.n_seqs * -(-self.heads // rows)), max(blocks // 4, min(blocks, 8)), 64))

    SPLIT_BYTES = 128 << 10
    RUN_BYTES = 64 << 10
    # How much larger than out_weight the matrix with up_v absorbed may be: a decode step reads so much in less time than
    # the kernel takes that it saves (4 us), and a prompt of 2,048 tokens multiplies by it in less (23 us at 8 heads)
    ABSORBED_BYTES = 8 << 20

    def forward(self, h, step, memory, stream):
        tokens = h.shape[0]
        kv = memory.kv()
        fused = step.buffer("latent.fused", tokens, self.fused_cols, "float32")
        K.gemm(h, self.fused_weight, K.epilogue_f32(fused), packed=self.fused_packed)
        if memory.writes == self.borrows:
            raise ValueError("latent attention: a mixer keeps a cache entry of its own, or borrows and reads another layer's")
        q = step.buffer("latent.queries", tokens, self.n_q, step.dtype)
        self.make_queries(fused, q, kv, step)
        self.attend(fused, q, kv, step, stream)

    def make_queries(self, fused, q, kv, step):
        """The absorbed and turned queries into ``q``, and the latent of a mixer that keeps one into the cache."""
        tokens = q.shape[0]
        small = tokens <= 64 and (not self.rot_dim or self.turns_in_product)
        if self.borrows and small and step.dtype_is_bf16 and self.q_cols == self.q_rank and K.Normalized.worth_it(tokens, self.q_rank):
            c_q = K.Normalized(fused[:, :self.q_rank], self.q_norm, None, self.eps, "rms_norm")
        else:
            c_q = step.buffer("latent.query_latent", tokens, self.q_cols, step.dtype)
            K.latent_norm(fused, self.q_rank, self.kv_offset, 0 if self.borrows else self.kv_rank, self.q_norm, self.kv_norm, self.eps,
                          c_q, step.tok_seq, step.tok_pos, kv, step.dtype, rot_dim=0 if self.borrows else self.rot_dim,
                          inv_freq=self.inv_freq, neighbours=self.neighbours, amplitude=self.amplitude)
        if not self.rot_dim:
            K.gemm(c_q, self.query_weight, K.epilogue_store(q), packed=self.query_packed)
        elif self.turns_in_product and K.takes_two_kinds(c_q):
            K.gemm(c_q, self.query_weight, K.epilogue_turn(q, self.head_dim, self.kv_rank, self.rot_dim, self.inv_freq, step.tok_pos,
                                                           self.amplitude), packed=self.query_packed)
        else:                    # the turned part of every head is rotated from the 32-bit sums
            sums = step.buffer("latent.query_sums", tokens, self.n_q, "float32")
            K.gemm(c_q, self.query_weight, K.epilogue_f32(sums), packed=self.query_packed)
            K.latent_query(sums, self.heads, self.head_dim, self.kv_rank, self.rot_dim, self.inv_freq, step.tok_pos, q,
                           neighbours=self.neighbours, amplitude=self.amplitude)

    def attend(self, fused, q, kv, step, stream):
        tokens = q.shape[0]
        gate = fused[:, self.gate_offset:] if self.gated else None
        if self.absorbs_values and step.decode and step.dtype_is_bf16 and K.Chunked.wanted(tokens):
            ctx = K.Chunked.take(step, "latent.context", tokens, self.n_q, step.dtype)       # read by the next product only
        else:
            ctx = step.buffer("latent.context", tokens, self.n_q, step.dtype)
        partial, runs, prompt_runs = None, self.decode_runs(step, q.device), self.prompt_runs(step, q.device)
        if runs > 1:
            partial = step.buffer("attention.partial", step.n_seqs * self.heads * runs, self.head_dim + 2, "float32")
        elif prompt_runs > 1:
            partial = step.buffer("attention.partial", tokens * self.heads * prompt_runs, self.head_dim + 2, "float32")
        args = K.attention_args(q, ctx, kv, step.tok_seq, step.tok_pos, step.seq_off, step.seq_start, self.heads,
                                step.n_seqs, step.max_count, self.scale, self.window, partial,
                                runs=prompt_runs if prompt_runs > 1 else None, keep=self.keep, gate=gate if self.absorbs_values else None,
                                value_dim=(self.kv_rank + 3) // 4 * 4)
        shared = self.shared_only or (self.shared_decode and step.decode)
        K.attention(args, step.dtype, step.decode, impl="shared" if shared else "auto")
        if self.absorbs_values:
            stream.add_product(step, ctx, self.out_weight, packed=self.out_packed)
            return
        mixed = step.buffer("latent.mixed", tokens, self.mixed_cols, step.dtype)
        K.head_project(ctx, self.up_v, self.heads, self.vdim, self.kv_rank, self.head_dim, mixed, gate=gate, gate_span=self.gate_span)
        stream.add_product(step, mixed, self.out_weight, packed=self.out_packed)
