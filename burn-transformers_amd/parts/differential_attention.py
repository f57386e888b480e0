"""Differential attention: two softmax maps a head over the same values, the second taken off the first.

The mixer is ``rotary_attention`` with two query and two key parts a head.  q_weight has heads * 2 * dim rows and k_weight
kv_heads * 2 * dim, head by head as [map 1, map 2]; every part is turned by its position on its own.  With a1 and a2 the
outputs of a head's two maps, o = a1 - lambda * a2, o <- o / sqrt(mean(o^2) + eps) * (1 - diff) over the head's vdim
channels; lambda = exp(lambda_q1 . lambda_k1) - exp(lambda_q2 . lambda_k2) + diff is one number for the layer, formed once
when the part is built.  Parameters beyond those of ``rotary_attention``: diff.  Tensors beyond its own: lambda_q1,
lambda_k1, lambda_q2, lambda_k2 [dim].

A key head's two parts lie side by side in ONE cached head, [map 1 | map 2], with the values the maps share beside them,
and a head's queries go to the attention kernels as two queries, [q1 | 0] and [0 | q2], on that cached head: the values
are kept and read once for both maps.  Attention leaves 32-bit rows (a difference of nearly equal rows keeps its digits),
and one kernel takes the difference and its norm and writes the output projection's operand.
"""

import torch

from ..kernels import library as K
from .base import pad_columns
from .registry import register
from .rotary_attention import RotaryAttention


@register("mixer", "differential_attention")
class DifferentialAttention(RotaryAttention):
    maps = 2

    def __init__(self, params, tensors):
        if params.get("gate") or params.get("weights", "softmax") != "softmax":
            raise ValueError("differential attention: the maps are softmaxes, and no gate stands behind them")
        super().__init__(params, tensors)
        self.diff = float(params["diff"])
        lambdas = [tensors[name].double().flatten() for name in ("lambda_q1", "lambda_k1", "lambda_q2", "lambda_k2")]
        if any(v.numel() != self.dim for v in lambdas):
            raise ValueError(f"differential attention: the lambda vectors are {[v.numel() for v in lambdas]}, expected {self.dim} each")
        q1, k1, q2, k2 = lambdas
        self.weight_of_second = float(torch.exp((q1 * k1).sum()) - torch.exp((q2 * k2).sum())) + self.diff

    def output_matrix(self, out):
        """(the difference is written head by head without gaps)"""
        return pad_columns(out, self.operand_cols())

    def operand_cols(self):
        return (self.heads * self.vdim + 7) // 8 * 8          # zeros behind the heads, for 16-byte reads in both types

    def wide_output(self, dtype):
        return dtype == torch.bfloat16

    def kernel_modules(self, dtype):
        return tuple(super().kernel_modules(dtype)) + ("differential",)

    def attend(self, q, gate, kv, step):
        tokens = q.shape[0]
        rows = step.buffer("attention.maps", tokens, self.n_q, "float32")
        self.run_attention(q, rows, None, kv, step)
        mixed = self.last_operand(step, "attention.mixed", tokens, self.operand_cols(),
                                  K.Chunked.wanted(tokens) and self.chunk_major(step, tokens))
        K.differential(rows, self.heads, self.vdim, self.head_dim, self.weight_of_second, 1.0 - self.diff, self.eps, mixed)
        return mixed

    def chunk_major(self, step, rows):
        return step.dtype_is_bf16
