"""Norms of the residual stream. RMS norm: y = x * rsqrt(mean(x^2) + eps) * weight (flow_engine/model.py:15-23).

The residual stream it reads is float32; statistics and products are float32
and the result is rounded once to the compute type. The weight is held in
float32 (exact for a bfloat16 checkpoint).
"""
from __future__ import annotations

from ..kernels import ops
from ..weights.spec import NORMAL, VECTOR, ONE_PLUS_NORMAL, TensorSpec
from .base import Norm


class RMSNorm(Norm):
    folds_pending = True

    def __init__(self, name, size, eps, suffix=".weight", offset=0.0):
        """offset: what the stored weight is to be increased by (1.0 for checkpoints that keep their norm weights
        around zero, y = unit(x) * (1 + w)); the sum is formed once, in float32, when the weights are bound."""
        self.offset = float(offset)
        self.name = name
        self.suffix = suffix              # what follows the name in the checkpoint
        self.size = int(size)
        self.eps = float(eps)
        self.weight = None

    def tensor_specs(self):
        return [TensorSpec(self.name + self.suffix, (self.size,), VECTOR, NORMAL if self.offset == 1.0 else ONE_PLUS_NORMAL)]

    def bind(self, tensors, dtype, device):
        self.weight = tensors.pop(self.name + self.suffix).contiguous()
        if self.offset:
            self.weight = (self.weight + self.offset).contiguous()

    def weight_tensors(self):
        return [self.weight]

    def forward(self, ctx, x, rows=None, add=None):
        tag = "norm.out" if rows is None else "norm.rows"        # a model's last norm (chosen rows) keeps its own buffer
        n_out = rows.numel() if rows is not None else x.shape[0]
        out = ctx.scratch(tag, (n_out, self.size))
        scratch = None
        if add is not None and rows is not None:
            import torch
            scratch = ctx.scratch(tag + ".rows", (n_out, self.size), torch.float32)
        return ops.rmsnorm(x, self.weight, self.eps, out, rows=rows, add=add, row_scratch=scratch)


class LayerNorm(Norm):
    """y = (x - mean) / sqrt(mean((x - mean)^2) + eps) * weight + bias, in float32, rounded once to the compute type."""
    folds_pending = True

    def __init__(self, name, size, eps, suffixes=(".weight", ".bias")):
        self.name, self.suffixes = name, tuple(suffixes)         # what follows the name in the checkpoint
        self.size, self.eps = int(size), float(eps)
        self.weight = self.bias = None

    def tensor_specs(self):
        w, b = (self.name + s for s in self.suffixes)
        return [TensorSpec(w, (self.size,), VECTOR, ONE_PLUS_NORMAL), TensorSpec(b, (self.size,), VECTOR, NORMAL)]

    def bind(self, tensors, dtype, device):
        self.weight, self.bias = (tensors.pop(self.name + s).contiguous() for s in self.suffixes)

    def weight_tensors(self):
        return [self.weight, self.bias]

    @property
    def pair(self):
        return self.weight, self.bias

    def forward(self, ctx, x, rows=None, add=None):
        tag = "norm.out" if rows is None else "norm.rows"        # a model's last norm (chosen rows) keeps its own buffer
        out = ctx.scratch(tag, (rows.numel() if rows is not None else x.shape[0], self.size))
        return ops.layer_norm(x, self.eps, add=add, norm=self.pair, out=out, rows=rows)
