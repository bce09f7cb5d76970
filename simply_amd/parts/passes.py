"""What a loop over layers does to the residual stream before every pass:

    x <- W [x; x0] + step_t

with x0 the embedding's output and step_t a learned vector for the pass t = 0, 1, ...; the product reads the stream in
the activation type and leaves it in 32-bit, the vector is added in the kernel of the norm behind it."""
from __future__ import annotations

import torch

from ..kernels import ops
from ..registry import PASS_INPUTS
from .base import ParamSpec, PassInput, as_product_weight


@PASS_INPUTS.register("projected_with_embedding")
class ProjectedWithEmbedding(PassInput):
    def __init__(self, hidden_size: int, times: int):
        self.hidden_size, self.times = int(hidden_size), int(times)
        self.proj = self.step = None

    def param_specs(self):
        D = self.hidden_size
        return {"proj": ParamSpec((D, 2 * D)), "step": ParamSpec((self.times, D), role="vector", init="norm")}

    def load(self, tensors):
        self.proj, self.step = as_product_weight(tensors["proj"]), tensors["step"].contiguous()

    def forward(self, h, x0, number, ctx, next_norm):
        h = ops.gemm(ops.concat_rows(h, x0, ctx.dtype), self.proj, out_dtype=torch.float32)
        step = self.step[number].expand(h.shape[0], -1)
        if next_norm is not None and next_norm.fuses_sum:
            return h, next_norm.after_sum(h, step, 1.0, ctx.dtype)
        ops.residual_add_norm(step, h)
        return h, next_norm.forward(h, ctx.dtype) if next_norm is not None else None
