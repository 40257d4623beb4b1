"""What happens to the residual stream ahead of a pass through a run of layers.

``concat_projection``: ``x <- W [x | x0]``, x0 being the embedding's output: the layers of the run see, in
every pass, what the pass before made of the stream blended with where it came from.  The stream, with what is
pending on it, and x0 lie side by side in the compute dtype (x0 is put there once a step); the product's float32 result
is the new stream (its first part, with the other parts pending, where it comes in partial sums over K).

``pass_vectors``: ``x <- x + x0 + s_t`` ahead of pass t (in the first pass without x0), s_t a learned vector of the
pass.  Both are left pending on the stream, beside the update of the layer before, for the kernel of the next norm.
"""

from __future__ import annotations

import torch
from torch import Tensor

from ..kernels import ops
from ..registry import register_part
from .base import BuildContext, ParamSpec, Residual, StreamEntry


class ConcatProjection(StreamEntry):
    CARRY = "stream entry"

    def __init__(self, ctx: BuildContext, prefix: str, *, hidden_size: int, leaf: str = "weight") -> None:
        super().__init__(ctx, prefix)
        self.hidden_size = hidden_size
        self.leaf = leaf
        self.weight: Tensor | None = None

    def param_specs(self):
        return {self.name(self.leaf): ParamSpec((self.hidden_size, 2 * self.hidden_size))}

    def set_param(self, name: str, tensor: Tensor) -> None:
        if name != self.name(self.leaf):
            raise KeyError(name)
        self.weight = tensor

    def begin(self, residual: Residual, batch) -> None:
        h = residual.flush()
        pair = torch.empty((h.shape[0], 2 * self.hidden_size), dtype=self.ctx.dtype, device=h.device)
        batch.carry[self.CARRY] = pair
        ops.stream_sum_cast(h, None, None, pair[:, self.hidden_size:])

    def forward(self, residual: Residual, batch, number: int = 0) -> None:
        if residual.streams is not None or residual.pending_norm is not None:
            residual.flush()
        pair = batch.carry[self.CARRY]
        update, bias = residual.take_biased()
        ops.stream_sum_cast(residual.h, update, bias, pair[:, :self.hidden_size])
        fresh = ops.linear_update(pair, self.weight)
        if fresh.dim() == 2:
            residual.replace(fresh)
        else:
            residual.replace(fresh[0], fresh[1:] if fresh.shape[0] > 1 else None)

    def kernel_libraries(self):
        return {"stream_ops", "gemm_f32", "gemm_skinny", "gemm_mid", "gemm_wide"}


class PassVectors(StreamEntry):
    CARRY = "stream entry"

    def __init__(self, ctx: BuildContext, prefix: str, *, hidden_size: int, passes: int, leaf: str = "step") -> None:
        super().__init__(ctx, prefix)
        self.hidden_size, self.passes, self.leaf = hidden_size, passes, leaf
        self.steps: Tensor | None = None       # [passes, hidden]

    def param_specs(self):
        return {self.name(self.leaf): ParamSpec((self.passes, self.hidden_size), kind="vector", init="unit")}

    def set_param(self, name: str, tensor: Tensor) -> None:
        if name != self.name(self.leaf):
            raise KeyError(name)
        self.steps = tensor.contiguous()

    def begin(self, residual: Residual, batch) -> None:
        if self.passes < 2:
            return
        h = residual.flush()
        batch.carry[self.CARRY] = ops.stream_sum_cast(h, None, None, torch.empty_like(h))     # the stream itself changes in place

    def forward(self, residual: Residual, batch, number: int = 0) -> None:
        if not 0 <= number < self.passes:
            raise ValueError(f"{self.prefix}: pass {number} of {self.passes}")
        residual.join(batch.carry[self.CARRY] if number else None, self.steps[number])

    def kernel_libraries(self):
        return {"stream_ops", "rowwise"}


register_part("entry", "concat_projection", ConcatProjection)
register_part("entry", "pass_vectors", PassVectors)
