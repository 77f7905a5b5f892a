"""What happens to the residual stream ahead of a pass through layers that run several times:
``x <- W [x; x0] + step[t]``, ``x0`` the embedded tokens and ``t`` the number of the pass.

The output of the run before, if it is still to be added, joins the stream in the kernel that lays
``[x | x0]`` out in the activation type; the product's sums stay float32, because they are the new stream."""
from __future__ import annotations

import torch

from ..config.specs import PassEntrySpec
from ..kernels import ops
from .base import DepthMixed, Part, Scaled, summed
from .registry import register_part


class JoinEmbedding(Part):
    def __init__(self, spec: PassEntrySpec, *, dtype: torch.dtype, device) -> None:
        super().__init__()
        if spec.times < 1:
            raise ValueError("a stretch of layers runs at least once")
        self.spec = spec
        self.dtype = dtype
        self.add_param("join", (spec.dim, 2 * spec.dim), dtype, device)
        self.add_param("step", (spec.times, spec.dim), torch.float32, device, role="vector")

    def forward(self, resid: torch.Tensor, delta, embedded: torch.Tensor, t: int, ctx):
        factor = 1.0
        if isinstance(delta, Scaled) and not isinstance(delta, DepthMixed) and delta.scale is None and delta.bias is None:
            delta, factor = delta.value, delta.factor
        elif delta is not None and not isinstance(delta, torch.Tensor):
            delta = summed(delta)
        joined = ops.pass_join(resid, delta, embedded, self.dtype, factor=factor)
        product = ops.linear_for_residual(joined, self.params["join"], out_dtype=torch.float32)
        return ops.pass_begin(resid, product, self.params["step"][t]), None


register_part("pass", "join_embedding", JoinEmbedding, replace=True)
