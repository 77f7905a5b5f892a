"""Gated linear attention: linear attention with a learned, input-dependent decay per key channel, no
softmax and no denominator.

``[q; k; v; g; a] = W h`` in one product; ``q`` times ``head_dim ** -0.5``; a key channel's decay is
``sigmoid(W_a2 a + b) ** (1 / tau)`` (``a`` has ``decay_rank`` numbers); per request and head a float32
state goes from token to token, ``S_t = diag(alpha_t) S_{t-1} + k_t v_t^T``, ``o_t = S_t^T q_t``; every
head's ``o`` is divided by its root mean square, multiplied by a weight shared by the heads and by
``silu(g)``, and projected.  The state lives in the request's state slot and starts at zero; decays (with
their logarithms and ``W_a2``), state, norm and gate are computed in float32 whatever the model's element
type."""
from __future__ import annotations

import torch

from ..config.specs import GatedLinearAttentionSpec
from ..kernels import ops
from .base import Part, StateRequirement
from .registry import register_part


class GatedLinearAttention(Part):
    def __init__(self, spec: GatedLinearAttentionSpec, *, dtype: torch.dtype, device) -> None:
        super().__init__()
        if not ops.gla_ok(spec.head_dim, spec.v_head_dim):
            raise ValueError(f"gated linear attention does not take heads of {spec.head_dim} x {spec.v_head_dim} elements")
        if spec.decay_rank < 1 or not spec.tau > 0:
            raise ValueError("gated linear attention needs a positive decay_rank and tau")
        self.spec = spec
        self.dtype = dtype
        qk, vg = spec.n_heads * spec.head_dim, spec.n_heads * spec.v_head_dim
        self.add_param("proj", (2 * qk + 2 * vg + spec.decay_rank, spec.hidden_size), dtype, device)
        self.add_param("a2", (qk, spec.decay_rank), torch.float32, device, role="vector")
        self.add_param("a2_bias", (qk,), torch.float32, device, role="vector")
        self.add_param("norm", (spec.v_head_dim,), torch.float32, device, role="vector")
        self.add_param("out", (spec.hidden_size, vg), dtype, device)

    def cache_requirement(self) -> StateRequirement:
        spec = self.spec
        return StateRequirement((spec.n_heads, spec.head_dim, spec.v_head_dim), torch.float32)

    def decode_signature(self, rows: int, bound: int) -> tuple:
        return ("gated_linear_attention",)  # nothing of its launches depends on the requests' lengths

    def forward(self, h: torch.Tensor, ctx, cache, stores: bool) -> torch.Tensor:
        spec = self.spec
        if not stores:
            raise ValueError("a gated linear attention layer cannot borrow another run's state")
        proj = ops.linear(h, self.params["proj"], out_dtype=self.dtype)
        mixed = ops.gla(
            proj, cache.state, self.params["a2"], self.params["a2_bias"], self.params["norm"], ctx.row_start,
            ctx.row_slots, rows=ctx.rows, heads=spec.n_heads, dim=spec.head_dim, vdim=spec.v_head_dim,
            rank=spec.decay_rank, tau=spec.tau, eps=spec.norm_eps, q_scale=spec.head_dim ** -0.5,
            max_count=ctx.max_count)
        return ops.linear_for_residual(mixed, self.params["out"], out_dtype=self.dtype)


register_part("mixer", "gated_linear_attention", GatedLinearAttention, replace=True)
