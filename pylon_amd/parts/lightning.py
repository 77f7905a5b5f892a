"""Lightning attention: linear attention with a fixed decay per head on activated projections.

``[q; k; v; g] = W h`` in one product; ``silu`` on q, k and v (in the recurrence's kernels, rounded to the
model's element type); per request and head a float32 state ``S`` of ``head_dim x v_head_dim`` numbers goes
from token to token, ``S_t = decay S_{t-1} + k_t v_t^T``, ``o_t = S_t^T q_t``.  The heads' outputs stay
float32 until all of them together have been divided by their root mean square and multiplied by a weight
and by ``sigmoid(g)``; then the output projection.  The state lives in the request's state slot and starts
at zero."""
from __future__ import annotations

import torch

from ..config.specs import LightningAttentionSpec
from ..kernels import ops
from .base import Part, StateRequirement
from .registry import register_part
from .retention import CHUNKED_FROM


class LightningAttention(Part):
    def __init__(self, spec: LightningAttentionSpec, *, dtype: torch.dtype, device) -> None:
        super().__init__()
        if len(spec.decay) != spec.n_heads:
            raise ValueError(f"lightning attention needs one decay per head: {len(spec.decay)} for {spec.n_heads} heads")
        if not 1 <= spec.v_head_dim <= 256 or not 1 <= spec.head_dim <= 1024:
            raise ValueError("lightning attention takes heads of up to 1024 key and 256 value elements")
        self.spec = spec
        self.dtype = dtype
        qk, vg = spec.n_heads * spec.head_dim, spec.n_heads * spec.v_head_dim
        self.gate_off = 2 * qk + vg
        self.add_param("qkvg", (2 * qk + 2 * vg, spec.hidden_size), dtype, device)
        self.add_param("norm", (vg,), torch.float32, device, role="vector")
        self.add_param("out", (spec.hidden_size, vg), dtype, device)
        self.decay = torch.tensor(list(spec.decay), dtype=torch.float32).to(device)

    def cache_requirement(self) -> StateRequirement:
        spec = self.spec
        return StateRequirement((spec.n_heads, spec.head_dim, spec.v_head_dim), torch.float32)

    def decode_signature(self, rows: int, bound: int) -> tuple:
        return ("lightning_attention",)  # nothing of its launches depends on the requests' lengths

    def forward(self, h: torch.Tensor, ctx, cache, stores: bool) -> torch.Tensor:
        spec = self.spec
        if not stores:
            raise ValueError("a lightning attention layer cannot borrow another run's state")
        proj = ops.linear(h, self.params["qkvg"], out_dtype=self.dtype)
        # prompt portions of a bfloat16 model run 32 tokens at a time on the matrix cores; steps of
        # single tokens, float32 models and odd head sizes token by token
        chunked = (not ctx.decode_only and ctx.max_count >= CHUNKED_FROM and ops.retention_chunked_ok(
            self.dtype, dim=spec.head_dim, vdim=spec.v_head_dim, rot_dims=0))
        mixed = ops.retention_recurrent(
            proj, cache.state, self.decay, None, ctx.positions, ctx.row_start, ctx.row_slots, rows=ctx.rows,
            heads=spec.n_heads, dim=spec.head_dim, vdim=spec.v_head_dim, rot_dims=0, eps=spec.norm_eps, k_scale=1.0,
            chunked=chunked, max_count=ctx.max_count, form="lightning")
        mixed = ops.norm_gate(mixed, self.params["norm"], proj[:, self.gate_off:], spec.norm_eps)
        return ops.linear_for_residual(mixed, self.params["out"], out_dtype=self.dtype)


register_part("mixer", "lightning_attention", LightningAttention, replace=True)
