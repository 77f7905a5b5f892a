"""Latent attention: softmax attention whose keys and values are linear maps of one small latent
per token, which is all that the cache keeps.

``[c_q'; c'; g] = W_down h`` in one product (float32 sums); ``c_q = norm(c_q')``, ``c = norm(c')``
(root mean square over the latent, times a weight) and ``sigmoid(g)`` in one kernel, which also
puts ``c`` into the token's cache slot; ``q = W_uq c_q``.  Per head ``k_j = W_uk c_j`` and
``v_j = W_uv c_j``, so ``q . k_j = (W_uk^T q) . c_j`` and ``sum_j p_j v_j = W_uv (sum_j p_j c_j)``:
the queries are carried into the latent's space head by head, attention runs over the cached
latents themselves (one key/value head that all query heads share, keys and values the same
tensor), and the result is carried to the value space head by head, multiplied by the gate.
The mask is a sliding window, chunks, or plain causal.

Without a query latent (``q_rank`` None) the one product is ``[q; c'; r'; g]``, and a part of every
query may carry the token's position: with ``rot_dim`` a head of q is ``[q_u | q_r]``, ``q_r`` and one
key part ``r'`` shared by all heads are rotated, and ``q . k_j = q_u . (W_uk c_j) + q_r . r_j = [W_uk^T
q_u | q_r] . [c_j | r_j]``: still one product over a row of the cache, whose first ``kv_rank`` elements
are the values.  The softmax may have a learned sink per head; the gate is one number per head or per
element.

The cache is ``[pages, page_size, 1, kv_rank + rot_dim]`` per run (``KVRequirement(values=False)``).
Without a rotated part and a sink, bfloat16 steps over latents of 64, 128 or 256 numbers run on the
matrix-core attention kernels (for a step of single tokens the heads are handed to the decode kernel
in groups of at most 16, each group as a query token of its own).  With them, bfloat16 steps over
pages of a multiple of 64 tokens run on kernels of their own (``attention_latent.hip``) that bring a block
of rows into LDS once and read it as keys and as values.  Everything else runs on the general kernel.
"""
from __future__ import annotations

import torch

from ..config.specs import LatentAttentionSpec
from ..kernels import ops
from .base import KVRequirement, Part
from .registry import build_part, register_part


def head_group(n_heads: int, most: int = 16) -> int:
    """The largest divisor of ``n_heads`` that is at most ``most``."""
    return max(g for g in range(1, min(n_heads, most) + 1) if n_heads % g == 0)


class LatentAttention(Part):
    def __init__(self, spec: LatentAttentionSpec, *, dtype: torch.dtype, device) -> None:
        super().__init__()
        for name in ("n_heads", "head_dim", "v_head_dim", "kv_rank"):
            if getattr(spec, name) < 1:
                raise ValueError(f"latent attention: {name} must be positive")
        if spec.q_rank is not None and spec.q_rank < 1:
            raise ValueError("latent attention: q_rank must be positive (or None)")
        if spec.rot_dim < 0 or spec.rot_dim % 2 or spec.rot_dim > 512:
            raise ValueError("latent attention: rot_dim must be even, at most 512")
        if spec.q_rank is not None and (spec.rot_dim or spec.gate_over != "head"):
            raise ValueError("a rotated part and gates per element go with queries straight from the input")
        if spec.kv_rank > 512:
            raise ValueError(f"a latent of {spec.kv_rank} numbers is not supported: the attention kernels take up to 512")
        if spec.window is not None and spec.window < 1:
            raise ValueError("window must be positive (or None)")
        if spec.chunk is not None and (spec.chunk < 1 or spec.window is not None):
            raise ValueError("chunk must be positive, and a layer has a window or chunks, not both")
        if spec.gate_over not in ("head", "element"):
            raise ValueError(f"gate_over must be 'head' or 'element', got {spec.gate_over!r}")
        self.spec = spec
        self.dtype = dtype
        self.n_gate = spec.gate_size
        # the rows of the one product over the input: q (or its latent), the latent, the shared rotated
        # key part, the gate
        self.q_rows = spec.n_heads * (spec.head_dim + spec.rot_dim) if spec.q_rank is None else spec.q_rank
        self.gate_off = self.q_rows + spec.kv_rank + spec.rot_dim
        self.width = spec.kv_rank + spec.rot_dim  # a row of the cache
        self.add_param("down", (self.gate_off + self.n_gate, spec.hidden_size), dtype, device)
        self.add_param("c_norm", (spec.kv_rank,), torch.float32, device, role="vector")
        if spec.q_rank is not None:
            self.add_param("q_norm", (spec.q_rank,), torch.float32, device, role="vector")
            self.add_param("uq", (spec.n_heads * spec.head_dim, spec.q_rank), dtype, device)
        self.add_param("uk", (spec.n_heads * spec.head_dim, spec.kv_rank), dtype, device)
        self.add_param("uv", (spec.n_heads * spec.v_head_dim, spec.kv_rank), dtype, device)
        self.add_param("out", (spec.hidden_size, spec.n_heads * spec.v_head_dim), dtype, device)
        if spec.sink:
            self.add_param("sink", (spec.n_heads,), torch.float32, device, role="vector")
        self.position = None
        if spec.rot_dim and spec.position is not None:
            self.position = self.add_child("position", build_part("position", spec.position, dtype=dtype, device=device))
            rotary = self.position.rotary()
            if rotary is not None and rotary[1] != spec.rot_dim:
                raise ValueError(f"latent attention rotates its whole part of {spec.rot_dim} elements, not {rotary[1]}")
        self._turned = {}  # parameter -> (its version, it with the last two axes of every head exchanged)

    def cache_requirement(self) -> KVRequirement:
        spec = self.spec
        return KVRequirement(1, self.width, spec.window, chunk=spec.chunk, values=False)

    def _map(self, name: str, rows: int) -> torch.Tensor:
        """A per-head matrix as it is stored, ``[heads, rows, kv_rank]``."""
        return self.params[name].view(self.spec.n_heads, rows, self.spec.kv_rank)

    def _map_turned(self, name: str, rows: int) -> torch.Tensor:
        """The same with the latent's axis first inside every head, ``[heads, kv_rank, rows]``; made anew
        when the parameter has been written."""
        param = self.params[name]
        key = (param.data_ptr(), param._version, param.dtype)
        if name not in self._turned or self._turned[name][0] != key:
            self._turned[name] = (key, self._map(name, rows).transpose(1, 2).contiguous())
        return self._turned[name][1]

    def _into_latent(self, q: torch.Tensor, out=None) -> torch.Tensor:
        """The queries' unrotated parts in the latent's space, ``q'_h = W_uk[h]^T q_h``."""
        dim = self.spec.head_dim
        return ops.head_project(q, self._map("uk", dim), out=out, by_output=self._map_turned("uk", dim))

    def _into_values(self, mixed: torch.Tensor, **gating) -> torch.Tensor:
        """Every head's weighted latent in its value space, ``W_uv[h] c``, times the gate."""
        dim = self.spec.v_head_dim
        return ops.head_project(mixed, self._map_turned("uv", dim), by_output=self._map("uv", dim), **gating)

    def _span(self, bound: int) -> int:
        limit = self.spec.window if self.spec.window is not None else self.spec.chunk
        return bound if limit is None else min(bound, limit)

    def _decode_launch(self, queries: int, span: int) -> tuple:
        """(cuts, waves) of the decode kernel for ``queries`` query tokens (a group of heads each) over
        one shared key/value head: with so few workgroups a request's latents are cut over workgroups
        down to 128 a cut, until the workgroups fill the chip."""
        units = ops.compute_units()
        cuts = 1
        while cuts < 64 and queries * cuts * 2 <= units and cuts * 2 * 128 <= span:
            cuts *= 2
        return cuts, ops.decode_splits(queries * cuts, 1, -(-span // cuts), units)

    def _group(self) -> int:
        """Query heads that go to the decode kernel as one query token.  It takes up to 16, but over
        latents of 256 numbers it is faster with 8 (8 requests, 32 heads, a window of 1,024: 38.7 us
        in groups of 16 over 8 cuts, 17.4 in groups of 8)."""
        return head_group(self.spec.n_heads, 8 if self.spec.kv_rank >= 256 else 16)

    def _matrix_cores(self) -> bool:
        spec = self.spec
        return (self.dtype == torch.bfloat16 and spec.kv_rank in ops.DECODE_HEAD_DIMS and not spec.rot_dim
                and not spec.sink)

    def decode_signature(self, rows: int, bound: int) -> tuple:
        if not self._matrix_cores():
            # over whole cache rows (whatever the page's size, which this does not know) the keys' cuts
            return ("latent_attention", ops.latent_cuts(rows, self.spec.n_heads, self._span(bound)))
        group = self._group()
        return ("latent_attention",) + tuple(self._decode_launch(rows * (self.spec.n_heads // group), self._span(bound)))

    def _row_kernels(self, page_size: int) -> bool:
        """Whether the matrix-core kernels over whole cache rows (a key with its value at the front) run."""
        spec = self.spec
        return bool(spec.rot_dim or spec.sink) and ops.latent_attention_ok(
            self.dtype, width=self.width, rank=spec.kv_rank, page_size=page_size)

    def forward(self, h: torch.Tensor, ctx, cache, stores: bool) -> torch.Tensor:
        spec = self.spec
        tokens = h.shape[0]
        heads, rank = spec.n_heads, spec.kv_rank
        gating = {}
        if spec.q_rank is None:
            q, gating["gate_logits"] = self._queries(h, ctx, cache, stores)
        else:
            down = ops.linear(h, self.params["down"], out_dtype=torch.float32)
            q_latent, gating["gate"] = ops.latent_prepare(
                down, cache.k if stores else None, cache.slot_map if stores else None, q_rank=spec.q_rank,
                kv_rank=rank, n_gate=self.n_gate, q_weight=self.params["q_norm"], c_weight=self.params["c_norm"],
                eps=spec.norm_eps, out_dtype=self.dtype)
            q = ops.linear(q_latent, self.params["uq"], out_dtype=self.dtype)
            q = self._into_latent(q.view(tokens, heads, spec.head_dim))
        mixed = self._attend(q, ctx, cache)
        context = self._into_values(mixed, **gating)
        return ops.linear_for_residual(context.view(tokens, heads * spec.v_head_dim), self.params["out"],
                                       out_dtype=self.dtype)

    def _queries(self, h: torch.Tensor, ctx, cache, stores: bool):
        """``(queries in the cache rows' space [tokens, heads, kv_rank + rot_dim], the gate's logits or
        None)`` of queries that come straight from the input; the tokens' rows go into the cache."""
        spec = self.spec
        tokens, heads, rank = h.shape[0], spec.n_heads, spec.kv_rank
        proj = ops.linear(h, self.params["down"], out_dtype=self.dtype)
        q = torch.empty((tokens, heads, self.width), dtype=self.dtype, device=h.device)
        rotary = self.position.rotary() if self.position is not None else None
        ops.latent_rotate(
            proj, q, cache.k if stores else None, cache.slot_map if stores else None, q_off=0, n_heads=heads,
            head_dim=spec.head_dim, rot_dim=spec.rot_dim, c_off=self.q_rows, kv_rank=rank, c_weight=self.params["c_norm"],
            eps=spec.norm_eps, inv_freq=rotary[0] if rotary else None,
            rot_scale=self.position.rot_scale if rotary else 1.0,
            interleaved=self.position.interleaved if rotary else True, positions=ctx.positions)
        unrotated = proj[:, : self.q_rows].view(tokens, heads, spec.head_dim + spec.rot_dim)[..., : spec.head_dim]
        self._into_latent(unrotated, out=q[..., :rank])
        return q, proj[:, self.gate_off:] if self.n_gate else None

    def _attend(self, q: torch.Tensor, ctx, cache) -> torch.Tensor:
        """``[tokens, heads, kv_rank]``: every head's weighted sum of its request's latents."""
        spec = self.spec
        tokens, heads, width = q.shape
        rank = spec.kv_rank
        mask = dict(window=spec.window, chunk=spec.chunk)
        latents = cache.k  # [pages, page_size, 1, kv_rank + rot_dim]: keys, and values at their front
        group = self._group()
        repeat = heads // group
        if self._matrix_cores() and q.dtype == latents.dtype and ctx.decode_only \
                and tokens * repeat <= ops.DECODE_MAX_TOKENS:
            positions, rows = ctx.positions, None
            if repeat > 1:  # every group of heads a query token of its own, on its request's row of the table
                key = ("latent_attention.groups", repeat)
                if key not in ctx.memo:  # once a step, not once a layer
                    ctx.memo[key] = (ctx.positions.repeat_interleave(repeat), ctx.tok_row.repeat_interleave(repeat))
                positions, rows = ctx.memo[key]
            cuts, splits = self._decode_launch(tokens * repeat, self._span(ctx.max_len))
            return ops.attention_decode(
                q.view(tokens * repeat, group, rank), latents, latents, cache.block_table, rows, positions,
                page_size=cache.page_size, scale=spec.scale, n_splits=splits, n_cuts=cuts, **mask,
            ).view(tokens, heads, rank)
        if self._matrix_cores() and q.dtype == latents.dtype and ops.prefill_attention_ok(q, latents, cache.block_table):
            rows = ops.prefill_rows(tokens, heads, heads)
            mixed = torch.empty_like(q)
            tiles = ctx.token_tiles(rows // heads, fold=ops.prefill_fold(1))
            return ops.attention_prefill(q, latents, latents, cache.block_table, tiles, page_size=cache.page_size,
                                         scale=spec.scale, rows=rows, out=mixed, **mask)
        if self._row_kernels(cache.page_size) and q.dtype == latents.dtype:
            options = dict(rank=rank, page_size=cache.page_size, scale=spec.scale, sink=self.params.get("sink"), **mask)
            rows = ops.latent_rows(heads, rank)
            # decoding requests at the head of a step go to the kernel of single tokens
            singles = tokens if ctx.decode_only else (ctx.leading_singles if rows else 0)
            if singles == tokens or rows:
                mixed = torch.empty((tokens, heads, rank), dtype=self.dtype, device=q.device)
                if singles:
                    length = ctx.max_len if ctx.decode_only else int(ctx.starts[:singles].max()) + 1
                    ops.latent_decode(q[:singles], latents, cache.block_table, ctx.positions[:singles],
                                      cuts=ops.latent_cuts(singles, heads, self._span(length)), out=mixed[:singles], **options)
                if singles < tokens:
                    tiles = ctx.token_tiles(rows // heads, skip_rows=singles, fold=ops.prefill_fold(1))
                    ops.latent_prefill(q, latents, cache.block_table, tiles, rows=rows, out=mixed, **options)
                return mixed
        return ops.paged_attention(q, latents, latents, cache.block_table, ctx.tok_row, ctx.positions,
                                   page_size=cache.page_size, scale=spec.scale, values_in_keys=rank,
                                   sink_logit=self.params.get("sink"), **mask)


register_part("mixer", "latent_attention", LatentAttention, replace=True)
