"""A decoder assembled from parts, and its one forward pass: the step.

The model is architecture-blind: it builds one block per :class:`LayerSpec`, runs the
blocks in the order the schedule lists them, and applies the final norm and the
vocabulary head only at the tokens whose logits are wanted
(/root/reference/src/pylon/model/model.py:124-144).  What an architecture does outside
its layers goes into two optional lists of parts: "stream" parts between the embedding and
the first layer (``forward(resid, ctx) -> resid``, the float32 residual stream of the step's
tokens), "logits" parts after the head (``forward(logits, ctx) -> logits``, float32, one row
per wanted token; under graph replay they must write in place).  A schedule entry with
``add_embedding`` has the embedded tokens (after the stream parts) added to the stream once more
before its run: how a model that runs a stretch of layers several times feeds every further pass.
Before an entry with ``begins_pass`` the model's "pass" part changes the stream instead.
A model may keep the residual stream in several copies (``ModelSpec.streams``), ``[copies, tokens,
dim]``: they start as the embedded tokens, the layers' arrangement says how they change, and the final
norm reads their sum.
"""
from __future__ import annotations

from dataclasses import replace
from typing import List, Optional

import torch

from ..config.specs import ModelSpec
from ..kernels import ops
from ..parts import build_part
from ..parts.base import KVRequirement, Part, requirement_list
from .batch import StepContext


class Model(Part):
    def __init__(self, spec: ModelSpec, *, dtype: torch.dtype, device) -> None:
        super().__init__()
        if dtype not in (torch.float32, torch.bfloat16):
            raise ValueError("the model runs in float32 or bfloat16")
        self.spec = spec
        self.dtype = dtype
        self.device = torch.device(device)
        self.schedule = spec.resolved_schedule()
        self.embedding_again = spec.embedding_again()
        if spec.streams < 1 or any(layer.streams != spec.streams for layer in spec.layers):
            raise ValueError(f"the model keeps its residual stream in {spec.streams} copies, its layers in "
                             f"{sorted({layer.streams for layer in spec.layers})}")
        if spec.streams > 1 and (spec.stream_parts or any(self.embedding_again)):
            raise ValueError("parts on the embedded tokens and tokens added again need a residual stream in one copy")
        begins = [(i, e.begins_pass) for i, e in enumerate(spec.schedule) if e.begins_pass is not None]
        if begins and (spec.pass_entry is None or spec.streams > 1):
            raise ValueError("runs that begin a pass need the model's pass_entry and a residual stream in one copy")
        if any(not 0 <= t < spec.pass_entry.times for _, t in begins):
            raise ValueError(f"a pass is numbered 0 to {spec.pass_entry.times - 1}")
        self.begins_pass = dict(begins)
        self.add_param("embed", (spec.vocab_size, spec.hidden_size), dtype, device)
        if not spec.tie_word_embeddings:
            self.add_param("lm_head", (spec.vocab_size, spec.hidden_size), dtype, device)
        self.blocks: List[Part] = []
        for index, layer in enumerate(spec.layers):
            block = build_part("block", layer, dtype=dtype, device=device)
            self.blocks.append(block)
            self.add_child(f"layers.{index}", block)
        self.pass_entry = None
        if spec.pass_entry is not None:
            self.pass_entry = self.add_child("pass_entry", build_part("pass", spec.pass_entry, dtype=dtype, device=device))
        self.final_norm = self.add_child(
            "final_norm", build_part("norm", spec.final_norm, dtype=dtype, device=device)
        )
        self.stream_parts = [self.add_child(f"stream.{i}", build_part("stream", part, dtype=dtype, device=device))
                             for i, part in enumerate(spec.stream_parts)]
        self.logit_parts = [self.add_child(f"logits.{i}", build_part("logits", part, dtype=dtype, device=device))
                            for i, part in enumerate(spec.logit_parts)]

    # ---- what the cache manager has to provide ------------------------------------------
    def cache_requirements(self) -> List[object]:
        """Per run of the schedule: what it keeps.  A run that borrows another run's keys and values
        keeps none of its own, but its fixed-size state (a token shift's last input, a convolution's
        window) is its own."""
        def split(need):
            parts = requirement_list(need)
            return ([p for p in parts if isinstance(p, KVRequirement)],
                    [p for p in parts if not isinstance(p, KVRequirement)])

        needs: List[object] = []
        for index, (layer, cache_id, stores) in enumerate(self.schedule):
            own = self.blocks[layer].cache_requirement()
            if stores:
                needs.append(own)
                continue
            kv, states = split(own)
            if kv != split(self.blocks[self.schedule[cache_id][0]].cache_requirement())[0]:
                raise ValueError(
                    f"run {index} borrows the cache of run {cache_id}, which has another geometry"
                )
            needs.append(None if not states else (states[0] if len(states) == 1 else tuple(states)))
        return needs

    def decode_signature(self, rows: int, bound: int) -> tuple:
        """What the launches of a decode-only step of ``rows`` requests take from a bound on
        the requests' lengths, over all layers: two bounds with equal signatures record the
        same graph.  A block or mixer without ``decode_signature`` is taken to depend on the
        bound itself."""
        seen = []
        for block in self.blocks:
            describe = getattr(block, "decode_signature", None)
            signature = ("bound", bound) if describe is None else describe(rows, bound)
            if signature not in seen:
                seen.append(signature)
        return tuple(seen)

    @property
    def head_weight(self) -> torch.Tensor:
        return self.params["embed"] if self.spec.tie_word_embeddings else self.params["lm_head"]

    # ---- the step --------------------------------------------------------------------------
    def step(self, ctx: StepContext) -> Optional[torch.Tensor]:
        """Run the step's tokens through every scheduled layer, from and into the cache.
        Returns float32 logits ``[n_logits, vocab]`` (None when no logits are wanted)."""
        resid = ops.embed(ctx.token_ids, self.params["embed"], scale=self.spec.embedding_scale,
                          chosen=ctx.chosen, copies=self.spec.streams)
        for part in self.stream_parts:
            resid = part.forward(resid, ctx)
        # a schedule may add the embedded tokens to the stream again before some of its runs
        embedded = resid.clone() if any(self.embedding_again) or self.begins_pass else None
        delta = None
        for run, ((layer, cache_id, stores), again) in enumerate(zip(self.schedule, self.embedding_again)):
            if again:
                ops.residual_add(resid, embedded)  # the pending output of the run before follows in the norm
            if run in self.begins_pass:
                resid, delta = self.pass_entry.forward(resid, delta, embedded, self.begins_pass[run], ctx)
            cache = ctx.cache(cache_id)
            if not stores:
                # the lender's keys and values, the run's own fixed-size state
                own = ctx.cache(run)
                cache = replace(cache, state=own.state, states=own.states)
            resid, delta = self.blocks[layer].forward(resid, delta, ctx, cache, stores)
        if ctx.n_logits == 0:
            return None
        h = self.final_norm.add_forward(resid, delta, row_idx=ctx.logit_idx)
        out = None if ctx.logits_out is None else ctx.logits_out[: ctx.n_logits]
        logits = ops.linear(h, self.head_weight, out_dtype=torch.float32, out=out)
        for part in self.logit_parts:
            logits = part.forward(logits, ctx)  # in place where ``out`` was given
        return logits
