"""The generic decoder: embedding, the scheduled blocks, final norm and head.

It is put together from a ``ModelPlan`` alone and knows no architecture. The order of
execution is the plan's ``schedule``: a list of runs, each naming a layer (a layer may be
named twice and then shares its weights) and optionally an earlier run whose cache it
reads instead of keeping one.
"""

from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import core
from ..ops.linear import linear
from ..parts.base import LayerCache, build_part
from ..parts.block import Block, settle
from ..parts.specs import ModelPlan, ParamSpec
from ..parts.streams import StreamReading


class DecoderModel:
    def __init__(self, plan: ModelPlan) -> None:
        self.plan = plan
        self.blocks: List[Block] = [Block(layer) for layer in plan.layers]
        self.final_norm = build_part("norm", plan.final_norm)
        self.position = build_part("position", plan.position) if plan.position is not None else None
        embedding_norm = getattr(plan, "embedding_norm", None)
        self.embedding_norm = build_part("norm", embedding_norm) if embedding_norm is not None else None
        self.junctions = {name: build_part("junction", spec) for name, spec in dict(getattr(plan, "junctions", None) or {}).items()}
        for index, entry in enumerate(plan.schedule):
            before = getattr(entry, "before", None)
            if before is not None and before not in self.junctions:
                raise ValueError(f"schedule entry {index} passes through the junction {before!r}, the plan has "
                                 f"{sorted(self.junctions) or 'none'}")
            if not 0 <= entry.layer < len(self.blocks):
                raise ValueError(f"schedule entry {index} names layer {entry.layer}, the plan has {len(self.blocks)}")
            if entry.reads_cache_of is not None:
                if not 0 <= entry.reads_cache_of < index:
                    raise ValueError(f"schedule entry {index} must read the cache of an earlier entry")
                if plan.schedule[entry.reads_cache_of].reads_cache_of is not None:
                    raise ValueError(f"schedule entry {index} reads the cache of an entry that keeps none")
        self.streams: Optional[int] = getattr(plan, "streams", None)
        mixes = [m.spec.streams for b in self.blocks for m in (b.streams, b.streams2) if m is not None]
        if self.streams is not None:
            if self.junctions or any(b.spec.arrangement != "streams" for b in self.blocks) or any(s != self.streams for s in mixes):
                raise ValueError(f"a stream of {self.streams} copies passes through blocks of the arrangement 'streams' for as many, and through no junction")
        elif mixes:
            raise ValueError("blocks that read several streams need a plan that names how many there are")
        self.embedding: Optional[torch.Tensor] = None
        self.head_weight: Optional[torch.Tensor] = None
        self.head_bias: Optional[torch.Tensor] = None
        self.dtype: Optional[torch.dtype] = None
        self.device: Optional[torch.device] = None

    # ------------------------------------------------------------------ tensors
    def params(self) -> Dict[str, ParamSpec]:
        """Checkpoint tensor name -> shape and role of every tensor the model owns."""
        plan = self.plan
        out = {plan.names["embedding"]: ParamSpec((plan.vocab_size, plan.dim), "matrix", "normal")}
        for block in self.blocks:
            out.update(block.params())
        for local, pspec in self.final_norm.params().items():
            out[plan.names[f"final_norm.{local}"]] = pspec
        if self.embedding_norm is not None:
            for local, pspec in self.embedding_norm.params().items():
                out[plan.names[f"embedding_norm.{local}"]] = pspec
        if self.position is not None:
            for local, pspec in self.position.params().items():
                out[plan.names[f"position.{local}"]] = pspec
        for name, junction in self.junctions.items():
            for local, pspec in junction.params().items():
                out[plan.names[f"junction.{name}.{local}"]] = pspec
        if not plan.tied_head:
            out[plan.names["head.weight"]] = ParamSpec((plan.vocab_size, plan.dim), "matrix", "normal")
        if plan.head_bias:
            out[plan.names["head.bias"]] = ParamSpec((plan.vocab_size,), "vector", "bias")
        return out

    def bind(self, tensors: Dict[str, torch.Tensor], dtype: torch.dtype, device: torch.device) -> None:
        plan = self.plan
        self.dtype, self.device = dtype, device
        self.embedding = tensors[plan.names["embedding"]].to(device).contiguous()
        for block in self.blocks:
            block.bind(tensors, dtype, device)
        self.final_norm.bind({k: tensors[plan.names[f"final_norm.{k}"]] for k in self.final_norm.params()}, dtype,
                             device)
        if self.embedding_norm is not None:
            self.embedding_norm.bind({k: tensors[plan.names[f"embedding_norm.{k}"]] for k in self.embedding_norm.params()}, dtype, device)
        if self.position is not None:
            self.position.bind({k: tensors[plan.names[f"position.{k}"]] for k in self.position.params()}, dtype, device)
        for name, junction in self.junctions.items():
            junction.bind({k: tensors[plan.names[f"junction.{name}.{k}"]] for k in junction.params()}, dtype, device)
        self.head_weight = self.embedding if plan.tied_head else tensors[plan.names["head.weight"]].to(device).contiguous()
        if plan.head_bias:
            self.head_bias = tensors[plan.names["head.bias"]].to(device=device, dtype=torch.float32).contiguous()

    # ------------------------------------------------------------------ cache needs
    def cache_needs(self):
        """Per schedule entry: ``(cache_spec or None, state_spec or None, reads_cache_of)``."""
        needs = []
        for entry in self.plan.schedule:
            mixer = self.blocks[entry.layer].mixer
            needs.append((mixer.cache_spec(), mixer.state_spec(), entry.reads_cache_of))
        # behind the schedule's entries: what parts outside the layers keep per request (no keys and values)
        position_state = getattr(self.position, "state_spec", None)
        if callable(position_state) and position_state() is not None:
            needs.append((None, position_state(), None))
        return needs

    def position_axes(self) -> int:
        """The most numbers any position encoding of the model (its own, or a mixer's) needs per token."""
        parts = [self.position] + [getattr(block.mixer, "position", None) for block in self.blocks]
        return max([1] + [int(getattr(part, "axes", 1)) for part in parts if part is not None])

    def replays_every_step(self) -> bool:
        """Whether steps of every shape may be captured and replayed: every part of the model says so
        (``Part.replays_every_step``)."""
        parts = [self.final_norm, self.embedding_norm, self.position] + list(self.junctions.values())
        for block in self.blocks:
            parts += list(block.parts().values()) + [getattr(block.mixer, "position", None)]
        return all(bool(getattr(part, "replays_every_step", False)) for part in parts if part is not None)

    def query_tiles(self):
        """Sizes of blocks of queries that the mixers' kernels want listed with a step."""
        return {tile for tile in (block.mixer.query_tile() for block in self.blocks) if tile}

    def _head_with_norm(self, x, batch, logits) -> bool:
        """A few decoded rows, every one of them wanted, in order: the head's launch normalises them itself
        (one launch less a step)."""
        ln = self.final_norm.layernorm_operands()
        rms = self.final_norm.rms_operands() if ln is None and callable(getattr(self.final_norm, "rms_operands", None)) else None
        if self.dtype != torch.bfloat16 or not batch.decode_only or not getattr(batch, "wants_every_token", False) \
                or (ln is None and rms is None):
            return False
        from ..ops import fast
        if ln is None:
            return fast.layernorm_linear(x, rms[0], None, rms[1], self.head_weight, self.head_bias, logits, 0, centred=False)
        return fast.layernorm_linear(x, *ln, self.head_weight, self.head_bias, logits, 0)

    # ------------------------------------------------------------------ forward
    def forward(self, batch, caches: List[LayerCache]) -> torch.Tensor:
        """Run the packed tokens of ``batch``; returns fp32 logits ``[wanted, vocab]``."""
        plan = self.plan
        ws = batch.workspace
        if getattr(batch, "host", None) is not None:
            # what parts make once a step for all layers: made anew by every run (a captured run must launch it itself)
            batch.host["made_once"] = {}
        x = ws.get("model.x", (batch.n_tokens, plan.dim), torch.float32)
        # (a norm of the embedded tokens reads them from a buffer of their own)
        looked_up = x if self.embedding_norm is None else ws.get("model.looked_up", (batch.n_tokens, plan.dim), torch.float32)
        core.embed(self.embedding, batch.token_ids, looked_up, batch.pending, plan.embedding_scale)
        if batch.given_embeds is not None:
            core.scatter_rows(batch.given_embeds, batch.given_rows, looked_up)
        if self.embedding_norm is not None:
            self.embedding_norm.forward(looked_up, x)
        if self.position is not None:
            position_state = getattr(self.position, "state_spec", None)
            if callable(position_state) and position_state() is not None:
                self.position.add_to_embeddings(x, batch, state=caches[len(plan.schedule)].state)
            else:
                self.position.add_to_embeddings(x, batch)
        for junction in self.junctions.values():
            junction.begin(x, batch)
        handed = None      # the next block's first norm of x, where a block's last launch has computed it
        final = None
        if self.streams is not None:
            # every stream starts as the embedding output; the launch that says so leaves what the first block reads
            embedded, x = x, ws.get("model.streams", (batch.n_tokens, self.streams, plan.dim), torch.float32)
            final = StreamReading(None, self.final_norm)
            first = self.blocks[plan.schedule[0].layer].reader if plan.schedule else None
            handed = ws.get("block.h", (batch.n_tokens, plan.dim), self.dtype) if first is not None else None
            core.streams_step(x, embedded=embedded, reading=first.operands() if first is not None else None, h=handed)
        for index, entry in enumerate(plan.schedule):
            after = plan.schedule[index + 1] if index + 1 < len(plan.schedule) else None
            # (a junction between two runs changes the stream: no norm is handed across it)
            then = self.blocks[after.layer].reader if after is not None and getattr(after, "before", None) is None else None
            if after is None and final is not None and batch.decode_only and getattr(batch, "wants_every_token", False):
                then = final       # (every row goes to the head, in order: the last launch leaves what the head reads)
            before = getattr(entry, "before", None)
            if before is not None:
                settle(x, batch)
                self.junctions[before].forward(x, batch, passage=int(getattr(entry, "passage", 0)))
                handed = None
            handed = self.blocks[entry.layer].forward(x, batch, caches[index], normed=handed, then=then)
        settle(x, batch)       # (what the last block has left to be added into the stream)
        wanted = int(batch.logit_rows.numel())
        logits = ws.get("model.logits", (wanted, plan.vocab_size), torch.float32)
        if wanted and self.streams is not None:
            normed = handed if batch.decode_only and getattr(batch, "wants_every_token", False) else None
            if normed is None:
                normed = ws.get("model.head_in", (wanted, plan.dim), self.dtype)
                core.streams_step(x, reading=final.operands(), h=normed, rows=batch.logit_rows)
            linear(normed, self.head_weight, self.head_bias, logits)
        elif wanted:
            if not self._head_with_norm(x, batch, logits):
                normed = ws.get("model.head_in", (wanted, plan.dim), self.dtype)
                self.final_norm.forward(x, normed, rows=batch.logit_rows)
                linear(normed, self.head_weight, self.head_bias, logits)
        if wanted:
            if plan.logit_scale != 1.0 or plan.logit_softcap is not None:
                core.adjust_logits(logits, plan.logit_scale, plan.logit_softcap)
        return logits
