"""A routed mixture of feed-forwards, gated or plain, with identity experts, groups of experts and a shared expert."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import core
from ..ops.linear import ACT_GATED, activation_code, linear, linear_gated, pair_rows
from .base import FeedForward, register_feed_forward
from .specs import ParamSpec, RoutedExpertsSpec


class RoutedExperts(FeedForward):
    """``sum over the chosen k of weight_k * expert_k(h) [+ sigmoid(shared.sg h) * shared(h)]``.

    Every expert is ``down(act(gate h) * (up h))`` without biases (tensors ``e<i>.gate.weight`` and so on), with clamps where
    ``spec.clamp`` says so, or, with ``spec.gated`` off, ``down(act(up h))``. The router
    (``router.weight`` ``[n_experts + n_identity, dim]``) writes fp32 logits from fp32 sums, and the choice is made in fp32; how its scores become a choice and weights is
    ``RoutedExpertsSpec``'s text (a stored bias of the logits, where there is one, enters in the router's linear). The router's last ``n_identity`` outputs are identity experts: their output is ``h``.
    The shared expert (``shared.*``) has the experts' form and a hidden size of its own; its gate ``shared.sg.weight``
    ``[1, dim]`` rides as one more row of the router's linear. A shared expert of the experts' own size and constants, without a
    gate, is laid behind the experts as one more, which every token chooses with weight 1: it then has no launches of its own.

    When the weights are bound, the experts' ``gate`` and ``up`` rows are laid in pairs and the experts stacked
    (``[E, 2 hidden, dim]``, plain ones ``[E, hidden, dim]``; ``[E, dim, hidden]``). A step runs: the router's linear (fp32), the choice
    (``ops.core.route``), the experts' two linears, and the weighted sum. In bf16, by the number of pairs (token, choice): a
    step of up to ``PAIR_BY_PAIR_TO`` computes every pair by itself, its expert's weights streamed for it
    (``ops.core.experts_linear``; fp32 always does); up to ``FEW_PAIRS_TO`` every chosen expert's weights are streamed once past its pairs
    (``ops.fast.experts_few_bf16``); beyond, the pairs are listed by expert first and each expert's go through the matrix cores in
    tiles (``ops.fast.experts_feed_forward_bf16``). Measured, both linears, 31 experts of 2,048 x 704: 4 tokens of 5 pairs 38, 38 and 94
    us in this order, 8 tokens 62, 52 and 98, 32 tokens 201, 72 and 106, 96 tokens (480 pairs) -, 118 and 119. Either way a
    pair's result depends on its own row alone."""

    replays_every_step = True
    PAIR_BY_PAIR_TO = 20
    FEW_PAIRS_TO = 512

    def __init__(self, spec: RoutedExpertsSpec) -> None:
        super().__init__(spec)
        if spec.n_experts <= 0 or spec.top <= 0 or spec.n_identity < 0:
            raise ValueError("routed experts need experts and a positive number of choices")
        self.n_outputs = spec.n_experts + spec.n_identity
        if spec.top > self.n_outputs:
            raise ValueError(f"{spec.top} choices among {self.n_outputs} router outputs")
        if spec.n_groups:
            if self.n_outputs % spec.n_groups or not 0 < spec.keep_groups <= spec.n_groups:
                raise ValueError(f"{spec.n_groups} groups (of which {spec.keep_groups} are kept) do not divide {self.n_outputs} router outputs")
            if spec.keep_groups * (self.n_outputs // spec.n_groups) < spec.top:
                raise ValueError("the kept groups hold fewer router outputs than a token chooses")
        self.act = activation_code(spec.activation)
        self.gated = bool(getattr(spec, "gated", True))
        self.weigh_chosen = bool(getattr(spec, "weigh_chosen", False))
        if self.weigh_chosen and spec.n_groups:
            raise ValueError("a router that weighs the chosen logits alone has no groups of experts")
        self.scores = str(getattr(spec, "scores", "softmax"))
        self.group_best = int(getattr(spec, "group_best", 1))
        if self.scores not in core.ROUTER_SCORES or self.group_best not in (1, 2):
            raise ValueError(f"a router's scores are one of {sorted(core.ROUTER_SCORES)} and its groups count by one or two of them")
        self.clamp = getattr(spec, "clamp", None)
        self.shared_clamp = getattr(spec, "shared_clamp", None)
        for clamp in (self.clamp, self.shared_clamp):
            if clamp is not None and (not self.gated or not clamp.limit > 0):
                raise ValueError("clamps are a gated expert's, with a positive limit")
        self.up_act = self.act | ACT_GATED if self.gated else self.act
        self.shared = spec.shared_hidden is not None
        self.gated_shared = self.shared and bool(spec.shared_gate)
        # the shared expert as one more expert that every token uses
        self.joined = self.shared and not self.gated_shared and spec.n_identity == 0 and spec.shared_hidden == spec.hidden_dim \
            and self.shared_clamp == self.clamp
        self.pairs = self.down = self.router = self.correction = self.router_bias = None
        self.shared_pairs = self.shared_down = None
        self.dtype: Optional[torch.dtype] = None

    def params(self) -> Dict[str, ParamSpec]:
        spec = self.spec
        out = {}
        for e in range(spec.n_experts):
            if self.gated:
                out[f"e{e}.gate.weight"] = ParamSpec((spec.hidden_dim, spec.dim))
            out[f"e{e}.up.weight"] = ParamSpec((spec.hidden_dim, spec.dim))
            out[f"e{e}.down.weight"] = ParamSpec((spec.dim, spec.hidden_dim))
        out["router.weight"] = ParamSpec((self.n_outputs, spec.dim))
        out["router.bias" if self.weigh_chosen else "correction"] = ParamSpec((self.n_outputs,), "vector", "bias")
        if self.shared:
            if self.gated:
                out["shared.gate.weight"] = ParamSpec((spec.shared_hidden, spec.dim))
            out["shared.up.weight"] = ParamSpec((spec.shared_hidden, spec.dim))
            out["shared.down.weight"] = ParamSpec((spec.dim, spec.shared_hidden))
            if self.gated_shared:
                out["shared.sg.weight"] = ParamSpec((1, spec.dim))
        return out

    def bind(self, tensors, dtype, device) -> None:
        spec = self.spec
        self.dtype = dtype

        def first_rows(name: str) -> torch.Tensor:
            up = tensors[f"{name}.up.weight"].to(device)
            return pair_rows(tensors[f"{name}.gate.weight"].to(device), up) if self.gated else up

        listed = [f"e{e}" for e in range(spec.n_experts)] + (["shared"] if self.joined else [])
        self.pairs = torch.stack([first_rows(name) for name in listed]).contiguous()
        self.down = torch.stack([tensors[f"{name}.down.weight"].to(device) for name in listed]).contiguous()
        # The router's rows stay in the type they are held in: products of bf16 numbers are exact in fp32 and every linear
        # kernel sums in fp32, so a bf16 run computes the router's sums in 32 bits from the rounded input, as an fp32 run does
        # from its own. The shared expert's gate rides as one more row.
        rows = [tensors["router.weight"].to(device)]
        if self.gated_shared:
            rows.append(tensors["shared.sg.weight"].to(device=device, dtype=rows[0].dtype).reshape(1, spec.dim))
        self.router = torch.cat(rows, dim=0).contiguous()
        if self.weigh_chosen:
            self.router_bias = torch.zeros(self.router.shape[0], dtype=torch.float32, device=device)
            self.router_bias[:self.n_outputs] = tensors["router.bias"].to(device=device, dtype=torch.float32)
        else:
            self.correction = tensors["correction"].to(device=device, dtype=torch.float32).contiguous()
        if self.shared and not self.joined:
            self.shared_pairs = first_rows("shared").contiguous()
            self.shared_down = tensors["shared.down.weight"].to(device).contiguous()

    def _outputs(self, h, batch):
        """Everything but the weighted sum: the pairs' outputs, the choice, its weights, the shared expert's output and gate."""
        spec = self.spec
        n = h.shape[0]
        ws = batch.workspace
        top = spec.top + self.joined
        logits = ws.get("experts.logits", (n, self.router.shape[0]), torch.float32)
        linear(h, self.router, self.router_bias, logits)
        chosen = ws.get("experts.chosen", (n, top), torch.int32)
        weights = ws.get("experts.weights", (n, top), torch.float32)
        core.route(logits, self.n_outputs, self.correction, spec.top, spec.n_groups, spec.keep_groups, spec.scale, chosen, weights,
                   weigh_chosen=self.weigh_chosen, scores=self.scores, group_best=self.group_best,
                   always=spec.n_experts if self.joined else None)
        hidden = ws.get("experts.hidden", (n * top, spec.hidden_dim), self.dtype)
        y = ws.get("experts.y", (n * top, spec.dim), torch.float32)
        done = False
        if self.dtype == torch.bfloat16 and n * top > self.PAIR_BY_PAIR_TO:
            from ..ops import fast
            operands = (h, self.pairs, self.down, chosen, hidden, y, self.up_act)
            done = n * top <= self.FEW_PAIRS_TO and fast.experts_few_bf16(*operands, clamp=self.clamp)
            done = done or fast.experts_feed_forward_bf16(*operands, ws, clamp=self.clamp)
        if not done:
            flat = chosen.view(-1)
            core.experts_linear(h, top, self.pairs, flat, hidden, self.up_act, clamp=self.clamp)
            core.experts_linear(hidden, 1, self.down, flat, y)
        shared_out = gate = None
        if self.shared and not self.joined:
            shared_hidden = ws.get("experts.shared_hidden", (n, spec.shared_hidden), self.dtype)
            if not self.gated:
                linear(h, self.shared_pairs, None, shared_hidden, act=self.act)
            elif self.shared_clamp is not None or (self.dtype == torch.bfloat16 and n >= 256):
                sums = ws.get("experts.shared_sums", (n, 2 * spec.shared_hidden), self.dtype)
                linear(h, self.shared_pairs, None, sums)
                if self.shared_clamp is not None:
                    core.clamped_pairs(sums, shared_hidden, self.shared_clamp.limit, self.shared_clamp.slope, self.shared_clamp.shift)
                else:
                    core.gated_pairs(sums, shared_hidden, self.act)
            else:
                linear_gated(h, self.shared_pairs, None, shared_hidden, self.act)
            shared_out = ws.get("experts.shared_out", (n, spec.dim), torch.float32)
            linear(shared_hidden, self.shared_down, None, shared_out)
            if self.gated_shared:
                gate = logits[:, self.n_outputs]
        return y, chosen, weights, shared_out, gate

    def mix(self, h, batch, out, accumulate: bool) -> None:
        """The feed-forward of ``h`` written into (or added to) fp32 ``out``."""
        y, chosen, weights, shared_out, gate = self._outputs(h, batch)
        core.experts_combine(y, h, chosen, weights, self.pairs.shape[0], shared_out, gate, out, accumulate)

    def mix_normed(self, h, batch, x, norm, then, rows) -> None:
        """The feed-forward of ``h``, normalised (``norm``: ``(gain, eps)`` of a root-mean-square norm) and added into fp32 ``x``
        by the launch that takes the weighted sum; ``then`` (the same form) of the new rows of ``x`` goes into ``rows``."""
        y, chosen, weights, shared_out, gate = self._outputs(h, batch)
        core.experts_combine_normed(y, h, chosen, weights, self.pairs.shape[0], shared_out, gate, x, norm, then, rows)

    def mix_streams(self, h, batch, x, streams, reading, rows) -> None:
        """The feed-forward of ``h`` written into the streams ``x`` by the numbers of ``streams`` (a ``StreamMix``), by the launch that
        takes the weighted sum; what ``reading`` sees of the new streams goes into ``rows`` (``ops.core.streams_step``)."""
        y, chosen, weights, shared_out, gate = self._outputs(h, batch)
        core.streams_experts(x, y, h, chosen, weights, self.pairs.shape[0], shared_out, gate, streams.matrix, streams.out, reading, rows)

    def forward(self, h, batch, residual) -> None:
        self.mix(h, batch, residual, True)


register_feed_forward("routed_experts", RoutedExperts)
