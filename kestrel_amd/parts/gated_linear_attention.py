"""Gated linear attention: a recurrence whose state forgets channel by channel, by factors computed from the input."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import core
from ..ops.linear import linear
from .base import LayerCache, Mixer, register_mixer
from .specs import GatedLinearAttentionSpec, ParamSpec, StateSpec


class GatedLinearAttention(Mixer):
    """Per head a state ``S`` ``[hd, hdv]``, fp32, zero for a new request and carried from token to token in the request's
    state slot (held transposed, a value channel's row of key channels after the other).

    With ``q = W_q h * hd ** -0.5``, ``k = W_k h`` (heads of ``hd``), ``v = W_v h`` (heads of ``hdv``) and per head and key channel the
    decay ``a = sigmoid(z) ** (1 / tau)``, ``z = W_a2 (W_a1 h) + b``, per head

        S_t = diag(a_t) S_(t-1) + k_t v_t^T          o_t = S_t^T q_t

    Every head's ``o`` is divided by its root mean square (``eps``) and multiplied by the gain ``norm.weight`` ``[hdv]`` that the heads
    share; the concatenated heads are multiplied by ``silu(W_gate h)`` and go through the output projection.

    One launch projects q | k | v | gate | a1 in the activation type. A step of single tokens is one more launch up to the output
    projection (``ops.core.gated_step``). Otherwise ``z`` comes from a linear of its own with fp32 output (what enters the recurrence
    besides the projections is fp32); steps of a few tokens, and fp32 runs, walk over every row's tokens in order
    (``ops.core.gated_linear_attention``), longer bf16 steps run on the matrix cores, the recurrence unrolled over chunks of 64
    tokens (``ops.fast.gated_chunks_bf16``); either leaves the read-outs in fp32, which one launch normalises and gates. Rows
    without a request (the padding of a replayed step) write zeros and touch no state."""

    replays_every_step = True
    # Tokens of a step from which the chunks' launches are run instead of the walk over tokens (a chain of that length at most)
    CHUNKS_FROM_TOKENS = 17

    def __init__(self, spec: GatedLinearAttentionSpec) -> None:
        super().__init__(spec)
        if not spec.tau > 0:
            raise ValueError(f"gated linear attention needs a positive tau, got {spec.tau}")
        self.qk_dim = spec.n_heads * spec.head_dim
        self.v_dim = spec.n_heads * spec.value_dim
        self.rank = -1 if spec.decay_rank is None else int(spec.decay_rank)
        self.offsets = (0, self.qk_dim, 2 * self.qk_dim)
        self.gate_at = 2 * self.qk_dim + self.v_dim
        self.low_at = self.gate_at + self.v_dim
        self.in_dim = self.low_at
        self.in_weight = self.a2_weight = self.a2_bias = self.gain = self.proj_weight = None
        self.dtype: Optional[torch.dtype] = None

    def params(self) -> Dict[str, ParamSpec]:
        spec = self.spec
        return {"q.weight": ParamSpec((self.qk_dim, spec.dim)), "k.weight": ParamSpec((self.qk_dim, spec.dim)),
                "v.weight": ParamSpec((self.v_dim, spec.dim)), "gate.weight": ParamSpec((self.v_dim, spec.dim)),
                "a1.weight": ParamSpec((self.rank, spec.dim)), "a2.weight": ParamSpec((self.qk_dim, self.rank)),
                "a2.bias": ParamSpec((self.qk_dim,), "vector", "bias"), "norm.weight": ParamSpec((spec.value_dim,), "vector", "gain"),
                "proj.weight": ParamSpec((spec.dim, self.v_dim))}

    def state_spec(self) -> StateSpec:
        return StateSpec((self.v_dim * self.spec.head_dim,), "float32")

    def bind(self, tensors, dtype, device) -> None:
        spec = self.spec
        self.dtype = dtype
        if not core.linear_attention_supported(spec.head_dim, spec.value_dim):
            raise ValueError(f"the kernels of linear attention take key heads of up to 512 channels, got {spec.head_dim}")
        self.in_weight = torch.cat([tensors[name].to(device) for name in ("q.weight", "k.weight", "v.weight", "gate.weight", "a1.weight")],
                                   dim=0).contiguous()
        self.in_dim = self.in_weight.shape[0]
        self.rank = self.in_dim - self.low_at
        self.a2_weight = tensors["a2.weight"].to(device).contiguous()
        if self.a2_weight.shape[1] != self.rank:
            raise ValueError(f"the decay's two linears meet in {self.rank} and {self.a2_weight.shape[1]} channels")
        self.a2_bias = tensors["a2.bias"].to(device=device, dtype=torch.float32).contiguous()
        self.gain = tensors["norm.weight"].to(device=device, dtype=torch.float32).contiguous()
        self.proj_weight = tensors["proj.weight"].to(device).contiguous()

    def input_projection(self):
        return self.in_weight, None, self.in_dim

    def output_projection(self):
        return self.proj_weight, None

    def share_projections(self, in_weight, proj_weight) -> None:
        self.in_weight, self.proj_weight = in_weight, proj_weight

    def takes_output_weight(self, weight: float) -> bool:
        return True

    def fold_output_weight(self, weight: float) -> None:
        self.gain = self.gain * float(weight)          # (the last factor of the heads before the gate, fp32)

    def attend(self, projected, batch, cache: LayerCache, beside=None, out: Optional[torch.Tensor] = None) -> torch.Tensor:
        """The recurrence over the step's tokens, normalised and gated: the input of the output projection."""
        spec = self.spec
        n = projected.shape[0]
        ws = batch.workspace
        if cache.state is None:
            raise RuntimeError("gated linear attention needs its per-request state from the cache manager")
        if out is None:
            out = ws.get("gated_attention.out", (n, self.v_dim), self.dtype)
        sizes = (spec.n_heads, spec.head_dim, spec.value_dim)
        q_scale = float(spec.head_dim) ** -0.5
        if batch.decode_only and core.gated_step(projected, (*self.offsets, self.gate_at, self.low_at), self.a2_weight, self.a2_bias, self.gain,
                                                 float(spec.tau), q_scale, float(spec.eps), cache.state, batch.row_slot, out, *sizes):
            return out
        pre = ws.get("gated_attention.pre", (n, self.qk_dim), torch.float32)
        linear(projected[:, self.low_at:self.low_at + self.rank], self.a2_weight, self.a2_bias, pre)
        raw = ws.get("gated_attention.raw", (n, self.v_dim), torch.float32)
        operands = (projected, self.offsets, pre, float(spec.tau), q_scale, cache.state, batch.cu_q, batch.row_slot, raw, *sizes)
        done = False
        if self.dtype == torch.bfloat16 and not batch.decode_only and n >= self.CHUNKS_FROM_TOKENS:
            # (sized by the host side of the batch alone: the same for every replay of a captured step)
            from ..ops import fast
            need = fast.gated_chunks_scratch(n, batch.n_rows, *sizes)
            if need:
                done = fast.gated_chunks_bf16(*operands, ws.get("gated_attention.chunks", (need,), torch.float32))
        if not done:
            core.gated_linear_attention(*operands)
        core.heads_rmsnorm(raw, self.gain, projected[:, self.gate_at:self.gate_at + self.v_dim], out, spec.n_heads, spec.value_dim, float(spec.eps))
        return out

    def mix(self, h, batch, cache: LayerCache, out, accumulate: bool) -> None:
        """The mixer's output written into (or added to) fp32 ``out``."""
        projected = batch.workspace.get("gated_attention.in", (h.shape[0], self.in_dim), self.dtype)
        linear(h, self.in_weight, None, projected)
        linear(self.attend(projected, batch, cache), self.proj_weight, None, out, accumulate=accumulate)

    def forward(self, h, batch, cache: LayerCache, residual) -> None:
        self.mix(h, batch, cache, residual, True)


register_mixer("gated_linear_attention", GatedLinearAttention)
