"""Attention without a softmax: a recurrence with one constant decay per head."""

from __future__ import annotations

import math
from typing import Dict, Optional

import torch

from ..ops import core
from ..ops.linear import activation_code, linear
from .base import LayerCache, Mixer, register_mixer
from .specs import LinearAttentionSpec, ParamSpec, StateSpec


class LinearAttention(Mixer):
    """Per head a state ``S`` ``[hd, hdv]``, fp32, zero for a new request and carried from token to token in the request's
    state slot (held transposed, a value channel's row of key channels after the other).

    With ``q = act(W_q h)``, ``k = act(W_k h)`` (heads of ``hd``) and ``v = act(W_v h)`` (heads of ``hdv``), per head

        S_t = decay_h S_(t-1) + k_t v_t^T          o_t = S_t^T q_t

    The concatenated heads are divided by one root mean square over all of them (``eps``), multiplied by the gain
    ``norm.weight`` and by ``sigmoid(W_gate h)``, and go through the output projection.

    One launch projects q | k | v | gate in the activation type; the kernels of the recurrence apply the activation to what
    they load. Steps of single tokens, steps of a few tokens, and fp32 runs walk over every row's tokens in order
    (``ops.core.linear_attention``); longer bf16 steps run on the matrix cores, the recurrence unrolled over chunks of 64
    tokens (``ops.fast.linear_attention_chunks_bf16``). Either leaves the read-outs in fp32, which one launch normalises and
    gates. Rows without a request (the padding of a replayed step) write zeros and touch no state."""

    replays_every_step = True
    # Tokens of a step from which the chunks' three launches are run instead of the walk over tokens (a chain of that length at most)
    CHUNKS_FROM_TOKENS = 17

    def __init__(self, spec: LinearAttentionSpec) -> None:
        super().__init__(spec)
        if len(spec.decay) != spec.n_heads or not all(0.0 < float(a) <= 1.0 for a in spec.decay):
            raise ValueError(f"linear attention needs a decay above 0 and at most 1 for each of its {spec.n_heads} heads, got {spec.decay}")
        self.qk_dim = spec.n_heads * spec.head_dim
        self.v_dim = spec.n_heads * spec.value_dim
        self.gated = bool(spec.output_gate)
        # (q | k | v | gate; the columns of each begin on multiples of 16 bytes where the head sizes allow it)
        self.in_dim = 2 * self.qk_dim + self.v_dim * (2 if self.gated else 1)
        self.offsets = (0, self.qk_dim, 2 * self.qk_dim)
        self.act = activation_code(spec.activation)
        self.in_weight = self.gain = self.proj_weight = self.decay = self.log2_decay = None
        self.dtype: Optional[torch.dtype] = None

    def params(self) -> Dict[str, ParamSpec]:
        spec = self.spec
        out = {"q.weight": ParamSpec((self.qk_dim, spec.dim)), "k.weight": ParamSpec((self.qk_dim, spec.dim)),
               "v.weight": ParamSpec((self.v_dim, spec.dim)), "proj.weight": ParamSpec((spec.dim, self.v_dim)),
               "norm.weight": ParamSpec((self.v_dim,), "vector", "gain")}
        if self.gated:
            out["gate.weight"] = ParamSpec((self.v_dim, spec.dim))
        return out

    def state_spec(self) -> StateSpec:
        return StateSpec((self.spec.n_heads * self.spec.value_dim * self.spec.head_dim,), "float32")

    def bind(self, tensors, dtype, device) -> None:
        spec = self.spec
        self.dtype = dtype
        if not core.linear_attention_supported(spec.head_dim, spec.value_dim):
            raise ValueError(f"the kernels of linear attention take key heads of up to 512 channels, got {spec.head_dim}")
        names = ["q.weight", "k.weight", "v.weight"] + (["gate.weight"] if self.gated else [])
        self.in_weight = torch.cat([tensors[name].to(device) for name in names], dim=0).contiguous()
        self.gain = tensors["norm.weight"].to(device=device, dtype=torch.float32).contiguous()
        self.proj_weight = tensors["proj.weight"].to(device).contiguous()
        self.decay = torch.tensor([float(a) for a in spec.decay], dtype=torch.float32, device=device)
        self.log2_decay = torch.tensor([math.log2(float(a)) for a in spec.decay], dtype=torch.float32, device=device)

    def input_projection(self):
        return self.in_weight, None, self.in_dim

    def output_projection(self):
        return self.proj_weight, None

    def attend(self, projected, batch, cache: LayerCache, beside=None) -> torch.Tensor:
        """The recurrence over the step's tokens, normalised and gated: the input of the output projection."""
        spec = self.spec
        n = projected.shape[0]
        ws = batch.workspace
        if cache.state is None:
            raise RuntimeError("linear attention needs its per-request state from the cache manager")
        raw = ws.get("linear_attention.raw", (n, self.v_dim), torch.float32)
        sizes = (spec.n_heads, spec.head_dim, spec.value_dim, self.act)
        done = False
        if self.dtype == torch.bfloat16 and not batch.decode_only and n >= self.CHUNKS_FROM_TOKENS:
            # (sized by the host side of the batch alone: the same for every replay of a captured step)
            from ..ops import fast
            need = fast.linear_attention_chunks_scratch(n, batch.n_rows, spec.n_heads, spec.head_dim, spec.value_dim)
            if need:
                scratch = ws.get("linear_attention.chunks", (need,), torch.float32)
                done = fast.linear_attention_chunks_bf16(projected, self.offsets, self.log2_decay, cache.state, batch.cu_q, batch.row_slot,
                                                         raw, *sizes, scratch)
        if not done:
            core.linear_attention(projected, self.offsets, self.decay, cache.state, batch.cu_q, batch.row_slot, raw, *sizes)
        out = ws.get("linear_attention.out", (n, self.v_dim), self.dtype)
        core.gated_rmsnorm(raw, self.gain, float(spec.eps), projected[:, 2 * self.qk_dim + self.v_dim:] if self.gated else None, out)
        return out

    def mix(self, h, batch, cache: LayerCache, out, accumulate: bool) -> None:
        """The mixer's output written into (or added to) fp32 ``out``."""
        projected = batch.workspace.get("linear_attention.in", (h.shape[0], self.in_dim), self.dtype)
        linear(h, self.in_weight, None, projected)
        linear(self.attend(projected, batch, cache), self.proj_weight, None, out, accumulate=accumulate)

    def forward(self, h, batch, cache: LayerCache, residual) -> None:
        self.mix(h, batch, cache, residual, True)


register_mixer("linear_attention", LinearAttention)
