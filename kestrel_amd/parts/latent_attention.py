"""Latent attention: queries, keys and values through low-rank latents; the cache holds the latent."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import core
from ..ops.linear import linear
from .base import LayerCache, Mixer, build_part, register_mixer
from .specs import LatentAttentionSpec, LatentCacheSpec, ParamSpec


class LatentAttention(Mixer):
    """With ``rms(x) = x / sqrt(mean(x^2) + eps)``:

        c_q = rms(W_dq h) g_q,   q = W_uq c_q                 per head [hd plain | dr rotated]
        [c' | k_r] = W_dkv h,    c = rms(c') g_kv             c: the latent (kv_rank), k_r: dr channels shared by all heads
        k_h = [W_uk,h c | rot(k_r)],   v_h = W_uv,h c
        score = scale * (q_plain . W_uk,h c + rot(q_rot) . rot(k_r)),   softmax over j <= i with exp(sink_h) in the denominator
        out = W_o (concat_h(sum_j w_j v_h,j) * sigmoid(W_g h))

    Forms, each by its field of the specification: queries projected directly, ``q = W_q h`` (``q_rank`` ``None``); no rotated
    part (``rot_dim`` 0); a window, so that ``j`` is seen while ``i - j < window`` and pages behind it go back; no sinks; no gate,
    or a gate of one number per head (it rides in the attention kernel, where it multiplies the weighted latents).

    Only ``[c | rot(k_r)]`` is cached, one row of ``kv_rank + dr`` channels per token (``LatentCacheSpec``). The per-head
    up-projections are moved to the query's side: ``q_plain . W_uk,h c = (W_uk,h^T q_plain) . c``, so every head's query
    becomes ``[W_uk,h^T q_plain | rot(q_rot)]`` against the cached row, and ``sum_j w_j W_uv,h c_j = W_uv,h sum_j w_j c_j``,
    so the attention kernel returns weighted sums of latents (the cached row's first ``kv_rank`` channels are its value)
    that ``W_uv,h`` then lifts to the head's values. To the kernel this is attention of ``H`` query heads over one key
    head whose values lie inside its keys (``ops.core.attention_generic`` with ``values_in_keys``).

    Long portions of prompts go the other way where they can (bf16, a window, no rotated part, sizes that the kernels
    cover): of every row that brings at least ``LIFT_FROM_TOKENS`` tokens, the latents that its queries see are lifted to keys
    and values per head once (``ops.fast.latent_expand_bf16``), and attention is the ordinary one over heads of ``hd`` and
    ``value_dim`` channels: a score and its value cost ``hd + value_dim`` multiply-adds instead of twice ``kv_rank``. The other rows
    of the step (decoded tokens, short portions) stay with the latents. Which rows are which is decided on the device, so a
    captured step serves any of its size; a step that is launched kernel by kernel leaves out the half that has no row."""

    replays_every_step = True
    # Tokens a row brings from which its visible latents are lifted. Lifting costs kv_rank (hd + value_dim) a key and head,
    # attention over the latents (2 kv_rank - hd - value_dim) more a key, head and query: even at about kv_rank / 8 queries for
    # heads of a quarter of the latent, and the wide form of the kernel computes scores several times over.
    LIFT_FROM_TOKENS = 64

    def __init__(self, spec: LatentAttentionSpec) -> None:
        super().__init__(spec)
        self.position = build_part("position", spec.position)
        self.q_head = spec.head_dim + spec.rot_dim
        self.q_dim = spec.n_heads * self.q_head
        self.row_dim = spec.kv_rank + spec.rot_dim              # a cached row, and a query head as the kernel sees it
        self.out_dim = spec.n_heads * spec.value_dim
        self.gated = bool(spec.output_gate)
        self.gate_per_head = self.gated and bool(getattr(spec, "gate_per_head", False))
        self.gate_dim = (spec.n_heads if self.gate_per_head else self.out_dim) if self.gated else 0
        self.window = getattr(spec, "window", None)
        self.q_latent = spec.q_rank is not None
        self.q_cols = spec.q_rank if self.q_latent else self.q_dim      # columns of the first linear that the queries come from
        used = self.q_cols + self.row_dim + self.gate_dim
        # (rows of the projected buffer start on multiples of 16 bytes: what is missing is filled with weight rows of zeros)
        self.down_dim = used if self.gate_dim == self.out_dim else -(-used // 8) * 8
        self.down_weight = self.uq_weight = self.absorb = self.lift = self.proj_weight = None
        self._q_gain = self._kv_gain = self._sinks = self._freqs = None
        self._pairing = "halves"
        self.lift_weight: Optional[torch.Tensor] = None         # [W_uk; W_uv] where portions may be lifted
        self.dtype: Optional[torch.dtype] = None

    def params(self) -> Dict[str, ParamSpec]:
        spec = self.spec
        if self.q_latent:
            out = {"dq.weight": ParamSpec((spec.q_rank, spec.dim)), "dq_norm.weight": ParamSpec((spec.q_rank,), "vector", "gain"),
                   "uq.weight": ParamSpec((self.q_dim, spec.q_rank))}
        else:
            out = {"q.weight": ParamSpec((self.q_dim, spec.dim))}
        out.update({"dkv.weight": ParamSpec((self.row_dim, spec.dim)),
               "dkv_norm.weight": ParamSpec((spec.kv_rank,), "vector", "gain"),
               "uk.weight": ParamSpec((spec.n_heads * spec.head_dim, spec.kv_rank)),
               "uv.weight": ParamSpec((self.out_dim, spec.kv_rank)), "proj.weight": ParamSpec((spec.dim, self.out_dim))})
        if spec.head_sinks:
            out["sink"] = ParamSpec((spec.n_heads,), "vector", "bias")
        if self.gated:
            out["gate.weight"] = ParamSpec((self.gate_dim, spec.dim))
        return out

    def cache_spec(self) -> LatentCacheSpec:
        return LatentCacheSpec(self.spec.kv_rank, self.spec.rot_dim, self.window)

    def bind(self, tensors, dtype, device) -> None:
        spec = self.spec
        self.dtype = dtype
        names = ["dq.weight" if self.q_latent else "q.weight", "dkv.weight"] + (["gate.weight"] if self.gated else [])
        # one launch projects the queries or their latent, the key/value latent with the shared key part, and the gate
        rows = [tensors[name].to(device) for name in names]
        missing = self.down_dim - sum(r.shape[0] for r in rows)
        if missing:
            rows.append(torch.zeros((missing, spec.dim), dtype=rows[0].dtype, device=device))
        self.down_weight = torch.cat(rows, dim=0).contiguous()
        if self.q_latent:
            self.uq_weight = tensors["uq.weight"].to(device).contiguous()
            self._q_gain = tensors["dq_norm.weight"].to(device=device, dtype=torch.float32).contiguous()
        # W_uk per head, transposed: [H, kv_rank, hd] (a linear's weight for q_plain -> latent space)
        self.absorb = tensors["uk.weight"].to(device).view(spec.n_heads, spec.head_dim, spec.kv_rank).transpose(1, 2).contiguous()
        self.lift = tensors["uv.weight"].to(device).view(spec.n_heads, spec.value_dim, spec.kv_rank).contiguous()
        if dtype == torch.bfloat16 and self.window is not None and not spec.rot_dim and not spec.head_sinks \
                and (self.gate_per_head or not self.gated) and spec.scale > 0:
            from ..ops import fast
            if fast.latent_expand_supported(spec.n_heads, spec.head_dim, spec.value_dim, spec.kv_rank, self.row_dim):
                self.lift_weight = torch.cat([tensors["uk.weight"].to(device), tensors["uv.weight"].to(device)], dim=0).contiguous()
        self.proj_weight = tensors["proj.weight"].to(device).contiguous()
        self._kv_gain = tensors["dkv_norm.weight"].to(device=device, dtype=torch.float32).contiguous()
        if spec.head_sinks:
            self._sinks = tensors["sink"].to(device=device, dtype=torch.float32).contiguous()
        if int(getattr(self.position, "axes", 1)) != 1:
            raise ValueError("latent attention rotates by a token's place in the sequence")
        rotation = self.position.rotation(device)
        if rotation is not None:
            if getattr(rotation, "frequencies", None) is None:
                raise ValueError("latent attention takes a rotation given by frequencies")
            if rotation.pairing not in core.ROTARY_PAIRINGS or 2 * rotation.frequencies.numel() > spec.rot_dim:
                raise ValueError(f"latent attention cannot apply this rotation to a part of {spec.rot_dim} channels")
            self._freqs, self._pairing = rotation.frequencies.to(device).contiguous(), rotation.pairing

    def query_tile(self) -> Optional[int]:
        if self.dtype != torch.bfloat16:
            return None                     # the generic kernel takes tokens one by one
        from ..ops import fast
        return fast.biased_query_block(self.row_dim, self.spec.kv_rank)

    def input_projection(self):
        return self.down_weight, None, self.down_dim

    def output_projection(self):
        return self.proj_weight, None

    def attend(self, down, batch, cache: LayerCache, beside=None) -> torch.Tensor:
        """From the projected row ``[c_q' or q | c' | k_r | gate]`` to the gated heads, the input of the output projection."""
        spec = self.spec
        n = down.shape[0]
        ws = batch.workspace
        group = batch.groups[cache.group]
        slots = group.slots if cache.writes else None
        cq = ws.get("latent.cq", (n, spec.q_rank), self.dtype) if self.q_latent else None
        core.latent_prepare(down, 0, spec.q_rank if self.q_latent else 0, self._q_gain, cq, self.q_cols, spec.kv_rank, self._kv_gain,
                            spec.rot_dim, self._freqs, self._pairing, batch.positions, slots, cache.k, spec.eps)
        if self.q_latent:
            q = ws.get("latent.q", (n, self.q_dim), self.dtype)
            linear(cq, self.uq_weight, None, q)
        else:
            q = down[:, :self.q_dim]
        gate_at = self.q_cols + self.row_dim
        gate = down[:, gate_at:gate_at + self.gate_dim] if self.gated else None
        heads = ws.get("latent.heads", (n, self.out_dim), self.dtype)
        plan, some_stay = self._lift_plan(batch, cache, group)
        if plan is not None:
            self._attend_lifted(q, gate, batch, cache, plan, heads)
            if not some_stay:
                return heads
        full = ws.get("latent.q_full", (n, spec.n_heads * self.row_dim), self.dtype)
        skip = plan.lifted if plan is not None else None
        if spec.rot_dim:
            core.rotate_tail(q, full, spec.n_heads, spec.head_dim, spec.rot_dim, spec.kv_rank, self._freqs, self._pairing, batch.positions)
        self._per_head(q, self.q_head, spec.head_dim, self.absorb, full, self.row_dim, spec.kv_rank, skip=skip)
        mixed = ws.get("latent.mixed", (n, spec.n_heads * spec.kv_rank), self.dtype)
        # (a number per head scales a head's weighted latents as well as its values: the attention kernel applies it)
        inside = gate if self.gate_per_head else None
        kv_lo = group.kv_lo if self.window is not None else None
        done = False
        if self.dtype == torch.bfloat16:
            from ..ops import fast
            done = fast.attention_latent_bf16(full, cache.k, group.block_table, batch.token_row, batch.kv_hi, mixed, float(spec.scale),
                                              spec.n_heads, self.row_dim, spec.kv_rank, self._sinks, batch, kv_lo=kv_lo, head_gate=inside,
                                              row_tokens=None if plan is None else (0, plan.row_tokens))
        if not done:
            core.attention_generic(full, cache.k, None, group.block_table, batch.token_row, group.kv_lo, batch.kv_hi, mixed,
                                   float(spec.scale), spec.n_heads, 1, self.row_dim, spec.kv_rank, sinks=self._sinks,
                                   values_in_keys=True, gate=inside, gate_per_head=inside is not None)
        gate = None if self.gate_per_head else gate
        if not self._per_head(mixed, spec.kv_rank, spec.kv_rank, self.lift, heads, spec.value_dim, spec.value_dim, gate, skip=skip) \
                and gate is not None:
            core.gate_mul(heads, gate)
        return heads

    def _lift_plan(self, batch, cache: LayerCache, group):
        """``(plan, some rows stay)``: which rows' latents are lifted in this step (made once a step and cache group), or ``None``
        where none is."""
        if self.lift_weight is None or batch.decode_only or batch.n_tokens < self.LIFT_FROM_TOKENS or group.page_size != 16 \
                or not self._stays_in_fast_kernels(batch):
            return None, True
        # (what a step that is launched kernel by kernel brings; nothing is known of a captured one)
        brings = batch.host.get("q_lens") if batch.host else None
        if brings and max(brings) < self.LIFT_FROM_TOKENS:
            return None, True
        some_stay = not brings or min(brings) < self.LIFT_FROM_TOKENS
        made, key = batch.host.setdefault("made_once", {}), f"latent.lift_plan.{cache.group}"
        if key not in made:
            from ..ops import fast
            made[key] = fast.latent_expand_plan(batch, group, str(cache.group), int(self.window), self.LIFT_FROM_TOKENS,
                                                int(cache.k.shape[0]))
        return made[key], some_stay

    def _stays_in_fast_kernels(self, batch) -> bool:
        """Whether the rows that are not lifted run in kernels that pass over the lifted ones: a list of blocks of queries of
        the size the attention kernel takes, and sizes the per-head linears cover."""
        tile = self.query_tile()
        return tile is not None and tile in (batch.query_blocks or {}) and self.spec.head_dim % 16 == 0 and self.spec.kv_rank % 16 == 0 \
            and self.down_dim % 8 == 0 and self.spec.value_dim % 4 == 0

    def _attend_lifted(self, q, gate, batch, cache: LayerCache, plan, heads) -> None:
        """The lifted rows of the step: their keys and values, then ordinary attention into their rows of ``heads``."""
        from ..ops import fast
        spec = self.spec
        group = batch.groups[cache.group]
        keys, values = fast.latent_expand_bf16(cache.k, self.lift_weight, plan, spec.n_heads, spec.head_dim, spec.value_dim, spec.kv_rank,
                                               batch.workspace)
        if not fast.attention_biased_bf16(q, keys, values, plan.table, batch.token_row, group.kv_lo, batch.kv_hi, heads, float(spec.scale),
                                          spec.n_heads, spec.n_heads, spec.head_dim, spec.value_dim, None, None, None, batch, gate=gate,
                                          gate_per_head=self.gate_per_head, row_tokens=(plan.row_tokens, 0x7fffffff)):
            raise RuntimeError("the attention kernel declined sizes that latents were lifted for")

    def _per_head(self, a, a_head: int, k: int, weights, out, out_head: int, n_out: int, gate=None, skip=None) -> bool:
        """``out[:, h, :n_out] = a[:, h, :k] @ weights[h].T`` for every head (rows of ``a`` hold heads of ``a_head`` channels, rows of
        ``out`` heads of ``out_head``; rows with a number in ``skip`` are left alone). True: the outputs were also multiplied by the
        sigmoid of ``gate``."""
        if self.dtype == torch.bfloat16:
            from ..ops import fast
            if fast.heads_linear_bf16(a, a_head, k, weights, out, out_head, n_out, gate, skip=skip):
                return gate is not None
        if skip is not None:
            raise RuntimeError("the linear per head declined sizes that latents were lifted for")
        for h in range(self.spec.n_heads):
            linear(a[:, h * a_head:h * a_head + k], weights[h], None, out[:, h * out_head:h * out_head + n_out])
        return False

    def mix(self, h, batch, cache: LayerCache, out, accumulate: bool) -> None:
        down = batch.workspace.get("latent.down", (h.shape[0], self.down_dim), self.dtype)
        linear(h, self.down_weight, None, down)
        linear(self.attend(down, batch, cache), self.proj_weight, None, out, accumulate=accumulate)

    def forward(self, h, batch, cache: LayerCache, residual) -> None:
        self.mix(h, batch, cache, residual, True)


register_mixer("latent_attention", LatentAttention)
