"""Mixers side by side: several mixers read the same input, their outputs, normalised or not, are summed with weights."""

from __future__ import annotations

from typing import Dict, List, Optional

import torch

from ..ops import core
from ..ops.linear import linear
from .base import LayerCache, Mixer, build_part, register_mixer
from .specs import BranchesSpec, ParamSpec, StateSpec


class Branches(Mixer):
    """``sum_i weights[i] * rms(branch_i(h)) * gain_i``: every branch is a mixer of any registered kind, built from its
    own specification; its output ``[n, dim]`` is divided by its root mean square over the model width (``eps``) and
    multiplied by a gain of its own (tensor ``out<i>.weight``) before the weighted sum enters the stream.

    With ``spec.norms`` off the sum is ``sum_i weights[i] * branch_i(h)``. Branches that offer their stages and take up
    their weights themselves (``Mixer.share_projections``, ``Mixer.fold_output_weight``) then run as one: one linear projects for all of
    them, each runs its core on its own columns, and one linear over what they return side by side is the sum.

    The tensors of branch ``i`` are named ``<i>.<local name>``. What the branches keep is the layer's: at most one of
    them may keep keys and values per token (a layer has one cache group); states per request lie side by side in the layer's
    one state tensor, each branch's on a multiple of 16 bytes, and each branch is handed its own part."""

    def __init__(self, spec: BranchesSpec) -> None:
        super().__init__(spec)
        if not spec.branches or len(spec.branches) != len(spec.weights) or len(spec.branches) > 2:
            raise ValueError("branches: one or two mixers, and a weight for each")
        self.branches: List[Mixer] = [build_part("mixer", b) for b in spec.branches]
        if sum(b.cache_spec() is not None for b in self.branches) > 1:
            raise ValueError("branches: at most one branch may keep a cache per token")
        states = [b.state_spec() for b in self.branches]
        if sum(s is not None for s in states) > 1 and any(s is not None and s.dtype != "float32" for s in states):
            raise ValueError("branches: states that lie side by side are fp32")
        self.normed = bool(getattr(spec, "norms", True))
        self.gains: List[Optional[torch.Tensor]] = [None] * len(self.branches)
        self.in_weight: Optional[torch.Tensor] = None       # of all branches (only where they run as one)
        self.proj_weight: Optional[torch.Tensor] = None
        self.dtype: Optional[torch.dtype] = None

    @property
    def replays_every_step(self) -> bool:
        return all(bool(getattr(b, "replays_every_step", False)) for b in self.branches)

    @property
    def position(self):
        """(the runner asks a mixer's position encoding how many numbers it takes per token)"""
        return next((getattr(b, "position", None) for b in self.branches if getattr(b, "position", None) is not None), None)

    def params(self) -> Dict[str, ParamSpec]:
        out = {}
        for i, branch in enumerate(self.branches):
            out.update({f"{i}.{name}": pspec for name, pspec in branch.params().items()})
            if self.normed:
                out[f"out{i}.weight"] = ParamSpec((self.spec.dim,), "vector", "gain")
        return out

    def bind(self, tensors, dtype, device) -> None:
        self.dtype = dtype
        for i, branch in enumerate(self.branches):
            branch.bind({name: tensors[f"{i}.{name}"] for name in branch.params()}, dtype, device)
            if self.normed:
                self.gains[i] = tensors[f"out{i}.weight"].to(device=device, dtype=torch.float32).contiguous()
        if not self.normed:
            self._join()

    def _join(self) -> None:
        ins = [b.input_projection() for b in self.branches]
        outs = [b.output_projection() for b in self.branches]
        if any(stage is None or stage[1] is not None for stage in ins + outs):
            return
        if any(type(b).share_projections is Mixer.share_projections for b in self.branches):
            return
        # (asked of all before any is changed: the weights are either all taken up or all applied to what the branches give)
        if not all(b.takes_output_weight(float(w)) for b, w in zip(self.branches, self.spec.weights)):
            return
        for b, w in zip(self.branches, self.spec.weights):
            b.fold_output_weight(float(w))
        self.in_weight = torch.cat([stage[0] for stage in ins], dim=0).contiguous()
        self.proj_weight = torch.cat([stage[0] for stage in outs], dim=1).contiguous()
        self.in_cols, self.out_cols = [0], [0]
        for b, first, last in zip(self.branches, ins, outs):
            self.in_cols.append(self.in_cols[-1] + first[2])
            self.out_cols.append(self.out_cols[-1] + last[0].shape[1])
            b.share_projections(self.in_weight[self.in_cols[-2]:self.in_cols[-1]], self.proj_weight[:, self.out_cols[-2]:self.out_cols[-1]])

    def cache_spec(self):
        return next((b.cache_spec() for b in self.branches if b.cache_spec() is not None), None)

    def _state_places(self):
        """Per branch the first number of its state in the layer's, or ``None``; and how many numbers there are in all."""
        places, at = [], 0
        for branch in self.branches:
            state = branch.state_spec()
            places.append(None if state is None else at)
            if state is not None:
                count = 1
                for extent in state.shape:
                    count *= int(extent)
                at += (count + 3) // 4 * 4
        return places, at

    def state_spec(self):
        states = [b.state_spec() for b in self.branches if b.state_spec() is not None]
        if len(states) <= 1:
            return states[0] if states else None
        return StateSpec((self._state_places()[1],), "float32")

    def _cache_of(self, i: int, cache: LayerCache) -> LayerCache:
        """The layer's cache as branch ``i`` sees it."""
        state = self.branches[i].state_spec()
        if state is None or cache.state is None or sum(b.state_spec() is not None for b in self.branches) <= 1:
            return cache
        place = self._state_places()[0][i]
        count = 1
        for extent in state.shape:
            count *= int(extent)
        view = cache.state[:, place:place + count]
        return LayerCache(cache.group, cache.tensors, cache.writes, view if len(state.shape) == 1 else view.unflatten(1, state.shape))

    def query_tile(self):
        return next((b.query_tile() for b in self.branches if b.query_tile()), None)

    def mix(self, h, batch, cache: LayerCache, out, accumulate: bool) -> None:
        """The mixer's output written into (or added to) fp32 ``out``."""
        n = h.shape[0]
        if self.in_weight is not None:
            projected = batch.workspace.get("branches.in", (n, self.in_cols[-1]), self.dtype)
            linear(h, self.in_weight, None, projected)
            heads = batch.workspace.get("branches.heads", (n, self.out_cols[-1]), self.dtype)
            for i, branch in enumerate(self.branches):
                branch.attend(projected[:, self.in_cols[i]:self.in_cols[i + 1]], batch, self._cache_of(i, cache),
                              out=heads[:, self.out_cols[i]:self.out_cols[i + 1]])
            linear(heads, self.proj_weight, None, out, accumulate=accumulate)
            return
        if not accumulate:
            out.zero_()                  # (a fill kernel)
        self.forward(h, batch, cache, out)

    def forward(self, h, batch, cache: LayerCache, residual) -> None:
        if self.in_weight is not None:
            self.mix(h, batch, cache, residual, True)
            return
        n = h.shape[0]
        outs = []
        for i, branch in enumerate(self.branches):
            out = batch.workspace.get(f"branches.out{i}", (n, self.spec.dim), torch.float32)
            mix = getattr(branch, "mix", None)
            own = self._cache_of(i, cache)
            if callable(mix):
                mix(h, batch, own, out, False)
            else:
                out.zero_()              # (a fill kernel: a mixer that only knows how to add)
                branch.forward(h, batch, own, out)
            outs.append(out)
        if not self.normed:
            for out, weight in zip(outs, self.spec.weights):
                core.add_scaled(residual, out, float(weight))
            return
        second = len(outs) > 1
        core.branches_sum(residual, outs[0], self.gains[0], self.spec.weights[0], outs[1] if second else None,
                          self.gains[1] if second else None, self.spec.weights[1] if second else 0.0, self.spec.eps)


register_mixer("branches", Branches)
