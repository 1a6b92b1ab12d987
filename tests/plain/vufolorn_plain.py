"""Plain implementation of the Vufolorn decoder: float64, whole sequences, no cache, one function per mechanism.

It shares no code with the package: it reads the ``config.json`` dictionary and the stored tensors by their names.
For tokens ``t_0 .. t_{n-1}`` (``rms(y) = y / sqrt(mean(y^2) + eps)``):

* ``x = rms(embed[t_p]) * embed.norm``, kept as ``x0``
* the runs of ``loop``: its layers several times over, each pass begun by ``x <- x + x0`` (not the first pass) and
  ``x <- x + loop.step[pass]``
* a layer: ``x <- x + ls1 * (rms(mixer(rms(x) norm1)) norm1b)``, then the same with ``ff``, ``norm2``, ``norm2b``, ``ls2``
* mixer ``lightning``: a linear recurrence with one decay per head
* mixer ``latent_attention``: softmax attention over a window whose keys and values are lifted from one latent a token
* ``ff``: routed experts, weights by a softmax over the chosen, and a shared expert behind a gate
* logits ``embed @ (rms(x) final.norm)``.
"""

from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch

F64 = torch.float64


def rms(y: torch.Tensor, eps: float) -> torch.Tensor:
    return y / torch.sqrt((y * y).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def relu_squared(z: torch.Tensor) -> torch.Tensor:
    return torch.clamp(z, min=0.0) ** 2


# ---------------------------------------------------------------------------------------------- linear recurrence
def decayed_sum(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, decay: Sequence[float]) -> torch.Tensor:
    """``q``, ``k`` ``[n, H, d]``, ``v`` ``[n, H, dv]``: per head ``S <- decay S + k v^T`` and then ``o = S^T q``, token by token
    from a zero state. Returns ``[n, H, dv]``."""
    n, H, d = q.shape
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    for h in range(H):
        state = torch.zeros(d, v.shape[2], dtype=F64)
        for t in range(n):
            state = float(decay[h]) * state + torch.outer(k[t, h], v[t, h])
            out[t, h] = q[t, h] @ state
    return out


def lightning(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """Mixer ``lightning``: returns ``[n, width]``."""
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = silu(h @ w[p + "q"].T).reshape(n, H, d)
    k = silu(h @ w[p + "k"].T).reshape(n, H, d)
    v = silu(h @ w[p + "v"].T).reshape(n, H, dv)
    o = decayed_sum(q, k, v, m["decay"]).reshape(n, H * dv)
    o = rms(o, eps) * w[p + "norm"]                          # one root mean square over all heads together
    return (o * torch.sigmoid(h @ w[p + "g"].T)) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- latent attention
def window_mask(n: int, size: Optional[int]) -> torch.Tensor:
    """``seen[i, j]``: ``0 <= i - j`` and, with a window, ``i - j < size``."""
    i = torch.arange(n)[:, None]
    j = torch.arange(n)[None, :]
    seen = j <= i
    if size is not None:
        seen = seen & (i - j < size)
    return seen


def softmax_over(scores: torch.Tensor, seen: torch.Tensor) -> torch.Tensor:
    s = scores.masked_fill(~seen, float("-inf"))
    e = torch.exp(s - s.max(dim=-1, keepdim=True).values)
    return e / e.sum(dim=-1, keepdim=True)


def latent_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """Mixer ``latent_attention``: returns ``[n, width]``."""
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[p + "q"].T).reshape(n, H, d)
    c = rms(h @ w[p + "dkv"].T, eps) * w[p + "dkv.norm"]
    k = (c @ w[p + "uk"].T).reshape(n, H, d)
    v = (c @ w[p + "uv"].T).reshape(n, H, dv)
    gate = torch.sigmoid(h @ w[p + "g"].T)                   # [n, H]
    seen = window_mask(n, int(m["mask"]["size"]) if m.get("mask") else None)
    out = torch.zeros(n, H, dv, dtype=F64)
    for a in range(H):
        weights = softmax_over((q[:, a] @ k[:, a].T) * float(m["scale"]), seen)
        out[:, a] = (weights @ v[:, a]) * gate[:, a:a + 1]
    return out.reshape(n, H * dv) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- feed-forward
def routing(z: torch.Tensor, top: int) -> Tuple[torch.Tensor, torch.Tensor]:
    """Logits ``[n, E]`` (bias included) -> the ``top`` largest of every row (``[n, top]``) and the softmax over those alone."""
    order = torch.sort(z, dim=-1, descending=True, stable=True).indices[:, :top]
    chosen = torch.gather(z, 1, order)
    e = torch.exp(chosen - chosen.max(dim=-1, keepdim=True).values)
    return order, e / e.sum(dim=-1, keepdim=True)


def expert(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return relu_squared(h @ w[p + ".up"].T) @ w[p + ".down"].T


def experts(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    """``p``: ``"l<i>.mlp."``. Returns ``[n, width]``."""
    z = h @ w[p + "router"].T + w[p + "router.b"]
    order, weights = routing(z, int(m["router"]["top"]))
    out = torch.zeros_like(h)
    for t in range(h.shape[0]):
        for slot in range(order.shape[1]):
            out[t] += weights[t, slot] * expert(h[t:t + 1], w, f"{p}e{int(order[t, slot])}")[0]
    if m.get("shared"):
        out = out + torch.sigmoid(h @ w[p + "shared.sg"].T) * expert(h, w, p + "shared")
    return out


# ---------------------------------------------------------------------------------------------- the stack
def runs_of(config: dict) -> List[Tuple[int, Optional[int]]]:
    """``(layer, pass)`` in the order of execution: ``pass`` is given for the first layer of every pass through the loop."""
    count = len(config["layers"])
    loop = config.get("loop")
    if not loop:
        return [(i, None) for i in range(count)]
    start, stop, times = int(loop["start"]), int(loop["stop"]), int(loop["times"])
    out: List[Tuple[int, Optional[int]]] = [(i, None) for i in range(start)]
    for t in range(times):
        out += [(i, t if i == start else None) for i in range(start, stop)]
    return out + [(i, None) for i in range(stop, count)]


def layer_step(x: torch.Tensor, w: Dict[str, torch.Tensor], i: int, layer: dict, eps: float) -> torch.Tensor:
    p = f"l{i}."
    mixer = {"lightning": lightning, "latent_attention": latent_attention}[layer["type"]]
    y = mixer(rms(x, eps) * w[p + "norm1"], w, p + "mix.", layer["mixer"], eps)
    x = x + rms(y, eps) * w[p + "norm1b"] * w[p + "ls1"]
    if layer.get("mlp"):
        y = experts(rms(x, eps) * w[p + "norm2"], w, p + "mlp.", layer["mlp"])
        x = x + rms(y, eps) * w[p + "norm2b"] * w[p + "ls2"]
    return x


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: Sequence[int], layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[n, vocab]`` in float64. ``layers_out``: a list that gets the stream after every layer run."""
    w = {name: t.to(F64) for name, t in weights.items()}
    eps = float(config["norm"]["eps"])
    x = rms(w["embed"][torch.tensor(list(tokens), dtype=torch.long)], eps) * w["embed.norm"]
    x0 = x.clone()
    for i, number in runs_of(config):
        if number is not None:
            if number > 0:
                x = x + x0
            x = x + w["loop.step"][number]
        x = layer_step(x, w, i, config["layers"][i], eps)
        if layers_out is not None:
            layers_out.append(x.clone())
    return (rms(x, eps) * w["final.norm"]) @ w["embed"].T
