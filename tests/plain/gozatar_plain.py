"""Plain implementation of the Gozatar decoder: float64, whole sequences, no cache, one function per mechanism.

It shares no code with the package: it reads the ``config.json`` dictionary and the stored tensors by their names.
For tokens ``t_0 .. t_{n-1}``:

* the state between sublayers is ``s`` streams ``X`` ``[s, n, width]``, all of them ``embed[t]`` at first
* a sublayer ``f`` with its norm and the numbers ``a`` (in) ``[s]``, ``b`` (out) ``[s]``, ``M`` (mix) ``[s, s]``: with
  ``y = f(norm(sum_s a_s X_s))`` the streams become ``X'_t = sum_s M[s, t] X_s + b_t y``
* a layer: the mixer, then the feed-forward (where it has one), each as such a sublayer
* mixer ``parallel``: ``left_scale * left(h) + right_scale * right(h)``, softmax attention over a window behind short
  convolutions beside a linear recurrence that decays channel by channel
* feed-forward: a dense one, or routed experts with a shared expert
* logits ``head norm(sum_s X_s)``.
"""

from __future__ import annotations

import math
from typing import Dict, Optional, Sequence, Tuple

import torch

F64 = torch.float64


def layer_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    centred = x - x.mean(dim=-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(dim=-1, keepdim=True) + eps) * weight


def rms(y: torch.Tensor, eps: float) -> torch.Tensor:
    return y / torch.sqrt((y * y).mean(dim=-1, keepdim=True) + eps)


def silu(z: torch.Tensor) -> torch.Tensor:
    return z * torch.sigmoid(z)


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---------------------------------------------------------------------------------------------- the streams
def read_streams(X: torch.Tensor, into: torch.Tensor) -> torch.Tensor:
    """``sum_s into[s] X[s]``."""
    return sum(into[s] * X[s] for s in range(X.shape[0]))


def write_streams(X: torch.Tensor, mix: torch.Tensor, out: torch.Tensor, y: torch.Tensor) -> torch.Tensor:
    """The new streams, all of them from the old ones: ``X'[t] = sum_s mix[s, t] X[s] + out[t] y``."""
    count = X.shape[0]
    return torch.stack([sum(mix[s, t] * X[s] for s in range(count)) + out[t] * y for t in range(count)])


# ---------------------------------------------------------------------------------------------- left: attention
def causal_conv(u: torch.Tensor, taps: torch.Tensor) -> torch.Tensor:
    """``y_t[c] = sum_j taps[c, j] u_(t - K + 1 + j)[c]`` for ``u`` ``[n, C]`` and ``taps`` ``[C, K]``; zeros before the start."""
    n, K = u.shape[0], taps.shape[1]
    y = torch.zeros_like(u)
    for t in range(n):
        for j in range(K):
            at = t - K + 1 + j
            if at >= 0:
                y[t] += taps[:, j] * u[at]
    return y


def rotate_halves(x: torch.Tensor, dims: int, base: float) -> torch.Tensor:
    """``x`` ``[n, heads, d]``, row ``p`` at place ``p``: channels ``i`` and ``i + dims / 2`` turned by ``p base^(-2i / dims)``."""
    out = x.clone()
    half = dims // 2
    for i in range(half):
        angle = torch.arange(x.shape[0], dtype=F64) * float(base) ** (-2.0 * i / dims)
        c, s = torch.cos(angle)[:, None], torch.sin(angle)[:, None]
        u, v = x[:, :, i], x[:, :, i + half]
        out[:, :, i] = u * c - v * s
        out[:, :, i + half] = v * c + u * s
    return out


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


def windowed_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """``p``: ``"l<i>.mix.left."``. Returns ``[n, width]``."""
    n = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])

    def projected(name: str) -> torch.Tensor:
        y = h @ w[p + name].T
        return causal_conv(y, w[p + name + ".conv"]) if m.get("conv") else y

    q, k, v = projected("q").reshape(n, H, d), projected("k").reshape(n, G, d), projected("v").reshape(n, G, dv)
    dims, base = int(m["rot"]["dims"]), float(m["rot"]["base"])
    q, k = rms(rotate_halves(q, dims, base), eps), rms(rotate_halves(k, dims, base), eps)
    seen = window_mask(n, int(m["mask"]["size"]) if m.get("mask") else None)
    out = torch.zeros(n, H, dv, dtype=F64)
    for a in range(H):
        g = a // (H // G)
        out[:, a] = softmax_over((q[:, a] @ k[:, g].T) * float(m["scale"]), seen) @ v[:, g]
    return out.reshape(n, H * dv) @ w[p + "o"].T


# ---------------------------------------------------------------------------------------------- right: the recurrence
def decays(z: torch.Tensor, tau: float) -> torch.Tensor:
    return torch.sigmoid(z) ** (1.0 / tau)


def gated_sum(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, alpha: torch.Tensor) -> torch.Tensor:
    """``q``, ``k``, ``alpha`` ``[n, H, d]``, ``v`` ``[n, H, dv]``: per head ``S <- diag(alpha_t) S + k_t v_t^T`` and then
    ``o_t = S^T q_t``, token by token from a zero state. Returns ``[n, H, dv]``."""
    n, H, d = q.shape
    out = torch.zeros(n, H, v.shape[2], dtype=F64)
    for h in range(H):
        state = torch.zeros(d, v.shape[2], dtype=F64)
        for t in range(n):
            state = alpha[t, h][:, None] * state + torch.outer(k[t, h], v[t, h])
            out[t, h] = q[t, h] @ state
    return out


def gated_linear_attention(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    """``p``: ``"l<i>.mix.right."``. Returns ``[n, width]``."""
    n = h.shape[0]
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    q = (h @ w[p + "q"].T).reshape(n, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).reshape(n, H, d)
    v = (h @ w[p + "v"].T).reshape(n, H, dv)
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    o = gated_sum(q, k, v, decays(z, float(m["tau"])).reshape(n, H, d))
    o = (rms(o, eps) * w[p + "norm"]).reshape(n, H * dv)         # (every head by itself, one gain for all)
    return (o * silu(h @ w[p + "g"].T)) @ w[p + "o"].T


def parallel(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict, eps: float) -> torch.Tensor:
    return float(m["left_scale"]) * windowed_attention(h, w, p + "left.", m["left"], eps) + \
        float(m["right_scale"]) * gated_linear_attention(h, w, p + "right.", m["right"], eps)


# ---------------------------------------------------------------------------------------------- feed-forward
def dense(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str) -> torch.Tensor:
    return gelu_tanh(h @ w[p + "up"].T) @ w[p + "down"].T


def expert(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, limit: float) -> torch.Tensor:
    """``p``: the expert's prefix without the last dot."""
    g = torch.clamp(h @ w[p + ".gate"].T, max=limit)
    u = torch.clamp(h @ w[p + ".up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[p + ".down"].T


def routing(z: torch.Tensor, correction: torch.Tensor, top: int, groups: Optional[Tuple[int, int]]) -> Tuple[torch.Tensor, torch.Tensor]:
    """Logits ``[n, E]`` -> the chosen experts ``[n, top]`` (best choice score first) and their weights."""
    s = torch.sigmoid(z)
    choice = s + correction
    if groups is not None:
        count, keep = groups
        n, E = z.shape
        per = E // count
        for t in range(n):
            scores = []
            for g in range(count):
                best = sorted(choice[t, g * per:(g + 1) * per].tolist(), reverse=True)[:2]
                scores.append(sum(best))
            kept = sorted(range(count), key=lambda g: -scores[g])[:keep]
            for g in range(count):
                if g not in kept:
                    choice[t, g * per:(g + 1) * per] = float("-inf")
    order = torch.sort(choice, dim=-1, descending=True, stable=True).indices[:, :top]
    chosen = torch.gather(s, 1, order)
    return order, chosen / (chosen.sum(dim=-1, keepdim=True) + 1e-20)


def experts(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    """``p``: ``"l<i>.mlp."``. Returns ``[n, width]``."""
    r = m["router"]
    groups = (int(r["groups"]["count"]), int(r["groups"]["keep"])) if r.get("groups") else None
    order, weights = routing(h @ w[p + "router"].T, w[p + "correction"], int(r["top"]), groups)
    limit = float(m["expert"]["limit"])
    out = torch.zeros_like(h)
    for e in range(int(r["experts"])):
        weight = (weights * (order == e)).sum(dim=-1)
        used = (order == e).any(dim=-1)
        if bool(used.any()):
            out[used] += weight[used][:, None] * expert(h[used], w, f"{p}e{e}", limit)
    if m.get("shared"):
        out = out + expert(h, w, p + "shared", float(m["shared"]["limit"]))
    return out


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], p: str, m: dict) -> torch.Tensor:
    return dense(h, w, p) if m["kind"] == "dense" else experts(h, w, p, m)


# ---------------------------------------------------------------------------------------------- the stack
def layer_step(X: torch.Tensor, w: Dict[str, torch.Tensor], i: int, layer: dict, eps: float) -> torch.Tensor:
    p = f"l{i}."
    y = parallel(layer_norm(read_streams(X, w[p + "hc1.in"]), w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps)
    X = write_streams(X, w[p + "hc1.mix"], w[p + "hc1.out"], y)
    if layer.get("mlp"):
        y = feed_forward(layer_norm(read_streams(X, w[p + "hc2.in"]), w[p + "norm2"], eps), w, p + "mlp.", layer["mlp"])
        X = write_streams(X, w[p + "hc2.mix"], w[p + "hc2.out"], y)
    return X


def forward(config: dict, weights: Dict[str, torch.Tensor], tokens: Sequence[int], layers_out: Optional[list] = None) -> torch.Tensor:
    """Logits ``[n, vocab]`` in float64. ``layers_out``: a list that gets the sum of the streams after every layer."""
    w = {name: t.to(F64) for name, t in weights.items()}
    eps = float(config["norm"]["eps"])
    x = w["embed"][torch.tensor(list(tokens), dtype=torch.long)]
    X = torch.stack([x.clone() for _ in range(int(config["streams"]))])
    for i, layer in enumerate(config["layers"]):
        X = layer_step(X, w, i, layer, eps)
        if layers_out is not None:
            layers_out.append(X.sum(dim=0))
    return layer_norm(X.sum(dim=0), w["final.norm"], eps) @ w["head"].T
