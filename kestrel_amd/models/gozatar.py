"""Gozatar: a small decoder whose residual stream is several copies (hyper-connections) and whose every layer mixes tokens by
windowed attention behind short convolutions beside gated linear attention, followed by a dense feed-forward or a routed
mixture of clamped experts.

The design, in this file's notation (``w`` the width, ``eps`` the one epsilon of all norms, ``rms(x) = x / sqrt(mean(x^2) + eps)``,
``ln(x) = (x - mean) / sqrt(var + eps)``):

* Each of the ``streams`` copies ``x_s`` starts as ``embed[token]``. A sublayer with the numbers ``a`` (``hc<q>.in``), ``b``
  (``hc<q>.out``) and ``M`` (``hc<q>.mix``, from and to) computes ``y = f(ln(sum_s a_s x_s) norm<q>)``, and then all at once
  ``x_t <- sum_s M[s, t] x_s + b_t y``. A layer is its mixer (``q`` = 1) and its feed-forward (``q`` = 2; a layer whose ``mlp`` is null
  has none). Logits are ``head (ln(sum_s x_s) final.norm)``.
* Layer type ``parallel``: ``left_scale * left(h) + right_scale * right(h)``.
  ``left``: attention of ``heads`` query heads over ``kv_heads`` key/value heads, keys of ``dim`` and values of ``vdim`` channels, no
  biases. Every channel of q, k and v passes a causal convolution of ``conv`` taps over time; then the first ``rot.dims`` channels
  of every query and key head are rotated (channel ``i`` with ``i + dims / 2``, angle ``place * base^(-2i / dims)``), and the head is
  divided by its root mean square. Score ``scale * (q . k)``; place ``i`` sees ``j`` with ``0 <= i - j < mask.size`` (no ``mask``: every
  ``j <= i``); an ordinary softmax.
  ``right``: ``parts/gated_linear_attention.py`` with ``tau``.
* ``mlp`` of kind ``dense``: ``down(gelu_tanh(up h))``. Of kind ``moe``: ``parts/experts.py`` with sigmoid scores, groups that count by
  their two best choice scores (``router.groups``), experts with clamps (``expert.limit``; slope 1.702, shift 1) and a shared expert
  of the same form without a gate.

Every size and constant above that is not a literal comes from ``config.json`` or from a tensor's shape. Tensor names: ``embed``,
``l<i>.{norm1,norm2}``, ``l<i>.hc{1,2}.{in,out,mix}``, ``l<i>.mix.left.{q,k,v,o}``, ``l<i>.mix.left.{q,k,v}.conv``,
``l<i>.mix.right.{q,k,v,g,o,norm,a1,a2,a2.b}``, ``l<i>.mlp.{up,down}``, ``l<i>.mlp.e<j>.{gate,up,down}``, ``l<i>.mlp.{router,correction}``,
``l<i>.mlp.shared.{gate,up,down}``, ``final.norm``, ``head``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..config.registry import ModelSpec, register
from ..parts.specs import (AttentionSpec, BranchesSpec, DenseFeedForwardSpec, GatedLinearAttentionSpec, GateClamp, LayerSpec, ModelPlan,
                           NormSpec, PositionSpec, QKNorm, RoutedExpertsSpec, ScheduleEntry, StreamMixSpec)

NAME = "gozatar"
DENSE_ACTIVATION = "gelu_tanh"
GATE_SLOPE = 1.702             # an expert's gate is g * sigmoid(1.702 g)
VALUE_SHIFT = 1.0              # and multiplies u + 1
GROUP_BEST = 2                 # a group of experts counts by its two largest choice scores
# The design has no longest sequence of its own (angles are computed, no table depends on one). ``config.json`` may name a
# bound (``max_positions``); without one this stands, and the engine's ``max_seq_len`` narrows it.
DEFAULT_MAX_POSITIONS = 1 << 17


def _positive_int(where: str, value) -> int:
    if isinstance(value, bool) or not isinstance(value, int) or value <= 0:
        raise ValueError(f"config.json: {where} must be a positive integer, got {value!r}")
    return value


def _number(where: str, value) -> float:
    if isinstance(value, bool) or not isinstance(value, (int, float)):
        raise ValueError(f"config.json: {where} must be a number, got {value!r}")
    return float(value)


def _positive(where: str, value) -> float:
    number = _number(where, value)
    if not number > 0:
        raise ValueError(f"config.json: {where} must be positive, got {value!r}")
    return number


def _object(where: str, value, keys=()) -> dict:
    if not isinstance(value, dict):
        raise ValueError(f"config.json: {where} must be an object")
    for key in keys:
        if key not in value:
            raise ValueError(f"config.json: {where}.{key} missing")
    return value


@dataclass(frozen=True)
class GozatarAttention:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    conv: Optional[int]
    window: Optional[int]
    rot_dims: int
    rot_base: float

    @classmethod
    def read(cls, where: str, m: dict) -> "GozatarAttention":
        _object(where, m, ("heads", "kv_heads", "dim", "vdim", "scale", "rot"))
        heads, kv_heads = _positive_int(f"{where}.heads", m["heads"]), _positive_int(f"{where}.kv_heads", m["kv_heads"])
        if heads % kv_heads:
            raise ValueError(f"config.json: {where}: {heads} heads are no multiple of {kv_heads} kv_heads")
        dim = _positive_int(f"{where}.dim", m["dim"])
        rot = _object(f"{where}.rot", m["rot"], ("base", "dims"))
        dims = _positive_int(f"{where}.rot.dims", rot["dims"])
        if dims % 2 or dims > dim:
            raise ValueError(f"config.json: {where}.rot.dims must be even and at most dim, got {dims}")
        conv, mask = m.get("conv"), m.get("mask")
        return cls(heads, kv_heads, dim, _positive_int(f"{where}.vdim", m["vdim"]), _number(f"{where}.scale", m["scale"]),
                   None if conv is None else _positive_int(f"{where}.conv", conv),
                   None if mask is None else _positive_int(f"{where}.mask.size", _object(f"{where}.mask", mask, ("size",))["size"]),
                   dims, _number(f"{where}.rot.base", rot["base"]))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "kv_heads": self.kv_heads, "dim": self.dim, "vdim": self.vdim, "scale": self.scale,
                               "rot": {"base": self.rot_base, "dims": self.rot_dims}}
        if self.conv is not None:
            out["conv"] = self.conv
        if self.window is not None:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class GozatarRecurrence:
    heads: int
    dim: int
    vdim: int
    tau: float
    decay_rank: Optional[int] = None           # (not a key of the design: only the writer of random weights needs it)

    @classmethod
    def read(cls, where: str, m: dict) -> "GozatarRecurrence":
        _object(where, m, ("heads", "dim", "vdim", "tau"))
        rank = m.get("decay_rank")
        return cls(_positive_int(f"{where}.heads", m["heads"]), _positive_int(f"{where}.dim", m["dim"]), _positive_int(f"{where}.vdim", m["vdim"]),
                   _positive(f"{where}.tau", m["tau"]), None if rank is None else _positive_int(f"{where}.decay_rank", rank))

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "tau": self.tau}
        if self.decay_rank is not None:
            out["decay_rank"] = self.decay_rank
        return out


@dataclass(frozen=True)
class GozatarExperts:
    experts: int
    ff: int
    limit: float
    top: int
    groups: Optional[Tuple[int, int]]          # (count, keep)
    shared: Optional[Tuple[int, float]]        # (ff, limit)

    @classmethod
    def read(cls, where: str, m: dict) -> "GozatarExperts":
        _object(where, m, ("expert", "router"))
        expert = _object(f"{where}.expert", m["expert"], ("ff", "limit"))
        r = _object(f"{where}.router", m["router"], ("experts", "top"))
        experts, top = _positive_int(f"{where}.router.experts", r["experts"]), _positive_int(f"{where}.router.top", r["top"])
        groups = r.get("groups")
        allowed = experts
        if groups is not None:
            _object(f"{where}.router.groups", groups, ("count", "keep"))
            groups = (_positive_int(f"{where}.router.groups.count", groups["count"]), _positive_int(f"{where}.router.groups.keep", groups["keep"]))
            if experts % groups[0] or groups[1] > groups[0]:
                raise ValueError(f"config.json: {where}.router.groups: {groups[0]} groups must divide the {experts} experts and hold the "
                                 f"{groups[1]} that are kept")
            allowed = experts // groups[0] * groups[1]
        if top > allowed:
            raise ValueError(f"config.json: {where}.router.top {top} exceeds the {allowed} experts that can be chosen")
        shared = m.get("shared")
        if shared is not None:
            _object(f"{where}.shared", shared, ("ff", "limit"))
            shared = (_positive_int(f"{where}.shared.ff", shared["ff"]), _positive(f"{where}.shared.limit", shared["limit"]))
        return cls(experts, _positive_int(f"{where}.expert.ff", expert["ff"]), _positive(f"{where}.expert.limit", expert["limit"]), top, groups, shared)

    def to_dict(self) -> Dict[str, Any]:
        router: Dict[str, Any] = {"experts": self.experts, "top": self.top}
        if self.groups is not None:
            router["groups"] = {"count": self.groups[0], "keep": self.groups[1]}
        out: Dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff, "limit": self.limit}, "router": router}
        if self.shared is not None:
            out["shared"] = {"ff": self.shared[0], "limit": self.shared[1]}
        return out


@dataclass(frozen=True)
class GozatarLayer:
    left: GozatarAttention
    right: GozatarRecurrence
    left_scale: float
    right_scale: float
    dense_ff: Optional[int]                    # hidden size of a dense feed-forward
    experts: Optional[GozatarExperts]          # or a routed one; neither: the layer has no feed-forward

    @classmethod
    def read(cls, where: str, entry: dict) -> "GozatarLayer":
        _object(where, entry, ("type", "mixer"))
        if entry["type"] != "parallel":
            raise ValueError(f"config.json: {where}.type is {entry['type']!r}; this design has the mixer 'parallel'")
        m = _object(f"{where}.mixer", entry["mixer"], ("left", "right", "left_scale", "right_scale"))
        mlp = entry.get("mlp")
        ff = experts = None
        if mlp is not None:
            kind = _object(f"{where}.mlp", mlp, ("kind",))["kind"]
            if kind == "dense":
                ff = _positive_int(f"{where}.mlp.ff", mlp.get("ff"))
            elif kind == "moe":
                experts = GozatarExperts.read(f"{where}.mlp", mlp)
            else:
                raise ValueError(f"config.json: {where}.mlp.kind is {kind!r}; this design has the kinds 'dense' and 'moe'")
        return cls(GozatarAttention.read(f"{where}.mixer.left", m["left"]), GozatarRecurrence.read(f"{where}.mixer.right", m["right"]),
                   _number(f"{where}.mixer.left_scale", m["left_scale"]), _number(f"{where}.mixer.right_scale", m["right_scale"]), ff, experts)

    def to_dict(self) -> Dict[str, Any]:
        mlp = None
        if self.dense_ff is not None:
            mlp = {"kind": "dense", "ff": self.dense_ff}
        elif self.experts is not None:
            mlp = self.experts.to_dict()
        return {"type": "parallel", "mixer": {"left": self.left.to_dict(), "right": self.right.to_dict(), "left_scale": self.left_scale,
                                              "right_scale": self.right_scale}, "mlp": mlp}


@dataclass(frozen=True)
class GozatarConfig:
    vocab: int
    width: int
    eps: float
    streams: int
    max_positions: int
    layers: Tuple[GozatarLayer, ...]
    raw: Any = None

    @classmethod
    def from_dict(cls, config: Dict[str, Any]) -> "GozatarConfig":
        for key in ("layers", "vocab", "width", "norm", "streams"):
            if key not in config:
                raise ValueError(f"config.json: key {key!r} missing")
        eps = _number("norm.eps", _object("norm", config["norm"], ("eps",))["eps"])
        if not eps >= 0:
            raise ValueError("config.json: norm.eps must not be negative")
        listed = config["layers"]
        if not isinstance(listed, list) or not listed:
            raise ValueError("config.json: 'layers' must be a list of layers")
        positions = config.get("max_positions", DEFAULT_MAX_POSITIONS)
        return cls(vocab=_positive_int("vocab", config["vocab"]), width=_positive_int("width", config["width"]), eps=eps,
                   streams=_positive_int("streams", config["streams"]), max_positions=_positive_int("max_positions", positions),
                   layers=tuple(GozatarLayer.read(f"layers[{i}]", entry) for i, entry in enumerate(listed)), raw=config)

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"architecture": "Gozatar", "vocab": self.vocab, "width": self.width, "streams": self.streams,
                               "norm": {"eps": self.eps}, "layers": [layer.to_dict() for layer in self.layers]}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out


def _mixer(cfg: GozatarConfig, p: str, layer: GozatarLayer, names: Dict[str, str]) -> BranchesSpec:
    a, r = layer.left, layer.right
    left, right = p + "mix.left.", p + "mix.right."
    names.update({f"mixer.0.{s}.weight": left + s for s in ("q", "k", "v")})
    names["mixer.0.proj.weight"] = left + "o"
    if a.conv is not None:
        names.update({f"mixer.0.{s}.conv": f"{left}{s}.conv" for s in ("q", "k", "v")})
    names.update({f"mixer.1.{s}.weight": right + s for s in ("q", "k", "v", "norm", "a1", "a2")})
    names.update({"mixer.1.gate.weight": right + "g", "mixer.1.proj.weight": right + "o", "mixer.1.a2.bias": right + "a2.b"})
    rotation = PositionSpec("rotary", rotary_dim=a.rot_dims, theta=a.rot_base, pairing="halves")
    # (a norm without gains is the same before the rotation as behind it)
    attention = AttentionSpec("attention", cfg.width, a.heads, a.kv_heads, a.dim, rotation, bias=False, scale=a.scale, window=a.window,
                              value_dim=a.vdim, split_projections=True, qk_norm=QKNorm("head", cfg.eps, gain=False), conv_taps=a.conv)
    recurrence = GatedLinearAttentionSpec("gated_linear_attention", cfg.width, r.heads, r.dim, r.vdim, r.tau, cfg.eps, decay_rank=r.decay_rank)
    return BranchesSpec("branches", cfg.width, (attention, recurrence), (layer.left_scale, layer.right_scale), cfg.eps, norms=False)


def build_plan(cfg: GozatarConfig) -> ModelPlan:
    norm = NormSpec("layernorm", cfg.width, cfg.eps, bias=False)
    streams = StreamMixSpec("stream_mix", cfg.streams)
    layers = []
    ignored = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        names = {"norm.weight": p + "norm1", "streams.in": p + "hc1.in", "streams.out": p + "hc1.out", "streams.mix": p + "hc1.mix"}
        mixer = _mixer(cfg, p, layer, names)
        feed_forward = None
        if layer.dense_ff is not None:
            feed_forward = DenseFeedForwardSpec("dense", cfg.width, layer.dense_ff, DENSE_ACTIVATION, bias=False)
            names.update({"feed_forward.fc1.weight": p + "mlp.up", "feed_forward.fc2.weight": p + "mlp.down"})
        elif layer.experts is not None:
            e = layer.experts
            feed_forward = RoutedExpertsSpec(
                "routed_experts", cfg.width, e.experts, e.ff, e.top, n_groups=e.groups[0] if e.groups else 0,
                keep_groups=e.groups[1] if e.groups else 0, shared_hidden=e.shared[0] if e.shared else None, shared_gate=False,
                scores="sigmoid", group_best=GROUP_BEST, clamp=GateClamp(e.limit, GATE_SLOPE, VALUE_SHIFT),
                shared_clamp=GateClamp(e.shared[1], GATE_SLOPE, VALUE_SHIFT) if e.shared else None)
            for j in range(e.experts):
                names.update({f"feed_forward.e{j}.{s}.weight": f"{p}mlp.e{j}.{s}" for s in ("gate", "up", "down")})
            names.update({"feed_forward.router.weight": p + "mlp.router", "feed_forward.correction": p + "mlp.correction"})
            if e.shared:
                names.update({f"feed_forward.shared.{s}.weight": f"{p}mlp.shared.{s}" for s in ("gate", "up", "down")})
        has_ff = feed_forward is not None
        if has_ff:
            names.update({"norm2.weight": p + "norm2", "streams2.in": p + "hc2.in", "streams2.out": p + "hc2.out", "streams2.mix": p + "hc2.mix"})
        else:
            ignored += [p + "norm2", p + "hc2."]       # (a layer without a feed-forward has no use for its norm and numbers)
        layers.append(LayerSpec(arrangement="streams", norm=norm, mixer=mixer, feed_forward=feed_forward, norm2=norm if has_ff else None,
                                names=names, streams=streams, streams2=streams if has_ff else None))
    return ModelPlan(
        architecture=NAME, vocab_size=cfg.vocab, dim=cfg.width, max_positions=cfg.max_positions, layers=tuple(layers),
        schedule=tuple(ScheduleEntry(i) for i in range(len(layers))), final_norm=norm, head_bias=False, tied_head=False,
        names={"embedding": "embed", "final_norm.weight": "final.norm", "head.weight": "head"}, ignored_prefixes=tuple(ignored),
        streams=cfg.streams,
    )


def _claims(config: Dict[str, Any]) -> bool:
    layers = config.get("layers")
    return isinstance(layers, list) and bool(layers) and "width" in config and "streams" in config and \
        all(isinstance(e, dict) and e.get("type") == "parallel" and isinstance(e.get("mixer"), dict) for e in layers)


register(ModelSpec(
    name=NAME,
    read_config=GozatarConfig.from_dict,
    build_plan=build_plan,
    aliases=("Gozatar",),
    claims=_claims,
    filename="model.safetensors",
))
