"""Vufolorn: a small decoder whose layers mix tokens by a linear recurrence with a constant decay per head or by latent
attention over a window, each followed by a routed mixture of plain experts, with norms around every sublayer and a looped
stretch of layers.

The design, in this file's notation (``w`` the width, ``eps`` the one epsilon of all norms, ``rms(x) = x / sqrt(mean(x^2) + eps)``):

* ``x = rms(embed[token]) embed.norm``; this is also ``x0``.
* The layers ``start .. stop - 1`` of ``loop`` run ``times`` times in a row with the same weights and a cache or state of their
  own each time; pass ``t`` begins with ``x <- x + x0`` (``t > 0`` only) and ``x <- x + loop.step[t]``.
* A layer: ``x <- x + ls1 norm1b rms(mix(rms(x) norm1))``, then ``x <- x + ls2 norm2b rms(mlp(rms(x) norm2))``; a layer whose
  ``mlp`` is null has the first half only. Logits are ``embed (rms(x) final.norm)``.
* Layer type ``lightning``: ``parts/linear_attention.py`` with silu on queries, keys and values, ``decay`` a list of one number per
  head.
* Layer type ``latent_attention``: ``parts/latent_attention.py`` with queries projected directly, no rotated part, no sinks,
  ``scale`` on the scores, the keys ``0 <= i - j < mask.size`` seen (no ``mask``: every ``j <= i``), and a gate of one number per head.
* ``mlp`` (``kind`` ``moe``): ``parts/experts.py``; an expert is ``down(relu(up h)^2)``; the ``top`` largest of the logits
  ``router h + router.b`` are chosen, weighed by the softmax over them; a shared expert of ``shared.ff`` times
  ``sigmoid(shared.sg h)``, one number per token.

Every size and constant above that is not a literal comes from ``config.json`` or from a tensor's shape. Tensor names:
``embed``, ``embed.norm``, ``loop.step``, ``l<i>.{norm1,norm1b,ls1,norm2,norm2b,ls2}``, ``l<i>.mix.{q,k,v,g,o,norm}``,
``l<i>.mix.{q,dkv,dkv.norm,uk,uv,g,o}``, ``l<i>.mlp.e<j>.{up,down}``, ``l<i>.mlp.router``, ``l<i>.mlp.router.b``,
``l<i>.mlp.shared.{up,down,sg}``, ``final.norm``.
"""

from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, Optional, Tuple

from ..config.registry import ModelSpec, register
from ..parts.specs import (LatentAttentionSpec, LayerSpec, LinearAttentionSpec, ModelPlan, NormSpec, PassVectorSpec, PositionSpec,
                           RoutedExpertsSpec, ScheduleEntry)

NAME = "vufolorn"
RECURRENT_ACTIVATION = "silu"
EXPERT_ACTIVATION = "relu_squared"
EMBEDDING_FROM_PASS = 1                # the embedding output comes back before every pass but the first
KINDS = ("lightning", "latent_attention")
# The design has no positions and so no longest sequence of its own. ``config.json`` may name a bound
# (``max_positions``); without one this stands, and the engine's ``max_seq_len`` narrows it.
DEFAULT_MAX_POSITIONS = 1 << 17


def _positive_int(where: str, value) -> int:
    if isinstance(value, bool) or not isinstance(value, int) or value <= 0:
        raise ValueError(f"config.json: {where} must be a positive integer, got {value!r}")
    return value


def _natural(where: str, value) -> int:
    if isinstance(value, bool) or not isinstance(value, int) or value < 0:
        raise ValueError(f"config.json: {where} must be an integer that is not negative, got {value!r}")
    return value


def _number(where: str, value) -> float:
    if isinstance(value, bool) or not isinstance(value, (int, float)):
        raise ValueError(f"config.json: {where} must be a number, got {value!r}")
    return float(value)


def _object(where: str, value, keys=()) -> dict:
    if not isinstance(value, dict):
        raise ValueError(f"config.json: {where} must be an object")
    for key in keys:
        if key not in value:
            raise ValueError(f"config.json: {where}.{key} missing")
    return value


@dataclass(frozen=True)
class VufolornRecurrence:
    heads: int
    dim: int
    vdim: int
    decay: Tuple[float, ...]

    @classmethod
    def read(cls, where: str, m: dict) -> "VufolornRecurrence":
        _object(where, m, ("heads", "dim", "vdim", "decay"))
        heads = _positive_int(f"{where}.heads", m["heads"])
        listed = m["decay"]
        if not isinstance(listed, (list, tuple)) or len(listed) != heads:
            raise ValueError(f"config.json: {where}.decay must be a list of {heads} numbers, one per head")
        decay = tuple(_number(f"{where}.decay", a) for a in listed)
        if not all(0.0 < a <= 1.0 for a in decay):
            raise ValueError(f"config.json: {where}.decay must lie above 0 and at most at 1, got {list(decay)}")
        return cls(heads, _positive_int(f"{where}.dim", m["dim"]), _positive_int(f"{where}.vdim", m["vdim"]), decay)

    def to_dict(self) -> Dict[str, Any]:
        return {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "decay": list(self.decay)}


@dataclass(frozen=True)
class VufolornLatent:
    heads: int
    dim: int
    vdim: int
    kv_rank: int
    scale: float
    window: Optional[int]

    @classmethod
    def read(cls, where: str, m: dict) -> "VufolornLatent":
        _object(where, m, ("heads", "dim", "vdim", "kv_rank", "scale"))
        mask = m.get("mask")
        window = None if mask is None else _positive_int(f"{where}.mask.size", _object(f"{where}.mask", mask, ("size",))["size"])
        return cls(_positive_int(f"{where}.heads", m["heads"]), _positive_int(f"{where}.dim", m["dim"]),
                   _positive_int(f"{where}.vdim", m["vdim"]), _positive_int(f"{where}.kv_rank", m["kv_rank"]),
                   _number(f"{where}.scale", m["scale"]), window)

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"heads": self.heads, "dim": self.dim, "vdim": self.vdim, "kv_rank": self.kv_rank, "scale": self.scale}
        if self.window is not None:
            out["mask"] = {"size": self.window}
        return out


@dataclass(frozen=True)
class VufolornExperts:
    experts: int
    ff: int
    top: int
    shared_ff: Optional[int]

    @classmethod
    def read(cls, where: str, m: dict) -> "VufolornExperts":
        if not isinstance(m, dict) or m.get("kind") != "moe":
            raise ValueError(f"config.json: {where} must be null or an object of kind 'moe'")
        _object(where, m, ("expert", "router"))
        ff = _positive_int(f"{where}.expert.ff", _object(f"{where}.expert", m["expert"], ("ff",))["ff"])
        r = _object(f"{where}.router", m["router"], ("experts", "top"))
        experts, top = _positive_int(f"{where}.router.experts", r["experts"]), _positive_int(f"{where}.router.top", r["top"])
        if top > experts:
            raise ValueError(f"config.json: {where}.router.top {top} exceeds the {experts} experts")
        shared = m.get("shared")
        shared_ff = None if shared is None else _positive_int(f"{where}.shared.ff", _object(f"{where}.shared", shared, ("ff",))["ff"])
        return cls(experts, ff, top, shared_ff)

    def to_dict(self) -> Dict[str, Any]:
        out: Dict[str, Any] = {"kind": "moe", "expert": {"ff": self.ff}, "router": {"experts": self.experts, "top": self.top}}
        if self.shared_ff is not None:
            out["shared"] = {"ff": self.shared_ff}
        return out


@dataclass(frozen=True)
class VufolornLayer:
    kind: str                                  # "lightning" or "latent_attention"
    mixer: Any                                 # VufolornRecurrence or VufolornLatent
    mlp: Optional[VufolornExperts]


@dataclass(frozen=True)
class VufolornConfig:
    vocab: int
    width: int
    eps: float
    max_positions: int
    layers: Tuple[VufolornLayer, ...]
    loop_start: int
    loop_stop: int
    loop_times: Optional[int]          # None: no stretch of layers is repeated and there is no ``loop.step``
    raw: Any = None

    @classmethod
    def from_dict(cls, config: Dict[str, Any]) -> "VufolornConfig":
        for key in ("layers", "vocab", "width", "norm"):
            if key not in config:
                raise ValueError(f"config.json: key {key!r} missing")
        eps = _number("norm.eps", _object("norm", config["norm"], ("eps",))["eps"])
        if not eps >= 0:
            raise ValueError("config.json: norm.eps must not be negative")
        listed = config["layers"]
        if not isinstance(listed, list) or not listed:
            raise ValueError("config.json: 'layers' must be a list of layers")
        layers = []
        for i, entry in enumerate(listed):
            where = f"layers[{i}]"
            _object(where, entry, ("type", "mixer"))
            kind = entry["type"]
            if kind not in KINDS:
                raise ValueError(f"config.json: {where}.type is {kind!r}; this design has the mixers {', '.join(KINDS)}")
            mixer = (VufolornRecurrence if kind == "lightning" else VufolornLatent).read(f"{where}.mixer", entry["mixer"])
            mlp = entry.get("mlp")
            layers.append(VufolornLayer(kind, mixer, None if mlp is None else VufolornExperts.read(f"{where}.mlp", mlp)))
        loop = config.get("loop")
        start = stop = 0
        times = None
        if loop is not None:
            _object("loop", loop, ("start", "stop", "times"))
            start, stop, times = (_natural(f"loop.{key}", loop[key]) for key in ("start", "stop", "times"))
            if not start <= stop <= len(layers):
                raise ValueError(f"config.json: loop {start} .. {stop} does not lie within the {len(layers)} layers")
        positions = config.get("max_positions", DEFAULT_MAX_POSITIONS)
        return cls(vocab=_positive_int("vocab", config["vocab"]), width=_positive_int("width", config["width"]), eps=eps,
                   max_positions=_positive_int("max_positions", positions), layers=tuple(layers), loop_start=start, loop_stop=stop,
                   loop_times=times, raw=config)

    def to_dict(self) -> Dict[str, Any]:
        layers = [{"type": layer.kind, "mixer": layer.mixer.to_dict(), "mlp": None if layer.mlp is None else layer.mlp.to_dict()}
                  for layer in self.layers]
        out: Dict[str, Any] = {"architecture": "Vufolorn", "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps}, "layers": layers}
        if self.loop_times is not None:
            out["loop"] = {"start": self.loop_start, "stop": self.loop_stop, "times": self.loop_times}
        if self.max_positions != DEFAULT_MAX_POSITIONS:
            out["max_positions"] = self.max_positions
        return out


def _mixer(cfg: VufolornConfig, i: int, layer: VufolornLayer, names: Dict[str, str]):
    p = f"l{i}.mix."
    m = layer.mixer
    if layer.kind == "lightning":
        names.update({f"mixer.{s}.weight": p + s for s in ("q", "k", "v", "norm")})
        names.update({"mixer.gate.weight": p + "g", "mixer.proj.weight": p + "o"})
        return LinearAttentionSpec("linear_attention", cfg.width, m.heads, m.dim, m.vdim, m.decay, cfg.eps, activation=RECURRENT_ACTIVATION)
    names.update({f"mixer.{s}.weight": p + s for s in ("q", "dkv", "uk", "uv")})
    names.update({"mixer.dkv_norm.weight": p + "dkv.norm", "mixer.gate.weight": p + "g", "mixer.proj.weight": p + "o"})
    return LatentAttentionSpec("latent_attention", cfg.width, m.heads, m.dim, 0, m.vdim, None, m.kv_rank, m.scale, cfg.eps, PositionSpec("none"),
                               head_sinks=False, gate_per_head=True, window=m.window)


def build_plan(cfg: VufolornConfig) -> ModelPlan:
    before = NormSpec("rmsnorm", cfg.width, cfg.eps, bias=False)
    behind = NormSpec("rmsnorm", cfg.width, cfg.eps, bias=False, scaled=True)
    layers = []
    ignored = []
    for i, layer in enumerate(cfg.layers):
        p = f"l{i}."
        names = {"norm.weight": p + "norm1", "norm_after.weight": p + "norm1b", "norm_after.scale": p + "ls1"}
        mixer = _mixer(cfg, i, layer, names)
        feed_forward = None
        if layer.mlp is not None:
            e = layer.mlp
            feed_forward = RoutedExpertsSpec("routed_experts", cfg.width, e.experts, e.ff, e.top, activation=EXPERT_ACTIVATION,
                                             shared_hidden=e.shared_ff, gated=False, weigh_chosen=True)
            for j in range(e.experts):
                names.update({f"feed_forward.e{j}.{s}.weight": f"{p}mlp.e{j}.{s}" for s in ("up", "down")})
            names.update({"feed_forward.router.weight": p + "mlp.router", "feed_forward.router.bias": p + "mlp.router.b"})
            if e.shared_ff is not None:
                names.update({f"feed_forward.shared.{s}.weight": f"{p}mlp.shared.{s}" for s in ("up", "down", "sg")})
            names.update({"norm2.weight": p + "norm2", "norm2_after.weight": p + "norm2b", "norm2_after.scale": p + "ls2"})
        else:
            ignored += [p + "norm2", p + "ls2"]        # (a layer without a feed-forward has no use for its norms and scale)
        has_ff = feed_forward is not None
        layers.append(LayerSpec(arrangement="norms_around", norm=before, mixer=mixer, feed_forward=feed_forward,
                                norm2=before if has_ff else None, names=names, norm_after=behind, norm2_after=behind if has_ff else None))
    names = {"embedding": "embed", "embedding_norm.weight": "embed.norm", "final_norm.weight": "final.norm"}
    junctions = {}
    if cfg.loop_times is None:
        schedule = [ScheduleEntry(i) for i in range(len(cfg.layers))]
        ignored.append("loop.step")
    else:
        schedule = [ScheduleEntry(i) for i in range(cfg.loop_start)]
        for t in range(cfg.loop_times):
            # every pass keeps a cache or a state of its own and begins at the junction
            schedule += [ScheduleEntry(i, before="loop_step" if i == cfg.loop_start else None, passage=t)
                         for i in range(cfg.loop_start, cfg.loop_stop)]
        schedule += [ScheduleEntry(i) for i in range(cfg.loop_stop, len(cfg.layers))]
        if cfg.loop_times > 0 and cfg.loop_stop > cfg.loop_start:
            junctions["loop_step"] = PassVectorSpec("pass_vector", cfg.width, cfg.loop_times, embedding_from=EMBEDDING_FROM_PASS)
            names["junction.loop_step.steps"] = "loop.step"
        else:
            ignored.append("loop.step")
    return ModelPlan(
        architecture=NAME, vocab_size=cfg.vocab, dim=cfg.width, max_positions=cfg.max_positions, layers=tuple(layers),
        schedule=tuple(schedule), final_norm=before, head_bias=False, tied_head=True, names=names, embedding_norm=before,
        junctions=junctions, ignored_prefixes=tuple(ignored),
    )


def _claims(config: Dict[str, Any]) -> bool:
    layers = config.get("layers")
    return isinstance(layers, list) and bool(layers) and "width" in config and "embedding" not in config and "residual_mult" not in config and \
        all(isinstance(e, dict) and e.get("type") in KINDS and isinstance(e.get("mixer"), dict) for e in layers)


register(ModelSpec(
    name=NAME,
    read_config=VufolornConfig.from_dict,
    build_plan=build_plan,
    aliases=("Vufolorn",),
    claims=_claims,
    filename="model.safetensors",
))
