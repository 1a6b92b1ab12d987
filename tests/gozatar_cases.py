"""Small Gozatar configurations for the tests, their model folders and crafted variants."""

from __future__ import annotations

import functools
import tempfile
from typing import Dict, Optional

import torch

from kestrel_amd.weights import InitRecipe, write_random_model
from tests.bogivik_cases import config_of, rewrite, stored_weights  # noqa: F401  (folders are read and edited the same way)


def moe(n, ff, limit, top, groups=None, shared=None):
    router = {"experts": n, "top": top}
    if groups is not None:
        router["groups"] = {"count": groups[0], "keep": groups[1]}
    out = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared is not None:
        out["shared"] = {"ff": shared[0], "limit": shared[1]}
    return out


def dense(ff):
    return {"kind": "dense", "ff": ff}


def parallel(left, right, scales, mlp=None):
    """``left``: heads, kv heads, dim, vdim, scale, taps, window, rotated channels, base; ``right``: heads, dim, vdim, tau, rank of the decay."""
    heads, kv_heads, dim, vdim, scale, taps, window, dims, base = left
    mixer = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": {"base": base, "dims": dims}}
    if taps is not None:
        mixer["conv"] = taps
    if window is not None:
        mixer["mask"] = {"size": window}
    r_heads, r_dim, r_vdim, tau, rank = right
    return {"type": "parallel", "mixer": {"left": mixer, "right": {"heads": r_heads, "dim": r_dim, "vdim": r_vdim, "tau": tau, "decay_rank": rank},
                                          "left_scale": scales[0], "right_scale": scales[1]}, "mlp": mlp}


def _config(vocab, width, streams, eps, layers):
    return {"architecture": "Gozatar", "vocab": vocab, "width": width, "streams": streams, "norm": {"eps": eps}, "layers": layers}


CONFIGS: Dict[str, dict] = {
    # sizes the matrix-core kernels take; three streams; two windows, of two and a half pages and of one and a half; a shared expert like the others and one with a size and a limit of its own
    "P": _config(300, 128, 3, 1e-5, [
        parallel((4, 2, 32, 64, 0.3, 4, 40, 16, 10000.0), (3, 32, 40, 8.0, 16), (0.8, 1.3), moe(8, 48, 1.2, 3, (4, 2), (48, 1.2))),
        parallel((2, 2, 64, 32, 0.2, 3, 24, 64, 500.0), (2, 48, 64, 4.0, 24), (1.4, -0.7), dense(176)),
        parallel((4, 1, 32, 64, 0.4, 2, 40, 32, 3000.0), (4, 16, 128, 30.0, 8), (1.0, 1.0), moe(6, 64, 0.8, 2, None, (80, 2.5))),
        parallel((2, 1, 64, 64, 0.25, 4, 24, 32, 10000.0), (1, 64, 8, 2.0, 40), (0.5, 2.0), None),
    ]),
    # sizes that fit none of the fast kernels' alignments: five streams, a window shorter than a page, a layer that sees every key,
    # one without convolutions and one with a single tap, more taps than the fast kernel keeps, no shared expert, groups of
    # three, one choice, decays that forget at once (tau below 1), a layer without a feed-forward
    "Q": _config(211, 100, 5, 1e-6, [
        parallel((3, 1, 12, 10, 0.35, 6, 7, 6, 100.0), (5, 10, 7, 0.3, 5), (1.2, 0.6), moe(6, 20, 0.7, 2, (2, 1))),
        parallel((5, 5, 20, 6, 0.25, None, None, 20, 2000.0), (2, 6, 33, 16.0, 3), (0.9, -0.8), None),
        parallel((4, 2, 18, 36, 0.3, 1, 11, 2, 7.0), (3, 22, 12, 1.0, 7), (-0.5, 1.1), moe(3, 24, 3.0, 1, None, (36, 0.5))),
        parallel((2, 1, 40, 18, 0.2, 5, 19, 12, 50.0), (1, 36, 20, 5.0, 9), (1.0, 0.9), dense(70)),
    ]),
    # the largest heads; two streams; windows of whole pages; key heads of the recurrence that the chunked kernels take and that
    # they do not; many experts, groups that are all kept; values wider than keys
    "R": _config(190, 256, 2, 1e-3, [
        parallel((2, 1, 128, 128, 0.09, 2, 64, 128, 1e6), (2, 128, 96, 16.0, 32), (1.0, 0.4), moe(16, 144, 1.0, 4, (4, 4), (144, 1.0))),
        parallel((4, 4, 64, 96, 0.125, 4, 32, 16, 1e4), (2, 224, 72, 64.0, 16), (0.7, 0.7), moe(24, 80, 1.6, 5, (8, 3), (144, 1.6))),
        parallel((8, 2, 16, 32, 0.3, 3, 32, 8, 300.0), (1, 256, 24, 10.0, 16), (1.1, 0.8), dense(264)),
    ]),
    # one stream, one head and one expert everywhere, a window of one key, groups of one expert, scales of 1
    "S": _config(77, 48, 1, 1e-5, [
        parallel((1, 1, 16, 16, 0.5, 2, 1, 2, 3.0), (1, 16, 8, 1.0, 1), (1.0, 1.0), moe(1, 40, 0.6, 1, (1, 1), (8, 1.0))),
        parallel((1, 1, 8, 24, 1.0, 4, 3, 8, 20.0), (1, 8, 16, 3.0, 4), (1.0, 0.5), moe(4, 16, 1.0, 2, (4, 2))),
    ]),
}
RECIPE = InitRecipe(std=0.08, bias_std=0.5, gain_std=0.2)
SEEDS = {"P": 51, "Q": 52, "R": 53, "S": 54}


@functools.lru_cache(maxsize=None)
def model_dir(name: str) -> str:
    folder = tempfile.mkdtemp(prefix=f"kestrel_amd_gozatar{name}_")
    write_random_model(folder, CONFIGS[name], SEEDS[name], RECIPE, store_dtype="bfloat16")
    return folder


@functools.lru_cache(maxsize=None)
def steady(base: str) -> str:
    """A variant of a folder whose routers always choose the same experts: the corrections of ``top`` of them, in as few groups as
    can be, are 4, which no score between 0 and 1 can bridge (the weights leave the corrections out). For runs in
    bfloat16: a choice is a step function of the scores, and where two of them lie closer than rounding moves them the step
    falls either way; the row then differs from the plain implementation by an expert, not by rounding."""
    config = config_of(base)

    def edit(weights):
        for i, layer in enumerate(config["layers"]):
            if not layer["mlp"] or layer["mlp"]["kind"] != "moe":
                continue
            router = layer["mlp"]["router"]
            name = f"l{i}.mlp.correction"
            count = router["experts"]
            gen = torch.Generator().manual_seed(count + i)
            groups = (router.get("groups") or {"count": 1})["count"]
            order = [g * (count // groups) + e for g in torch.randperm(groups, generator=gen).tolist()
                     for e in torch.randperm(count // groups, generator=gen).tolist()]
            lifted = torch.zeros(count)
            lifted[order[:router["top"]]] = 4.0
            weights[name] = lifted.to(weights[name].dtype)

    return rewrite(base, edit)


def folder_for(name: str, dtype) -> str:
    """The model folder a run in ``dtype`` is tested on: as written for float32, with steady routers for bfloat16."""
    folder = model_dir(name)
    return steady(folder) if dtype in (torch.bfloat16, "bfloat16") else folder


CALL, ECHO = 5, 6


@functools.lru_cache(maxsize=None)
def crafted(base: str) -> str:
    """A variant of a folder in which one key stands out: in every layer the query of the token ``CALL`` and the key of the token
    ``ECHO`` point the same way, in channels that are not rotated or slowly; other keys point elsewhere. The convolutions
    let the current token through alone. The embedded tokens are large beside what a sublayer adds, so that a token is
    recognised as itself in the later layers too, and attention speaks loudly enough to be heard."""
    config = config_of(base)

    def edit(weights):
        weights["embed"] = (weights["embed"].float() * 60.0).to(weights["embed"].dtype)
        rows = weights["embed"].float()
        unit = rows - rows.mean(dim=1, keepdim=True)
        unit = unit / unit.pow(2).mean(dim=1, keepdim=True).sqrt()
        call, echo = (unit[t] / unit[t].pow(2).sum() for t in (CALL, ECHO))
        for i, layer in enumerate(config["layers"]):
            m, p = layer["mixer"]["left"], f"l{i}.mix.left."
            gen = torch.Generator().manual_seed(70 + i)
            width, d, heads, kv_heads = config["width"], m["dim"], m["heads"], m["kv_heads"]
            weights[f"l{i}.norm1"] = torch.ones_like(weights[f"l{i}.norm1"])
            for name in ("q", "k", "v"):
                if m.get("conv"):
                    taps = torch.zeros_like(weights[p + name + ".conv"])
                    taps[:, -1] = 1.0
                    weights[p + name + ".conv"] = taps
            way = torch.zeros(kv_heads, d)
            way[:, -(d // 4):] = torch.randn(kv_heads, d // 4, generator=gen)
            way = way / way.pow(2).mean(dim=1, keepdim=True).sqrt()
            for name, count, token in (("q", heads, call), ("k", kv_heads, echo)):
                own = way.repeat_interleave(count // kv_heads, dim=0).reshape(-1, 1) * token[None, :]
                noise = torch.randn(count * d, width, generator=gen) * (0.3 / width ** 0.5)
                weights[p + name] = (own + noise).to(torch.bfloat16)
            weights[p + "o"] = (weights[p + "o"].float() * 2.0).to(torch.bfloat16)

    def edit_config(config):
        for layer in config["layers"]:
            layer["mixer"]["left"]["scale"] = 30.0 / layer["mixer"]["left"]["dim"]

    return rewrite(base, edit, edit_config)
