"""Small Vufolorn configurations for the tests, their model folders and crafted variants."""

from __future__ import annotations

import functools
import tempfile
from typing import Dict, Optional

import torch

from kestrel_amd.weights import InitRecipe, write_random_model
from tests.bogivik_cases import config_of, rewrite, stored_weights  # noqa: F401  (folders are read and edited the same way)


def experts(n, ff, top, shared=None):
    out = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": n, "top": top}}
    if shared is not None:
        out["shared"] = {"ff": shared}
    return out


def lightning(dim, vdim, decay, mlp=None):
    return {"type": "lightning", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": list(decay)}, "mlp": mlp}


def latent(heads, dim, vdim, kv_rank, scale, window: Optional[int], mlp=None):
    mixer = {"heads": heads, "dim": dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}
    if window is not None:
        mixer["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": mixer, "mlp": mlp}


def _config(vocab, width, eps, layers, loop=None):
    out = {"architecture": "Vufolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop is not None:
        out["loop"] = dict(zip(("start", "stop", "times"), loop))
    return out


CONFIGS: Dict[str, dict] = {
    # sizes the matrix-core kernels take; a loop over both kinds, run twice; two windows, of two and a half pages and of
    # one and a half, so two cache groups
    "P": _config(300, 128, 1e-5, [
        latent(4, 16, 24, 64, 0.3, 40, experts(6, 48, 2, 32)),
        lightning(32, 40, (0.3, 0.9, 0.99, 0.9995), experts(6, 48, 2, 32)),
        latent(2, 32, 64, 48, 0.25, 24, experts(5, 64, 3, 80)),
        lightning(48, 64, (1.0, 0.7), None),
    ], (1, 3, 2)),
    # sizes that fit none of the fast kernels' alignments: a window shorter than a page, a layer that sees every key, layers
    # without a feed-forward, no shared expert, one choice, a loop of one layer run three times, heads of one channel
    "Q": _config(211, 100, 1e-6, [
        lightning(10, 7, (0.95, 0.2, 0.999, 0.5, 0.98), experts(5, 20, 1)),
        latent(3, 12, 10, 36, 0.35, 7, experts(3, 24, 2, 20)),
        latent(5, 20, 6, 20, 0.25, None, None),
        lightning(1, 33, (0.9, 0.99, 0.8), experts(4, 24, 4, 36)),
    ], (1, 2, 3)),
    # the largest heads; latents wider than the attention kernel keeps in registers; windows of whole pages; more than 64
    # choices' worth of experts; no loop
    "R": _config(190, 256, 1e-3, [
        latent(2, 128, 128, 192, 0.09, 64, experts(16, 144, 4, 80)),
        lightning(128, 96, (0.97, 0.9999), experts(16, 144, 4, 80)),
        lightning(256, 8, (0.9,), None),
        latent(8, 64, 16, 128, 0.125, 32, experts(8, 80, 2, 144)),
    ]),
    # one head and one expert everywhere, a window of one key, nothing forgotten, a loop over every layer, run once
    "S": _config(77, 48, 1e-5, [
        latent(1, 16, 16, 32, 0.5, 1, experts(1, 40, 1, 8)),
        lightning(16, 8, (1.0,), experts(2, 16, 1)),
    ], (0, 2, 1)),
}
RECIPE = InitRecipe(std=0.08, bias_std=0.5, gain_std=0.2)
SEEDS = {"P": 41, "Q": 42, "R": 43, "S": 44}


@functools.lru_cache(maxsize=None)
def model_dir(name: str) -> str:
    folder = tempfile.mkdtemp(prefix=f"kestrel_amd_vufolorn{name}_")
    write_random_model(folder, CONFIGS[name], SEEDS[name], RECIPE, store_dtype="bfloat16")
    return folder


@functools.lru_cache(maxsize=None)
def steady(base: str) -> str:
    """A variant of a folder whose routers always choose the same experts: the logits' biases lift ``top`` of them by 30,
    which no logit can bridge; the weights of the chosen still follow their own logits. For runs in bfloat16: a router's
    choice is a step function of its logits, and where two of them lie closer than rounding moves them the step falls
    either way; the row then differs from the plain implementation by an expert, not by rounding."""
    config = config_of(base)

    def edit(weights):
        for i, layer in enumerate(config["layers"]):
            if layer["mlp"] is None:
                continue
            name = f"l{i}.mlp.router.b"
            count = weights[name].numel()
            order = torch.randperm(count, generator=torch.Generator().manual_seed(count + i))
            lifted = weights[name].float()
            lifted[order[:layer["mlp"]["router"]["top"]]] += 30.0
            weights[name] = lifted.to(weights[name].dtype)

    return rewrite(base, edit)


def folder_for(name: str, dtype) -> str:
    """The model folder a run in ``dtype`` is tested on: as written for float32, with steady routers for bfloat16."""
    folder = model_dir(name)
    return steady(folder) if dtype in (torch.bfloat16, "bfloat16") else folder


CALL, ECHO = 5, 6


@functools.lru_cache(maxsize=None)
def crafted(base: str) -> str:
    """A variant of a folder in which one key stands out: in every latent layer the query of the token ``CALL`` is the key of the
    token ``ECHO`` many times over, and every other token's query is next to nothing. The embedded tokens are large
    enough beside what a sublayer adds for a token to be recognised as itself in the later layers too, and these layers
    speak loudly enough to be heard."""
    config = config_of(base)

    def edit(weights):
        weights["embed.norm"] = torch.full_like(weights["embed.norm"], 5.0)
        rows = weights["embed"].float()
        unit = rows / rows.pow(2).mean(dim=1, keepdim=True).sqrt()
        call, echo = unit[CALL], unit[ECHO]
        for i, layer in enumerate(config["layers"]):
            if layer["type"] != "latent_attention":
                continue
            p = f"l{i}."
            m = layer["mixer"]
            for name in ("norm1", "norm1b", "ls1", "mix.dkv.norm"):
                weights[p + name] = torch.full_like(weights[p + name], 3.0 if name == "ls1" else 1.0)
            c = weights[p + "mix.dkv"].float() @ echo
            c = c / c.pow(2).mean().sqrt()
            key = (weights[p + "mix.uk"].float() @ c).reshape(m["heads"], m["dim"])
            # (a score of about 14 against the echo, whatever the head's size and the design's scale)
            query = key * (14.0 / (m["scale"] * key.pow(2).sum(dim=1, keepdim=True)))
            weights[p + "mix.q"] = (query.reshape(-1, 1) * (call / call.pow(2).sum())[None, :]).to(torch.bfloat16)
            # (every head speaks: its gate is open)
            weights[p + "mix.g"] = (3.0 * call / call.pow(2).sum())[None, :].repeat(m["heads"], 1).to(torch.bfloat16)

    return rewrite(base, edit)
