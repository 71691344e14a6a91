"""Small Nirotar configurations for the tests, with random weights, and helpers around them.

The configurations differ from each other in every size and in the number, order and kinds of their layers; between them they
cover query heads sharing a key/value head by two, three, six and eight and not at all, head counts that are no power of two and
one beyond a tile of sixteen, key and value sizes on both sides of a wave, no power of two, odd, and equal, rotations of a part
of a head and of all of it, with frequencies in every band of the scaling and without scaling, windows below, at and above a page
and none, latents of several sizes (some that the matrix cores' kernels do not take), layers that read the latents of the layer
right before them, of one further back, and two that read the same ones, with head counts and value sizes of their own, tables
of one choice and of all experts, with and without a shared expert of the experts' size or another, layers without a
feed-forward, and a width that no vector divides.
"""
from __future__ import annotations

import json
from pathlib import Path

import torch

from palm_infra_amd.config import config_from_dict
from palm_infra_amd.weights import random_tensors, write_safetensors


def rotation(dims, base, scaling=None):
    r = {"dims": dims, "base": base}
    if scaling:
        r["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return r


def attention(heads, kv, dim, vdim, scale, window=None, rot=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if window:
        m["mask"] = {"size": window}
    if rot:
        m["rot"] = rotation(*rot)
    return {"type": "attention", "mixer": m}


def latent(heads, dim, rot_dim, vdim, rank, scale, base, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": rank, "scale": scale, "rot": rotation(rot_dim, base)}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m}


def moe(experts, top, ff, shared=None):
    f = {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}
    if shared:
        f["shared"] = {"ff": shared}
    return f


def layer(mixer, mlp=None):
    return dict(mixer, mlp=mlp)


def model(vocab, width, eps, layers):
    return {"architecture": "Nirotar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


CONFIGS = {
    "A": model(211, 64, 1e-5, [
        layer(attention(6, 2, 24, 40, 0.2, window=37, rot=(16, 500.0, (4.0, 1.0, 4.0, 256))), moe(8, 3, 24, shared=40)),
        layer(latent(5, 16, 8, 24, 40, 0.22, 3000.0), moe(5, 1, 32, shared=32)),
        layer(attention(3, 3, 40, 24, 0.16, window=70, rot=(40, 10000.0)), None),
        layer(latent(3, 24, 8, 40, 40, 0.18, 3000.0, kv_from=1), moe(4, 4, 16))]),
    # rows for the exact kernels only (sizes in no steps of eight), an unrotated attention without a window
    "B": model(130, 48, 2e-6, [
        layer(latent(4, 12, 6, 20, 37, 0.25, 40.0), None),
        layer(latent(2, 20, 6, 9, 37, 0.2, 40.0, kv_from=0), moe(6, 2, 40)),
        layer(attention(3, 1, 40, 72, 0.15), moe(3, 2, 16, shared=8)),
        layer(latent(7, 9, 6, 12, 37, 0.3, 40.0, kv_from=0), moe(9, 5, 8, shared=24))]),
    # larger sizes: more heads than a tile of sixteen, eight query heads for each key/value head, windows over several pages
    "C": model(150, 96, 1e-5, [
        layer(attention(16, 2, 64, 32, 0.125, window=130, rot=(32, 20.0, (8.0, 1.0, 2.0, 64))), moe(12, 2, 24, shared=56)),
        layer(latent(18, 32, 16, 36, 128, 0.15, 700.0), moe(6, 2, 24, shared=24)),
        layer(latent(4, 64, 16, 96, 128, 0.11, 700.0, kv_from=1), None),
        layer(latent(2, 40, 32, 16, 200, 0.12, 90.0), moe(4, 1, 64, shared=16))]),
    # a window at a page's size, a single kind of layer at the end, no shared experts
    "D": model(97, 40, 1e-6, [
        layer(attention(4, 4, 8, 12, 0.5, window=64, rot=(4, 8.0, (2.0, 0.5, 2.0, 32))), moe(3, 1, 8)),
        layer(attention(6, 1, 16, 8, 0.3, window=5, rot=(16, 100.0, (16.0, 2.0, 8.0, 512))), None),
        layer(latent(1, 8, 16, 8, 24, 0.3, 25.0), moe(2, 2, 8))]),
    # a width, key sizes and value sizes that no kernel's vectors divide
    "E": model(61, 50, 1e-5, [
        layer(latent(3, 9, 2, 7, 33, 0.35, 9.0), moe(6, 2, 5, shared=11)),
        layer(attention(5, 5, 9, 15, 0.3, window=66, rot=(6, 30.0, (3.0, 1.0, 3.0, 100))), moe(3, 2, 9)),
        layer(latent(2, 15, 2, 33, 33, 0.25, 9.0, kv_from=0), moe(2, 1, 7, shared=7))]),
}
SEEDS = {"A": 111, "B": 112, "C": 113, "D": 114, "E": 115}
# one layer, for the tests of a mechanism alone
SINGLE = {
    "attention": model(90, 32, 1e-6, [layer(attention(4, 2, 12, 20, 0.3, window=50, rot=(8, 60.0, (4.0, 1.0, 4.0, 128))))]),
    "latent": model(90, 32, 1e-6, [layer(latent(3, 12, 8, 20, 24, 0.25, 80.0))]),
    "borrowed": model(90, 32, 1e-6, [layer(latent(2, 12, 8, 16, 24, 0.25, 80.0)), layer(latent(5, 8, 8, 12, 24, 0.3, 80.0, kv_from=0))]),
    "experts": model(90, 32, 1e-6, [layer(latent(1, 8, 4, 8, 16, 0.3, 50.0), moe(9, 2, 16, shared=12))]),
}


def tensors_of(raw: dict, seed: int, store: str) -> dict:
    """The random-weights mode's numbers (the description makes projections of a scale at which scores spread)."""
    tensors = random_tensors(config_from_dict(raw).spec(), seed, "float32")
    dt = {"bfloat16": torch.bfloat16, "float32": torch.float32}[store]
    return {k: t if t.dtype == torch.int32 else t.to(dt) for k, t in tensors.items()}


def write_model(raw: dict, seed: int, path, store: str) -> Path:
    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    (path / "config.json").write_text(json.dumps(raw))
    write_safetensors(path / "model.safetensors", tensors_of(raw, seed, store))
    return path


def prompts(raw: dict, lengths, seed: int = 0) -> list:
    g = torch.Generator().manual_seed(8000 + seed)
    return [torch.randint(0, raw["vocab"], (n,), generator=g).tolist() for n in lengths]
