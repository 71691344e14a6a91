"""Small Vovalix configurations for the tests, with random weights, and helpers around them.

The configurations differ from each other in every size and in the number, order and kinds of their layers; between them they
cover query heads sharing a key/value head by two, three, six and eight and not at all, head counts that are no power of two,
key and value sizes on both sides of a wave, no power of two, odd, and equal, chunks below, at and above a page and none at all,
delta layers with one q/k head for several value heads and with one each, convolutions of one to five taps, decays' low-rank
maps of several ranks, tau of one and more, routed experts in groups and without, with and without a shared expert, one choice
a token and all of them, layers without a feed-forward, layers that use an earlier or a later layer's weights, widths that the
matrix cores' kernels take and one that they do not.
"""
from __future__ import annotations

import json
from pathlib import Path

import torch

from palm_infra_amd.config import config_from_dict
from palm_infra_amd.weights import random_tensors, write_safetensors


def gla(heads, dim, vdim, tau, rank):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau, "decay_rank": rank}}


def attention(heads, kv, dim, vdim, scale, chunk=None):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        m["mask"] = {"size": chunk}
    return {"type": "attention", "mixer": m}


def delta(heads, kv, dim, vdim, conv):
    return {"type": "delta", "mixer": {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "conv": conv}}


def moe(experts, top, ff, limit, groups=None, shared=None):
    f = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if groups:
        f["router"]["groups"] = {"count": groups[0], "keep": groups[1]}
    if shared:
        f["shared"] = {"ff": shared[0], "limit": shared[1]}
    return f


def layer(mixer, mlp=None, weights_of=None):
    out = dict(mixer, mlp=mlp)
    if weights_of is not None:
        out["weights_of"] = weights_of
    return out


def model(vocab, width, eps, scale, layers):
    return {"architecture": "Vovalix", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": scale, "layers": layers}


_A_ATT = (attention(6, 2, 24, 40, 0.2, chunk=37), moe(12, 3, 24, 1.2, groups=(3, 2), shared=(40, 0.9)))
_A_GLA = (gla(3, 16, 24, 8.0, 5), None)
_D_ATT = (attention(6, 1, 8, 12, 0.5, chunk=5), moe(16, 4, 8, 2.5, groups=(4, 2), shared=(24, 1.0)))
CONFIGS = {
    "A": model(211, 64, 1e-5, 0.7, [
        layer(delta(6, 2, 24, 40, 3), moe(8, 1, 32, 1.0, groups=(4, 1), shared=(16, 2.0))),
        layer(*_A_ATT), layer(*_A_GLA), layer(*_A_ATT, weights_of=1), layer(*_A_GLA, weights_of=2)]),
    "B": model(130, 48, 2e-6, 1.0, [
        layer(attention(3, 3, 40, 72, 0.15, chunk=70), moe(4, 2, 16, 1.5)),
        layer(delta(1, 1, 40, 130, 2)),
        layer(gla(1, 40, 130, 1.0, 16), moe(6, 3, 24, 0.8, groups=(2, 1), shared=(8, 0.5))),
        layer(delta(2, 2, 16, 16, 1), moe(4, 4, 16, 2.0))]),
    # larger sizes: eight query heads for each key/value head, key sizes of two waves, chunks of several pages and none
    "C": model(150, 96, 1e-5, 3.0, [
        layer(attention(16, 2, 64, 32, 0.125, chunk=130), moe(6, 2, 24, 1.0, shared=(48, 1.5))),
        layer(gla(2, 128, 64, 16.0, 24)),
        layer(delta(4, 2, 128, 16, 4), moe(9, 2, 40, 1.3, groups=(3, 2))),
        layer(attention(4, 4, 32, 96, 0.2), moe(5, 5, 16, 3.0)),
        layer(gla(4, 32, 16, 4.0, 3))]),
    # the first layer uses the third one's weights
    "D": model(97, 40, 1e-6, 1.5, [
        layer(*_D_ATT, weights_of=2),
        layer(delta(2, 1, 8, 12, 5), moe(5, 5, 16, 0.5)),
        layer(*_D_ATT),
        layer(gla(2, 8, 64, 2.0, 1), moe(3, 1, 8, 1.0, shared=(8, 1.0)))]),
    # a width, key sizes and value sizes that no kernel's vectors divide
    "E": model(61, 50, 1e-5, 0.9, [
        layer(gla(3, 9, 7, 3.0, 2), moe(6, 2, 5, 1.1, groups=(3, 1), shared=(11, 0.7))),
        layer(attention(5, 5, 9, 15, 0.3, chunk=64), moe(3, 2, 9, 1.4)),
        layer(delta(3, 1, 33, 5, 4), moe(2, 1, 7, 2.0, shared=(3, 1.0)))]),
}
SEEDS = {"A": 91, "B": 92, "C": 93, "D": 94, "E": 95}
# one layer, for the tests of a mechanism alone
SINGLE = {
    "attention": model(90, 32, 1e-6, 1.0, [layer(attention(4, 2, 12, 20, 0.3, chunk=50))]),
    "gla": model(90, 32, 1e-6, 1.0, [layer(gla(3, 12, 20, 6.0, 4))]),
    "delta": model(90, 32, 1e-6, 1.0, [layer(delta(4, 2, 12, 20, 4))]),
    "experts": model(90, 32, 1e-6, 1.0, [layer(gla(1, 8, 8, 2.0, 2), moe(9, 2, 16, 0.9, groups=(3, 2), shared=(12, 0.6)))]),
}


def tensors_of(raw: dict, seed: int, store: str) -> dict:
    """The random-weights mode's numbers (the description makes projections of a scale at which scores spread, gates open and
    close and caps bite)."""
    tensors = random_tensors(config_from_dict(raw).spec(), seed, "float32")
    return {k: t.to({"bfloat16": torch.bfloat16, "float32": torch.float32}[store]) for k, t in tensors.items()}


def write_model(raw: dict, seed: int, path, store: str, keep_ranks: bool = False) -> Path:
    """``keep_ranks`` false: config.json does not say the ranks that the tensors' shapes give."""
    path = Path(path)
    path.mkdir(parents=True, exist_ok=True)
    written = json.loads(json.dumps(raw))
    if not keep_ranks:
        for entry in written["layers"]:
            entry["mixer"].pop("decay_rank", None)
    (path / "config.json").write_text(json.dumps(written))
    write_safetensors(path / "model.safetensors", tensors_of(raw, seed, store))
    return path


def prompts(raw: dict, lengths, seed: int = 0) -> list:
    g = torch.Generator().manual_seed(7000 + seed)
    return [torch.randint(0, raw["vocab"], (n,), generator=g).tolist() for n in lengths]
