"""A plain, slow Nirotar in float64 on the CPU, written from the design's equations: one function per mechanism, whole
sequences only, no cache, no batching.  It shares no code with the library; the tests compare the library with it.

In this file's notation (i, j: positions from 0; N: a layer's RMS norm):

  layer       x' = x + mixer(N1(x));  x'' = x' + ff(N2(x')): a layer may have no feed-forward
  attention   grouped heads, the first dimensions of q and k rotated in neighbouring pairs with stretched slow frequencies, a
              sliding window, one more term exp(sink_h) in the softmax's denominator
  latent      all heads' keys and values made from one normed latent and one rotated key part per position; the same sinks, no
              window; a layer may read an earlier layer's latents and rotated parts with matrices of its own
  experts     a table by token id instead of a router, equal weights, relu(z)^2 inside; one shared expert for every token

A model is a raw config.json dict and a dict of tensors by checkpoint name.  Every function takes and returns float64.
"""
from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F64 = torch.float64


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps) * w


# ---- rotation ------------------------------------------------------------------------------------------------------

def frequencies(rot):
    """The angle per position of every pair [dims / 2]."""
    dims, base = int(rot["dims"]), float(rot["base"])
    out = []
    for i in range(dims // 2):
        f = base ** (-2.0 * i / dims)
        sc = rot.get("scaling")
        if sc:
            wavelength = 2.0 * math.pi / f
            factor, low, high, original = (float(sc[k]) for k in ("factor", "low", "high", "original"))
            if wavelength > original / low:
                f = f / factor
            elif wavelength >= original / high:
                s = (original / wavelength - low) / (high - low)
                f = (1.0 - s) * f / factor + s * f
        out.append(f)
    return torch.tensor(out, dtype=F64)


def rotate_pairs(x, rot):
    """x [T, heads, n]: dimensions 2i and 2i + 1 of the first ``dims`` turn by position times frequency i."""
    f = frequencies(rot)
    dims = int(rot["dims"])
    a = torch.arange(x.shape[0], dtype=F64)[:, None] * f[None, :]
    c, s = torch.cos(a)[:, None, :], torch.sin(a)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


# ---- attention -----------------------------------------------------------------------------------------------------

def sink_softmax_heads(scores, sink, window):
    """scores [H, T, T] (query, key) -> weights of the same shape: query i sees the keys j <= i, of them the last ``window``
    (None: all); head h's denominator has one more term exp(sink[h])."""
    T = scores.shape[1]
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    seen = j <= i
    if window is not None:
        seen = seen & (i - j < window)
    s = scores.masked_fill(~seen, -math.inf)
    top = torch.maximum(s.max(dim=2, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - top)
    return e / (e.sum(dim=2, keepdim=True) + torch.exp(sink[:, None, None] - top))


def attention_mixer(h, w, p, m, eps, shelf):
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ w[p + "q"].T).reshape(T, H, d)
    k = (h @ w[p + "k"].T).reshape(T, G, d)
    v = (h @ w[p + "v"].T).reshape(T, G, dv)
    if m.get("rot"):
        q, k = rotate_pairs(q, m["rot"]), rotate_pairs(k, m["rot"])
    of_head = torch.tensor([a // (H // G) for a in range(H)])
    kh, vh = k[:, of_head], v[:, of_head]
    scores = torch.stack([(q[:, a] @ kh[:, a].T) * float(m["scale"]) for a in range(H)])
    pr = sink_softmax_heads(scores, w[p + "sink"], int(m["mask"]["size"]) if m.get("mask") else None)
    o = torch.stack([pr[a] @ vh[:, a] for a in range(H)], dim=1)
    return o.reshape(T, H * dv) @ w[p + "o"].T


def latent_rows(h, w, p, m, eps):
    """What a position keeps: the normed latent [T, kv_rank] and the rotated key part [T, rot_dim]."""
    R = int(m["kv_rank"])
    down = h @ w[p + "dkv"].T
    return rms_norm(down[:, :R], w[p + "dkv.norm"], eps), rotate_pairs(down[:, None, R:], m["rot"])[:, 0]


def latent_mixer(h, w, p, m, eps, shelf):
    """``shelf``: layer prefix -> the rows it made; a layer that borrows takes another's."""
    H, d, dr, dv = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"])
    T = h.shape[0]
    if m.get("kv_from") is None:
        shelf[p] = latent_rows(h, w, p, m, eps)
        c, r = shelf[p]
    else:
        c, r = shelf[f"l{int(m['kv_from'])}.mix."]
    q = (h @ w[p + "q"].T).reshape(T, H, d + dr)
    q_plain, q_rot = q[..., :d], rotate_pairs(q[..., d:], m["rot"])
    k_plain = (c @ w[p + "uk"].T).reshape(T, H, d)
    v = (c @ w[p + "uv"].T).reshape(T, H, dv)
    scores = torch.stack([(q_plain[:, a] @ k_plain[:, a].T + q_rot[:, a] @ r.T) * float(m["scale"]) for a in range(H)])
    pr = sink_softmax_heads(scores, w[p + "sink"], int(m["mask"]["size"]) if m.get("mask") else None)
    o = torch.stack([pr[a] @ v[:, a] for a in range(H)], dim=1)
    return o.reshape(T, H * dv) @ w[p + "o"].T


# ---- experts -------------------------------------------------------------------------------------------------------

def squared_relu_expert(h, w, p):
    z = torch.clamp(h @ w[p + "up"].T, min=0.0)
    return (z * z) @ w[p + "down"].T


def table_experts(h, ids, w, p, f):
    table = w[p + "table"].long()
    top = int(f["router"]["top"])
    out = torch.zeros_like(h)
    for t, token in enumerate(ids):
        for c in range(top):
            out[t] += squared_relu_expert(h[t], w, f"{p}e{int(table[token, c])}.") / top
    if f.get("shared"):
        out = out + squared_relu_expert(h, w, p + "shared.")
    return out


# ---- the model -----------------------------------------------------------------------------------------------------

MIXERS = {"attention": attention_mixer, "latent_attention": latent_mixer}


def forward(raw, tensors, ids, layer_results=None):
    """Logits [T, vocab] of one sequence from its first token.  ``layer_results``: a list that gets the residual stream
    after every layer."""
    w = {k: t.to(F64) for k, t in tensors.items()}
    eps = float(raw["norm"]["eps"])
    x = w["embed"][torch.tensor(ids, dtype=torch.long)]
    shelf = {}
    for i, layer in enumerate(raw["layers"]):
        p = f"l{i}."
        x = x + MIXERS[layer["type"]](rms_norm(x, w[p + "norm1"], eps), w, p + "mix.", layer["mixer"], eps, shelf)
        if layer.get("mlp") is not None:
            x = x + table_experts(rms_norm(x, w[p + "norm2"], eps), ids, w, p + "mlp.", layer["mlp"])
        if layer_results is not None:
            layer_results.append(x)
    return rms_norm(x, w["final.norm"], eps) @ w["head"].T


def read_model(path):
    """(raw config, tensors by name) of a model folder."""
    from safetensors.torch import load_file
    path = Path(path)
    return json.loads((path / "config.json").read_text()), load_file(str(path / "model.safetensors"))


def greedy(cfg, tensors, prompt, n_new):
    ids = list(prompt)
    for _ in range(n_new):
        ids.append(int(forward(cfg, tensors, ids)[-1].argmax()))
    return ids[len(prompt):]
