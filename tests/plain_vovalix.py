"""A plain, slow Vovalix in float64 on the CPU, written from the design's equations: one function per mechanism, whole
sequences only, no cache, no batching.  It shares no code with the library; the tests compare the library with it.

In this file's notation (t, i, j: positions from 0; N: the layer's norm with its weight kept around zero):

  layer       x' = x + mixer(N(x)) + ff(N(x)): one norm, both branches read its output; a layer may have no feed-forward,
              and may use another layer's weights
  gla         per head S [key, value]: S <- diag(a_t) S + k_t v_t^T, o_t = S^T q_t, a_t = sigmoid(low-rank map of h)^(1/tau)
  attention   grouped heads over unit-rms q and k, score minus a slope per head times the distance, only keys of the
              query's own chunk of positions
  delta       per head S <- g_t S; u = beta_t (v_t - S^T k_t); S <- S + k_t u^T; o_t = S^T q_t behind short convolutions
  experts     a softmax router over all experts; only experts of the best groups (by their largest score); capped gates; one
              shared expert for every token

A model is a raw config.json dict and a dict of tensors by checkpoint name.  Every function takes and returns float64.
"""
from __future__ import annotations

import json
import math
from pathlib import Path

import torch

F64 = torch.float64
GATE_SLOPE = 1.702


def unit_rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def norm_around_zero(x, w, eps):
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def log_sigmoid(z):
    return torch.where(z >= 0, -torch.log1p(torch.exp(-z.abs())), z - torch.log1p(torch.exp(-z.abs())))


def softplus(z):
    return torch.where(z > 0, z + torch.log1p(torch.exp(-z.abs())), torch.log1p(torch.exp(-z.abs())))


def gated_heads(o, w, p, h, eps):
    """o [T, heads, vdim]: each head's rms norm with one weight for all heads, times silu of the gate, then the output matrix."""
    T = o.shape[0]
    y = (unit_rms(o, eps) * w[p + "norm"]).reshape(T, -1) * silu(h @ w[p + "g"].T)
    return y @ w[p + "o"].T


# ---- gated linear attention ----------------------------------------------------------------------------------------

def channel_decays(h, w, p, tau):
    z = (h @ w[p + "a1"].T) @ w[p + "a2"].T + w[p + "a2.b"]
    return torch.exp(log_sigmoid(z) / tau)


def gla_recurrence(q, k, v, a):
    """q, k, a [T, heads, dim], v [T, heads, vdim] -> o [T, heads, vdim] and the state left behind [heads, dim, vdim]."""
    T, H, d = q.shape
    S = torch.zeros((H, d, v.shape[2]), dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = a[t][:, :, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = (S * q[t][:, :, None]).sum(1)
    return out, S


def gla_mixer(h, w, p, m, eps):
    H, d, dv = int(m["heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = (h @ w[p + "q"].T).reshape(T, H, d) * d ** -0.5
    k = (h @ w[p + "k"].T).reshape(T, H, d)
    v = (h @ w[p + "v"].T).reshape(T, H, dv)
    a = channel_decays(h, w, p, float(m["tau"])).reshape(T, H, d)
    return gated_heads(gla_recurrence(q, k, v, a)[0], w, p, h, eps)


# ---- attention -----------------------------------------------------------------------------------------------------

def head_slopes(heads):
    return [2.0 ** (-8.0 * (h + 1) / heads) for h in range(heads)]


def chunk_softmax_heads(q, k, v, scale, slopes, size):
    """q [T, H, d], k [T, G, d], v [T, G, dv] of one sequence -> [T, H, dv].  Query i sees the keys j <= i of its own chunk
    of ``size`` positions (None: every j <= i); head h's score loses slopes[h] * (i - j) (slopes None: nothing)."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    i = torch.arange(T)
    seen = i[:, None] >= i[None, :]
    if size is not None:
        seen = seen & (i[:, None] // size == i[None, :] // size)
    out = torch.zeros((T, H, v.shape[2]), dtype=F64)
    for h in range(H):
        s = (q[:, h] @ k[:, h // per].T) * scale
        if slopes is not None:
            s = s - slopes[h] * (i[:, None] - i[None, :]).to(F64)
        out[:, h] = torch.softmax(s.masked_fill(~seen, -math.inf), dim=1) @ v[:, h // per]
    return out


def attention_mixer(h, w, p, m, eps):
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q = unit_rms((h @ w[p + "q"].T).reshape(T, H, d), eps)
    k = unit_rms((h @ w[p + "k"].T).reshape(T, G, d), eps)
    v = (h @ w[p + "v"].T).reshape(T, G, dv)
    size = int(m["mask"]["size"]) if m.get("mask") else None
    o = chunk_softmax_heads(q, k, v, float(m["scale"]), head_slopes(H), size)
    return o.reshape(T, H * dv) @ w[p + "o"].T


# ---- the delta rule ------------------------------------------------------------------------------------------------

def short_convolution(u, taps_w):
    """u [T, C], taps_w [C, taps]: y_t = sum_j taps_w[:, j] u_(t - taps + 1 + j), zeros before the start."""
    T, C = u.shape
    taps = taps_w.shape[1]
    padded = torch.cat([torch.zeros((taps - 1, C), dtype=F64), u], dim=0)
    y = torch.zeros((T, C), dtype=F64)
    for j in range(taps):
        y = y + taps_w[:, j][None, :] * padded[j:j + T]
    return y


def unit_vectors(x):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + 1e-6)


def delta_recurrence(q, k, v, beta, g):
    """q, k [T, G, dim], v [T, H, vdim], beta, g [T, H] -> o [T, H, vdim]; head h reads q/k head h // (H / G)."""
    T, H, dv = v.shape
    rep = H // q.shape[1]
    qh, kh = q.repeat_interleave(rep, 1), k.repeat_interleave(rep, 1)
    S = torch.zeros((H, q.shape[2], dv), dtype=F64)
    out = torch.zeros_like(v)
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - (S * kh[t][:, :, None]).sum(1))
        S = S + kh[t][:, :, None] * u[:, None, :]
        out[t] = (S * qh[t][:, :, None]).sum(1)
    return out


def delta_mixer(h, w, p, m, eps):
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    T = h.shape[0]
    q, k, v = (silu(short_convolution(h @ w[p + n].T, w[p + n + ".conv"])) for n in "qkv")
    q = unit_vectors(q.reshape(T, G, d)) * d ** -0.5
    k = unit_vectors(k.reshape(T, G, d))
    beta = torch.sigmoid(h @ w[p + "b"].T)
    g = torch.exp(-torch.exp(w[p + "A_log"]) * softplus(h @ w[p + "a"].T + w[p + "dt_bias"]))
    return gated_heads(delta_recurrence(q, k, v.reshape(T, H, dv), beta, g), w, p, h, eps)


# ---- experts -------------------------------------------------------------------------------------------------------

def capped_expert(h, w, p, limit):
    g = torch.clamp(h @ w[p + "gate"].T, max=limit)
    u = torch.clamp(h @ w[p + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(GATE_SLOPE * g) * (u + 1.0)) @ w[p + "down"].T


def route(z, r):
    """Router logits z [T, experts] -> chosen [T, top] (expert indices) and weights [T, top]."""
    E, top = int(r["experts"]), int(r["top"])
    s = torch.softmax(z, dim=-1)
    T = z.shape[0]
    choice = s
    if r.get("groups"):
        count, keep = int(r["groups"]["count"]), int(r["groups"]["keep"])
        by_group = s.reshape(T, count, E // count)
        best = by_group.max(dim=2).values.topk(keep, dim=1).indices
        allowed = torch.zeros((T, count), dtype=torch.bool).scatter_(1, best, True)
        choice = by_group.masked_fill(~allowed[:, :, None], -math.inf).reshape(T, E)
    chosen = choice.topk(top, dim=1).indices
    picked = s.gather(1, chosen)
    return chosen, picked / (picked.sum(dim=1, keepdim=True) + 1e-20)


def route_margins(z, r):
    """How far each token's choice is from another one [T]: the smallest difference of router logits between an expert that is
    chosen and one that could be, and between the largest of a kept group and of one that is not."""
    E, top = int(r["experts"]), int(r["top"])
    count, keep = (int(r["groups"]["count"]), int(r["groups"]["keep"])) if r.get("groups") else (1, 1)
    by_group = z.reshape(z.shape[0], count, E // count)
    best = by_group.max(dim=2).values
    ranked = best.sort(dim=1, descending=True).values
    out = ranked[:, keep - 1] - ranked[:, keep] if keep < count else torch.full((z.shape[0],), math.inf, dtype=F64)
    inside = by_group.masked_fill((best < ranked[:, keep - 1:keep])[:, :, None], -math.inf).reshape(z.shape[0], E).sort(dim=1, descending=True).values
    return torch.minimum(out, inside[:, top - 1] - inside[:, top]) if top < E else out


def routed_feed_forward(h, w, p, f):
    chosen, weights = route(h @ w[p + "router"].T, f["router"])
    out = torch.zeros_like(h)
    for e in range(int(f["router"]["experts"])):
        for c in range(chosen.shape[1]):
            rows = (chosen[:, c] == e).nonzero().flatten()
            if rows.numel():
                out[rows] += weights[rows, c][:, None] * capped_expert(h[rows], w, f"{p}e{e}.", float(f["expert"]["limit"]))
    if f.get("shared"):
        out = out + capped_expert(h, w, p + "shared.", float(f["shared"]["limit"]))
    return out


# ---- the model -----------------------------------------------------------------------------------------------------

MIXERS = {"gla": gla_mixer, "attention": attention_mixer, "delta": delta_mixer}


def forward(raw, tensors, ids, layer_results=None, margins=None):
    """Logits [T, vocab] of one sequence from its first token.  ``layer_results``: a list that gets the residual stream
    after every layer; ``margins``: one that gets every router's ``route_margins``."""
    w = {k: t.to(F64) for k, t in tensors.items()}
    eps = float(raw["norm"]["eps"])
    x = w["embed"][torch.tensor(ids, dtype=torch.long)]
    for i, layer in enumerate(raw["layers"]):
        j = i
        while raw["layers"][j].get("weights_of") is not None:
            j = int(raw["layers"][j]["weights_of"])
        p = f"l{j}."
        h = norm_around_zero(x, w[p + "norm1"], eps)
        y = MIXERS[layer["type"]](h, w, p + "mix.", layer["mixer"], eps)
        if layer.get("mlp") is not None:
            y = y + routed_feed_forward(h, w, p + "mlp.", layer["mlp"])
            if margins is not None:
                margins.append(route_margins(h @ w[p + "mlp.router"].T, layer["mlp"]["router"]))
        x = x + y
        if layer_results is not None:
            layer_results.append(x)
    return norm_around_zero(x, w["final.norm"], eps) @ w["embed"].T * float(raw.get("logit_scale", 1.0))


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
