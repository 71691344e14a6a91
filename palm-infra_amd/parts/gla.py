"""Gated linear attention: linear attention whose state decays by a number for every key channel and token.

Per head, with q_t (times ``query_scale``), k_t of size ``key_dim`` and v_t of size ``value_dim``:

    a_t = sigmoid(W_2 (W_1 h_t) + b)^(1/tau);   S_t = diag(a_t) S_(t-1) + k_t v_t^T;   o_t = S_t^T q_t

each head's o_t is normed over value_dim (one weight vector for all heads) and multiplied by silu of a gate projection; the heads
are joined and projected back.  One joined product makes q | k | v | gate; W_1 h (``decay_rank`` values) comes from a product
with a 32-bit result, and the pass that prepares q and k makes the decays from it.  S is float32 and is kept per sequence
(``StateNeed``); decays and everything in the recurrence are 32-bit whatever the run's type.
"""
from __future__ import annotations

import torch

from ..cache import StateNeed
from ..kernels import ops
from .base import register_part
from .linear import Linear


@register_part("mixer", "gla")
class GatedLinearAttention:
    capturable = True

    def __init__(self, spec, builder):
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.nh, self.dk, self.dv, self.rank = (int(p[k]) for k in ("num_heads", "key_dim", "value_dim", "decay_rank"))
        self.tau, self.query_scale, self.eps = float(p["tau"]), float(p["query_scale"]), float(p["eps"])
        if not self.tau > 0:
            raise ValueError(f"gla: tau = {self.tau} must be positive")
        t = lambda name: builder.tensor(spec, name)
        # the input products are this part's own, or wider ones that the block makes for all its branches (``input`` "shared")
        self.shared_input = p.get("input") == "shared"
        self.in_rows, self.exact_rows = self.nh * 2 * (self.dk + self.dv), self.rank
        self.qkvg = None if self.shared_input else Linear(t("qkvg"))
        self.low = None if self.shared_input else Linear(t("low"))
        self.out = Linear(t("out"))
        up, self.bias, self.norm_w = t("decay_up"), t("decay_bias"), t("norm")
        want = {"out": (self.out.weight, (self.hidden, self.nh * self.dv)), "decay_up": (up, (self.nh * self.dk, self.rank)),
                "decay_bias": (self.bias, (self.nh * self.dk,)), "norm": (self.norm_w, (self.dv,))}
        if not self.shared_input:
            want.update({"qkvg": (self.qkvg.weight, (self.in_rows, self.hidden)), "low": (self.low.weight, (self.rank, self.hidden))})
        for name, (tensor, shape) in want.items():
            if tuple(tensor.shape) != shape:
                raise ValueError(f"gla: {name} is {tuple(tensor.shape)}, expected {shape}")
        self.decay_up = up.to(torch.float32).t().contiguous()           # neighbouring channels read neighbouring weights

    @staticmethod
    def cache_needs(spec):
        p = spec.params
        return [StateNeed("gla", (int(p["num_heads"]), int(p["key_dim"]), int(p["value_dim"])))]

    def forward(self, h, ctx):
        if self.shared_input:
            raise RuntimeError("gla whose input products are shared gets its rows from the part that makes them")
        return self.forward_rows(self.qkvg(h), 0, ctx, self.low(h, out_dtype=torch.float32), 0)

    def forward_rows(self, rows, col0, ctx, exact, exact_col0):
        """``rows`` [n, >= col0 + in_rows]: q | k | v | gate from column ``col0``; ``exact`` float32: W_1 h from ``exact_col0``."""
        lc = ctx.layer_cache
        if lc is None or not lc.states or "gla" not in lc.states:
            raise RuntimeError("gla needs its state; the step gave it no cache")
        o = ops.gla(rows, exact[:, exact_col0:exact_col0 + self.rank], self.decay_up, self.bias, self.tau, self.norm_w, self.nh, self.dk,
                    self.dv, self.query_scale, self.eps, lc.states["gla"], ctx, col0=col0)
        return self.out(o)
