"""Feed-forwards.

``gated_silu``: down( silu(gate(h)) * up(h) ), silu(z) = z / (1 + exp(-z)), with gate and up
joined into one [2I, H] product (models/qwen3.py:276-287; kernels/elementwise.cpp:529-583).

``routed_gated_silu``: ``experts`` gated-silu feed-forwards of which every token goes through ``top``: the router's
logits W_r h + b are 32-bit, the ``top`` largest choose the experts, their weights are the softmax over those logits
alone, and the output is the weighted sum of the chosen experts' outputs.  A step of few rows (a decode step) reads each
(token, choice)'s expert in the kernel, nothing planned on the host (and so it can be recorded); a prompt's (token,
choice) pairs are grouped by expert on the device and all experts' rows go through two grouped products on the matrix
cores (bfloat16); in the float32 mode, and for sizes those do not take, the host groups the pairs and every expert's
rows go through its two products as ``Linear`` makes them.

``capped_gated``: down( g * sigmoid(slope * g) * (u + shift) ) with g = min(gate(h), limit) and u = clamp(up(h), -limit,
limit); gate and up joined into one [2I, H] product.

``dense``: down(act(up(h))) with an activation chosen by name.  ``xielu`` has two learned numbers p, q (tensor
``activation``, float32 [2]): for z > 0, softplus(p) z^2 + z/2; for z <= 0, (1/2 + softplus(q)) (exp(z) - 1 - z) + z/2.
``relu_squared`` is max(z, 0)^2, ``gelu_erf`` the exact gelu, ``gelu_tanh`` its tanh form.

``routed_scored`` (as follows, with the options named at the end): ``experts`` plain feed-forwards down(gelu(up(h))) (the exact gelu, no biases) of which every token goes
through ``top``.  The router's logits are 32-bit, the scores their sigmoid; the choice is made by score plus the tensor
``correction``, the weights by the scores without it: the chosen experts' scores over their sum (+ 1e-20), times ``scale``.
With ``groups`` the experts lie in that many equal groups of neighbours, a group ranks by the sum of its two largest
corrected scores, and only experts of the best ``keep`` groups can be chosen.  With ``shared_size`` one more expert of that
inner size runs for every token and is added, times the sigmoid of one more router row (the last row of the tensor
``router``), one number per token.  The experts run as those of ``routed_gated_silu`` do.

Options of ``routed_scored``: ``form`` "capped_gated": the experts are those of ``capped_gated`` (tensors ``up`` and ``shared_up``
then hold gate rows before up rows, expert by expert), with ``limit`` and for the shared expert ``shared_limit``; ``score``
"softmax": the scores are the softmax over all experts' logits; ``group_score`` "largest": a group ranks by its largest score;
``shared_gate`` false: the shared expert's output is added as it is.  ``input`` "shared": the shared expert's first product and
the router's are columns of wider products that the block makes for all its branches (``forward_rows``); rows that another
branch of the block made can be added where the experts' weighted sum is written (``addend``).

``routed_table``: no router: the integer tensor ``table`` [vocab, top] gives every token id its experts (the entries of a row
differ), and each weighs 1 / top.  Plain experts (``form`` "relu_squared": down(max(up(h), 0)^2), or "gelu").  With ``shared_size`` one more
expert of the same form and of that inner size runs for every token and is added; in a step of few rows it runs in the
experts' own kernels."""
from __future__ import annotations

import numpy as np
import torch

from ..kernels import ops
from .base import register_part
from .linear import Linear
from .residual import as_tensor


@register_part("feed_forward", "gated_silu")
class GatedSiluFeedForward:
    capturable = True

    def __init__(self, spec, builder):
        self.hidden = int(spec.params["hidden_size"])
        self.inter = int(spec.params["intermediate_size"])
        bias = lambda name: builder.tensor(spec, name) if name in spec.tensors else None
        self.gate_up = Linear(builder.tensor(spec, "gate_up"), bias("gate_up_bias"))
        self.down = Linear(builder.tensor(spec, "down"), bias("down_bias"))
        if self.gate_up.weight.shape != (2 * self.inter, self.hidden) or self.down.weight.shape != (self.hidden, self.inter):
            raise ValueError(f"feed-forward: weights {tuple(self.gate_up.weight.shape)}, {tuple(self.down.weight.shape)} "
                             f"do not fit hidden {self.hidden}, intermediate {self.inter}")

    takes_sink = True

    def forward(self, h, ctx, sink=None):
        return self.down(self.gate_up.gated(h), sink=sink)


@register_part("feed_forward", "capped_gated")
class CappedGatedFeedForward:
    capturable = True

    def __init__(self, spec, builder):
        p = spec.params
        self.hidden, self.inter = int(p["hidden_size"]), int(p["intermediate_size"])
        self.limit, self.slope, self.shift = float(p["limit"]), float(p.get("slope", 1.0)), float(p.get("shift", 0.0))
        if not self.limit > 0:
            raise ValueError(f"feed-forward: limit = {self.limit} must be positive")
        self.gate_up = Linear(builder.tensor(spec, "gate_up"))
        self.down = Linear(builder.tensor(spec, "down"))
        if self.gate_up.weight.shape != (2 * self.inter, self.hidden) or self.down.weight.shape != (self.hidden, self.inter):
            raise ValueError(f"feed-forward: weights {tuple(self.gate_up.weight.shape)}, {tuple(self.down.weight.shape)} "
                             f"do not fit hidden {self.hidden}, intermediate {self.inter}")

    def forward(self, h, ctx):
        return self.down(ops.capped_gate(self.gate_up(as_tensor(h)), self.limit, self.slope, self.shift))


@register_part("feed_forward", "dense")
class DenseFeedForward:
    capturable = True
    ACTIVATIONS = ("xielu", "relu_squared", "gelu_erf", "gelu_tanh")

    def __init__(self, spec, builder):
        self.hidden = int(spec.params["hidden_size"])
        self.inter = int(spec.params["intermediate_size"])
        self.activation = str(spec.params.get("activation", "xielu"))
        if self.activation not in self.ACTIVATIONS:
            raise ValueError(f"feed-forward: activation {self.activation!r} is not one of {self.ACTIVATIONS}")
        self.up = Linear(builder.tensor(spec, "up"))
        self.down = Linear(builder.tensor(spec, "down"))
        self.act_params = builder.tensor(spec, "activation") if self.activation == "xielu" else None
        if self.up.weight.shape != (self.inter, self.hidden) or self.down.weight.shape != (self.hidden, self.inter):
            raise ValueError(f"feed-forward: weights {tuple(self.up.weight.shape)}, {tuple(self.down.weight.shape)} "
                             f"do not fit hidden {self.hidden}, intermediate {self.inter}")
        if self.act_params is not None and self.act_params.shape != (2,):
            raise ValueError(f"feed-forward: xielu takes two numbers, got {tuple(self.act_params.shape)}")

    takes_sink = True

    def forward(self, h, ctx, sink=None):
        z = self.up(as_tensor(h))
        mid = ops.xielu(z, self.act_params) if self.act_params is not None else ops.activation(z, self.activation)
        return self.down(mid, sink=sink)


class RoutedExperts:
    """The experts of a routed feed-forward and how a step's rows go through them, whatever chose them.  ``form``:
    "gated_silu" (an expert's first matrix holds its gate rows, then its up rows), "gelu" or "relu_squared" (up rows alone), or "capped_gated"
    (gate rows and up rows, capped as ``cap`` = (limit, slope, shift) says)."""
    DIRECT_ROWS = 128            # as many rows as a recorded step holds at most

    def _set_experts(self, first, down, experts: int, inter: int, hidden: int, form: str, cap=ops.NO_CAP):
        self.cap = cap
        self.first, self.down_all, self.form = first, down, form
        self.experts, self.inter, self.hidden = experts, inter, hidden
        per = ops.expert_rows(form) * inter
        if first.shape != (experts * per, hidden) or down.shape != (experts * hidden, inter):
            raise ValueError(f"routed feed-forward: weights {tuple(first.shape)}, {tuple(down.shape)} do not fit {experts} experts of inner "
                             f"size {inter} over hidden {hidden}")
        # every expert's two matrices as products of their own, for the rows that a prompt sends it
        self.expert_first = [Linear(first[e * per:(e + 1) * per]) for e in range(experts)]
        self.expert_down = [Linear(down[e * hidden:(e + 1) * hidden]) for e in range(experts)]

    def _mid(self, e: int, xs):
        if self.form == "gated_silu":
            return self.expert_first[e].gated(xs)
        z = self.expert_first[e](xs)
        return ops.capped_gate(z, *self.cap) if self.form == "capped_gated" else ops.activation(z, ops.PLAIN_EXPERTS[self.form])

    def run_few(self, h, chosen, weight, add=(), ids=None, shared=None, planes_ok=False):
        """``run_experts`` for at most DIRECT_ROWS rows, planned nowhere: the matrix cores, or the kernels that each (row, choice)
        reads its expert in.  ``ids``, ``shared``: see ``ops.moe_experts``; ``planes_ok``: float32 planes may come back."""
        args = (h, self.first, self.down_all, chosen, weight, self.inter, self.form, self.cap, add, ids, shared)
        if ops.moe_few_serves(h, self.first, self.inter, self.experts, chosen.shape[1], shared):
            return ops.moe_few(*args, planes_ok=planes_ok)
        return ops.moe_experts(*args)

    def run_experts(self, h, chosen, weight, add=()):
        """float32 [n, hidden]: sum_c weight[t, c] * expert chosen[t, c] of h[t], plus the rows ``add`` (up to two)."""
        top = chosen.shape[1]
        if h.shape[0] <= self.DIRECT_ROWS:
            return self.run_few(h, chosen, weight, add)
        if ops.moe_grouped_serves(h, self.first, self.inter):
            return ops.moe_grouped(h, self.first, self.down_all, chosen, weight, self.inter, self.form, self.cap, add)
        # group the (token, choice) pairs by expert; within an expert in the order of the tokens
        flat = chosen.to("cpu").numpy().reshape(-1)
        order = np.argsort(flat, kind="stable").astype(np.int32)
        counts = np.bincount(flat, minlength=self.experts)
        src = torch.from_numpy(order // top).to(h.device)                        # the token of every pair, grouped
        pair_weight = weight.reshape(-1)
        xs = ops.gather_rows(h, src)
        ws = ops.gather_rows(pair_weight.reshape(-1, 1), torch.from_numpy(order).to(h.device)).reshape(-1)
        out = torch.zeros((h.shape[0], self.hidden), dtype=torch.float32, device=h.device)
        if add:
            every = torch.arange(h.shape[0], dtype=torch.int32, device=h.device)
            ones = torch.ones((h.shape[0],), dtype=torch.float32, device=h.device)
            for y in add:
                ops.scatter_add(out, y, every, ones)
        at = 0
        for e in range(self.experts):
            n = int(counts[e])
            if n:
                y = self.expert_down[e](self._mid(e, xs[at:at + n]))
                ops.scatter_add(out, y, src[at:at + n], ws[at:at + n])
                at += n
        return out


@register_part("feed_forward", "routed_gated_silu")
class RoutedGatedSiluFeedForward(RoutedExperts):
    capturable = True            # steps of up to DIRECT_ROWS rows plan nothing on the host; longer ones are never recorded

    def __init__(self, spec, builder):
        p = spec.params
        self.top = int(p["top"])
        E = int(p["num_experts"])
        if not 1 <= self.top <= E:
            raise ValueError(f"routed feed-forward: {self.top} of {E} experts a token")
        self.router = Linear(builder.tensor(spec, "router"), builder.tensor(spec, "router_bias") if "router_bias" in spec.tensors else None)
        if self.router.weight.shape != (E, int(p["hidden_size"])):
            raise ValueError(f"routed feed-forward: router {tuple(self.router.weight.shape)} does not fit {E} experts")
        self._set_experts(builder.tensor(spec, "gate_up"), builder.tensor(spec, "down"), E, int(p["intermediate_size"]), int(p["hidden_size"]),
                          "gated_silu")
        self.gate_up, self.down = self.first, self.down_all
        self.expert_gate_up = self.expert_first

    def forward(self, h, ctx):
        h = as_tensor(h)
        chosen, weight = ops.moe_route(self.router(h, out_dtype=torch.float32), self.top)
        return self.run_experts(h, chosen, weight)


@register_part("feed_forward", "routed_scored")
class RoutedScoredFeedForward(RoutedExperts):
    capturable = True
    FORMS = ("gelu", "capped_gated")

    def __init__(self, spec, builder):
        p = spec.params
        W, E = int(p["hidden_size"]), int(p["num_experts"])
        self.top, self.scale = int(p["top"]), float(p.get("scale", 1.0))
        self.groups, self.keep = int(p.get("groups") or 1), int(p.get("keep") or 1)
        self.score, self.group_score = str(p.get("score", "sigmoid")), str(p.get("group_score", "two_largest"))
        form = str(p.get("form", "gelu"))
        if form not in self.FORMS:
            raise ValueError(f"routed feed-forward: form {form!r} is not one of {self.FORMS}")
        if not 1 <= self.top <= E or E % self.groups or not 1 <= self.keep <= self.groups or self.keep * (E // self.groups) < self.top:
            raise ValueError(f"routed feed-forward: {self.top} of {E} experts a token, from {self.keep} of {self.groups} groups")
        cap = lambda limit: (float(p[limit]), float(p.get("slope", 1.0)), float(p.get("shift", 0.0))) if form == "capped_gated" else ops.NO_CAP
        self.shared = int(p["shared_size"]) if p.get("shared_size") else None
        self.shared_gate = bool(self.shared) and bool(p.get("shared_gate", True))
        self.shared_input = p.get("input") == "shared"
        self._set_experts(builder.tensor(spec, "up"), builder.tensor(spec, "down"), E, int(p["intermediate_size"]), W, form, cap("limit"))
        per = ops.expert_rows(form)
        # what the block's wider products make for this part: the shared expert's first rows; the router's logits
        self.in_rows, self.exact_rows = per * (self.shared or 0), E + (1 if self.shared_gate else 0)
        self.router = None if self.shared_input else Linear(builder.tensor(spec, "router"))   # the experts' rows (, the shared expert's gate row)
        if self.router is not None and self.router.weight.shape != (self.exact_rows, W):
            raise ValueError(f"routed feed-forward: router {tuple(self.router.weight.shape)} does not fit {E} experts"
                             + (" and a shared expert's gate" if self.shared_gate else ""))
        self.correction = builder.tensor(spec, "correction") if "correction" in spec.tensors else None
        if self.shared:
            self.shared_cap = cap("shared_limit")
            self.shared_up = None if self.shared_input else Linear(builder.tensor(spec, "shared_up"))
            self.shared_down = Linear(builder.tensor(spec, "shared_down"))
            if (self.shared_up is not None and self.shared_up.weight.shape != (self.in_rows, W)) or self.shared_down.weight.shape != (W, self.shared):
                raise ValueError(f"routed feed-forward: the shared expert's weights do not fit inner size {self.shared} over hidden {W}: down "
                                 f"{tuple(self.shared_down.weight.shape)}")

    def forward(self, h, ctx, addend=None):
        h = as_tensor(h)
        if self.shared_input:
            raise RuntimeError("a routed feed-forward whose input products are shared gets its rows from the part that makes them")
        return self._run(h, self.router(h, out_dtype=torch.float32), self.shared_up(h) if self.shared else None, addend)

    def forward_rows(self, h, rows, col0, ctx, exact, exact_col0, addend=None):
        """``rows`` [n, >= col0 + in_rows]: the shared expert's first product from column ``col0``; ``exact`` float32: the router's
        logits from ``exact_col0`` on."""
        return self._run(h, exact[:, exact_col0:], rows[:, col0:col0 + self.in_rows] if self.shared else None, addend)

    takes_addend = True

    def _run(self, h, logits, first, addend):
        chosen, weight = ops.moe_route_scored(logits, self.experts, self.top, self.correction, self.groups, self.keep, self.scale,
                                              self.score, self.group_score)
        add = [] if addend is None else [addend]
        if self.shared:
            mid = ops.capped_gate(first, *self.shared_cap) if self.form == "capped_gated" else ops.activation(first.contiguous(), "gelu_erf")
            y = self.shared_down(mid)
            if not self.shared_gate:
                add.append(y)
        out = self.run_experts(h, chosen, weight, add)
        if self.shared_gate:
            ops.add_gated_rows(out, y, logits, self.experts)
        return out


@register_part("feed_forward", "routed_table")
class RoutedTableFeedForward(RoutedExperts):
    capturable = True
    takes_sink = True            # (for planes of partial sums, which the norm that reads the stream next adds)
    SHARED_DIRECT_ROWS = 16      # as many rows share the shared expert's weights well enough when each reads them for itself

    def __init__(self, spec, builder):
        p = spec.params
        W, E = int(p["hidden_size"]), int(p["num_experts"])
        self.top = int(p["top"])
        form = str(p.get("form", "relu_squared"))
        if form not in ops.PLAIN_EXPERTS:
            raise ValueError(f"routed feed-forward: form {form!r} is not one of {sorted(ops.PLAIN_EXPERTS)}")
        self.table = builder.tensor(spec, "table")
        if self.table.shape != (int(p["vocab_size"]), self.top) or not 1 <= self.top <= E:
            raise ValueError(f"routed feed-forward: the table {tuple(self.table.shape)} is not [{p['vocab_size']}, {self.top}] over {E} experts")
        # the kernels take the entries as they are
        low, high = int(self.table.min()), int(self.table.max())
        if low < 0 or high >= E:
            raise ValueError(f"routed feed-forward: the table names expert {low if low < 0 else high}; there are {E}")
        self._set_experts(builder.tensor(spec, "up"), builder.tensor(spec, "down"), E, int(p["intermediate_size"]), W, form)
        self.shared = None
        if p.get("shared_size"):
            self.shared = (Linear(builder.tensor(spec, "shared_up")), Linear(builder.tensor(spec, "shared_down")))
            shapes = tuple(tuple(s.weight.shape) for s in self.shared)
            if shapes != ((int(p["shared_size"]), W), (W, int(p["shared_size"]))):
                raise ValueError(f"routed feed-forward: the shared expert's weights {shapes} do not fit inner size {p['shared_size']} over hidden {W}")
            self.shared_fits = (all(s.weight.dtype == self.first.dtype for s in self.shared)
                                and self.top * self.inter + int(p["shared_size"]) <= ops.MOE_ROW_VALUES)

    def forward(self, h, ctx, sink=None):
        h = as_tensor(h)
        out = self._run(h, ctx, sink is not None and sink.takes_planes)
        return out if sink is None else sink.finish(out)

    def _run(self, h, ctx, planes_ok):
        n, shared = h.shape[0], tuple(s.weight for s in self.shared) if self.shared is not None else None
        # in a step of few rows the shared expert rides in the experts' own kernels
        rides = shared is not None and n <= self.DIRECT_ROWS and (
            ops.moe_few_serves(h, self.first, self.inter, self.experts, self.top, shared) or (n <= self.SHARED_DIRECT_ROWS and self.shared_fits))
        add = []
        if shared is not None and not rides:
            up, down = self.shared
            add.append(down(ops.activation(up(h), ops.PLAIN_EXPERTS[self.form])))
        if n <= self.DIRECT_ROWS:
            return self.run_few(h, self.table, None, add, ids=ctx.token_ids, shared=shared if rides else None, planes_ok=planes_ok)
        if ops.moe_grouped_serves(h, self.first, self.inter):
            return ops.moe_grouped(h, self.first, self.down_all, self.table, None, self.inter, self.form, self.cap, add, ids=ctx.token_ids)
        chosen, weight = ops.moe_route_table(ctx.token_ids, self.table)
        return self.run_experts(h, chosen, weight, add)
