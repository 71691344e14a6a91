"""Attention whose keys and values are made from one compressed row per position.

    [c_q' | c' | r'] = W_down h                 one joined product (the per-head output gates ride in it too)
    c_q = norm(c_q'),  q = W_uq c_q             per head [plain (key_dim) | to rotate (rot_dim)]
    c = norm(c'),      r = rotate(r')           the cache keeps [c | r] for every position: kv_rank + rot_dim values
    head h: key_j = [U_k,h c_j | r_j],  value_j = U_v,h c_j
    score = (q_plain . U_k,h c_j + rotate(q_rot) . r_j) * scale over the visible positions (causal; the last ``window``)
    out = W_o concat_h( sigmoid(gate_h) * sum_j softmax_j(score) value_j )

Keys and values are never expanded: q_plain goes through U_k,h once (a_h = U_k,h^T q_plain, kv_rank values), the scores
are a_h . c_j + q_rot . r_j, the weighted sum is taken over the rows c_j, and U_v,h is applied to the sum.  All heads read
the same rows.  The rotation's angles and the scores, weights and sums are 32-bit.  In the bfloat16 mode the cache keeps the
latents a second time with the positions innermost, which is how the kernels on the matrix cores read them (prompts, and
single tokens with their key range in slices); the float32 mode and sizes those do not take go through the exact kernel, which
reads the rows alone.  A long prompt is the exception: there the keys and values of every visible position are expanded by two
products (a score then takes key_dim + rot_dim multiply-adds instead of kv_rank + rot_dim), where that pays.

Options: without ``q_rank`` the joined product makes the queries themselves (q = W_q h, no latent, no norm; tensor ``down``: q
| latent and key part | gates).  ``sink`` "learned": head h's softmax has one more term exp(sink_h) in its denominator (tensor
``sink_scores``).  The position part's ``pairing`` may be "interleaved" (dimension 2i with 2i + 1).  ``kv`` "borrowed": the part
makes no latents; its run-order entry reads the rows that another entry wrote (``cache_of``), with its own queries, key and
value matrices, window and sinks.  ``storage_window``: the window by which the rows are kept if other entries read them with a
longer one (None: every position).
"""
from __future__ import annotations

from ..cache import RowsNeed
from ..kernels import ops
from .base import register_part
from .linear import Linear


@register_part("mixer", "latent_attention")
class LatentAttention:
    capturable = True

    def __init__(self, spec, builder):
        p = spec.params
        self.hidden = int(p["hidden_size"])
        self.nh, self.dk, self.dr, self.dv = int(p["num_heads"]), int(p["key_dim"]), int(p["rot_dim"]), int(p["value_dim"])
        self.q_rank, self.kv_rank = int(p["q_rank"]) if p.get("q_rank") else None, int(p["kv_rank"])
        self.scale, self.eps = float(p["scale"]), float(p["eps"])
        self.window = int(p["window"]) if p.get("window") else None
        self.gated = bool(p.get("gated", False))
        self.borrows = p.get("kv", "own") == "borrowed"
        if p.get("kv", "own") not in ("own", "borrowed") or (self.borrows and self.q_rank):
            raise ValueError(f"latent attention: kv {p.get('kv')!r} is 'own', or 'borrowed' by a part whose queries have no latent")
        if p.get("sink") not in (None, "learned"):
            raise ValueError(f"latent attention: sink {p.get('sink')!r} is neither None nor 'learned'")
        t = lambda name: builder.tensor(spec, name)
        q_size = self.nh * (self.dk + self.dr)
        self.down = Linear(t("down"))
        self.out = Linear(t("out"))
        self.uk, self.uv = t("uk"), t("uv")
        self.sink = t("sink_scores") if p.get("sink") else None
        # columns of the joined product: the queries' latent (or the queries), the row's latent and key part, the gates
        self.kv_off = self.q_rank or q_size
        self.gate_off = self.kv_off + (0 if self.borrows else self.kv_rank + self.dr)
        want = {"down": (self.down.weight, (self.gate_off + (self.nh if self.gated else 0), self.hidden)),
                "out": (self.out.weight, (self.hidden, self.nh * self.dv)), "uk": (self.uk, (self.nh * self.dk, self.kv_rank)),
                "uv": (self.uv, (self.nh * self.dv, self.kv_rank))}
        if self.q_rank:
            self.uq, self.q_norm_w = Linear(t("uq")), t("q_norm")
            want.update(uq=(self.uq.weight, (q_size, self.q_rank)), q_norm=(self.q_norm_w, (self.q_rank,)))
        if not self.borrows:
            self.kv_norm_w = t("kv_norm")
            want["kv_norm"] = (self.kv_norm_w, (self.kv_rank,))
        if self.sink is not None:
            want["sink_scores"] = (self.sink, (self.nh,))
        for name, (tensor, shape) in want.items():
            if tuple(tensor.shape) != shape:
                raise ValueError(f"latent attention: {name} is {tuple(tensor.shape)}, expected {shape}")
        self.position = builder.build(spec.parts["position"]) if "position" in spec.parts and self.dr else None
        if self.position is not None and self.position.rotary_dim != self.dr:
            raise ValueError("latent attention: the rotation covers the whole rotated part")
        self.pairing = self.position.pairing if self.position is not None else "half_split"
        self.uk_t = ops.latent_key_transposes(self.uk, self.nh, self.dk, self.kv_rank)
        self.dtype = builder.dtype

    @staticmethod
    def cache_needs(spec):
        p = spec.params
        if p.get("kv", "own") == "borrowed":
            raise ValueError("latent attention that borrows its rows runs as an entry that reads another entry's cache")
        window = int(p["window"]) if p.get("window") else None
        if "storage_window" in p:                       # others read these rows, by windows of their own
            window = int(p["storage_window"]) if p["storage_window"] else None
        # the rows, and the latents once more in bfloat16 for the kernels on the matrix cores (a page of them is read
        # there with the positions innermost: [kv_rank, 64] in the room of [64, kv_rank])
        return [RowsNeed("latent", (int(p["kv_rank"]) + int(p["rot_dim"]),), None, window),
                RowsNeed("latent_t", (int(p["kv_rank"]),), "bfloat16", window)]

    @staticmethod
    def cache_needs_beside_shared(spec):
        return []

    def forward(self, h, ctx):
        lc = ctx.layer_cache
        if lc is None or not lc.rows or "latent" not in lc.rows:
            raise RuntimeError("latent attention needs the rows of its layer; the step gave it no cache")
        if self.borrows and lc.writes:
            raise RuntimeError("latent attention: a part without latents of its own reads another entry's rows")
        view = lc.rows["latent"]
        rows_t = table_t = None
        if "latent_t" in lc.rows and ops.latent_mfma_serves(view.data, self.kv_rank, self.dr):
            turned = lc.rows["latent_t"]
            rows_t, table_t = turned.data.view(turned.data.shape[0], self.kv_rank, turned.data.shape[1]), turned.table_dev
        down = self.down(h)
        tables = self.position.tables(ctx) if self.position is not None else None
        cos, sin = tables if tables is not None else (None, None)
        sizes = (self.nh, self.dk, self.dr, self.kv_rank)
        if self.q_rank:
            cq = ops.latent_prep(down, self.q_rank, self.kv_off, self.kv_rank, self.dr, self.q_norm_w, self.kv_norm_w, self.eps, cos, sin,
                                 view.data, view.table_dev, ctx, write_cache=lc.writes, rows_t=rows_t, table_t=table_t, pairing=self.pairing)
            q, store = self.uq(cq), None
        else:
            store = None if not lc.writes else ops.LatentStore(down[:, self.kv_off:self.gate_off], self.kv_norm_w, self.eps, view.data,
                                                              view.table_dev, rows_t, table_t)
            q = down[:, :self.kv_off]
        gate = down[:, self.gate_off:] if self.gated else None
        if ops.latent_expanded_serves(q, view.data, self.uk, self.uv, ctx, *sizes, self.dv, self.window):
            return self.out(ops.latent_attention_expanded(q, self.uk, self.uv, cos, sin, *sizes, self.dv, self.pairing, ctx, store, view.data,
                                                          view.table_dev, self.scale, self.window, self.sink, gate))
        qa = ops.latent_query(q, self.uk, cos, sin, *sizes, pairing=self.pairing, ctx=ctx, store=store, uk_t=self.uk_t)
        attend = (qa, view.data, view.table_dev, ctx, self.nh, self.kv_rank, self.dr, self.scale, self.window)
        # on the matrix cores the value matrices and the gates ride in the attention's own launches
        if ops.latent_decode_serves(view.data, rows_t, self.uv, ctx, self.kv_rank, self.dr):
            o = ops.latent_attention_decode(*attend, rows_t, table_t, self.uv, gate, self.dv, sink=self.sink)
        elif ops.latent_fused_serves(qa, view.data, rows_t, self.uv, ctx, self.kv_rank, self.dr, self.dv):
            o = ops.latent_attention_fused(*attend, rows_t, table_t, self.uv, gate, self.dv, sink=self.sink)
        else:
            o_lat = ops.latent_attention(*attend, rows_t=rows_t, table_t=table_t, sink=self.sink)
            o = ops.latent_output(o_lat, self.uv, gate, self.nh, self.kv_rank, self.dv, self.dtype)
        return self.out(o)
