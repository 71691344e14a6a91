"""The typed configuration of the Vovalix decoder and its description as parts.

A Vovalix model is a list of layers whose two branches run side by side on one norm's output, x += mixer(h) + ff(h) with h =
norm(x); norm weights are stored as the distance from one.  A layer's mixer is of one of three kinds:

  gla         linear attention whose state decays by a number for every key channel and token, the decays from a low-rank map
              of the layer's input; each head's output is normed with one weight for all heads and gated by silu
  attention   softmax attention with grouped key/value heads of a key size and a value size of their own, q and k divided by
              their root mean square per head, no rotation: a head's scores fall with the distance by a slope of its own, and
              a query sees the keys of its own chunk of positions only
  delta       a gated delta rule with one decay a head behind short causal convolutions; outputs as gla's

A layer's feed-forward is a mixture of small capped gated experts behind a softmax router that chooses within the best groups
of neighbouring experts, plus a shared expert for every token; or the layer has none.  A layer may use another layer's weights
(``weights_of``) while keeping a cache and state of its own.  The head is the embedding table; the logits are multiplied by
``logit_scale``.

config.json: ``architecture`` "Vovalix", ``vocab``, ``width``, ``norm.eps``, ``logit_scale`` and ``layers``, a list of ``{"type":
"gla", "mixer": {heads, dim, vdim, tau}, "mlp": ..}``, ``{"type": "attention", "mixer": {heads, kv_heads, dim, vdim, scale, mask:
{size}}, "mlp": ..}`` and ``{"type": "delta", "mixer": {heads, kv_heads, dim, vdim, conv}, "mlp": ..}`` with ``mlp`` null or ``{"kind":
"moe", "expert": {ff, limit}, "router": {experts, top, groups: {count, keep}}, "shared": {ff, limit}}`` and optionally
``weights_of``.  A missing ``mask`` is plain causal attention, missing ``groups`` one group, a missing ``shared`` no shared expert, a
missing ``logit_scale`` one.  The rank of gla's low-rank map is the shape of its tensors; a configuration that was not read
beside a checkpoint takes it from ``mixer.decay_rank``.  Tensor names: ``embed``, ``final.norm``, ``l<i>.norm1``,
``l<i>.mix.{q,k,v,o}`` (all), ``l<i>.mix.{g,norm}`` (gla, delta), ``l<i>.mix.{a1,a2}`` and ``a2.b`` (gla),
``l<i>.mix.{q,k,v}.conv`` and ``l<i>.mix.{a,b,A_log,dt_bias}`` (delta), ``l<i>.mlp.e<k>.{gate,up,down}``, ``l<i>.mlp.router``,
``l<i>.mlp.shared.{gate,up,down}``.
"""
from __future__ import annotations

from dataclasses import dataclass, replace

from .registry import ConfigError, register_architecture
from .spec import LayerCall, ModelSpec, PartSpec, joined, tensor

LAYER_TYPES = ("gla", "attention", "delta")
MAX_TAPS, MAX_EXPERTS, MAX_TOP = 16, 512, 64
# an expert's gate is g * sigmoid(GATE_SLOPE * g), and its up row is shifted by UP_SHIFT
GATE_SLOPE, UP_SHIFT = 1.702, 1.0
_AROUND_ZERO = ("normal", 0.0, 0.1)          # norm weights are kept as the distance from one
_AROUND_ONE = ("normal", 1.0, 0.1)


def _get(table, key: str, typ, where: str):
    if not isinstance(table, dict) or key not in table or table[key] is None:
        raise ConfigError(f"config.json: {where} lacks {key!r}")
    try:
        return typ(table[key])
    except (TypeError, ValueError):
        raise ConfigError(f"config.json: {where}.{key} = {table[key]!r} is not {typ.__name__}") from None


def _positive(value, what: str):
    if not value > 0:
        raise ConfigError(f"config.json: {what} = {value} must be positive")
    return value


@register_architecture("Vovalix", model_type="vovalix")
@dataclass(frozen=True)
class VovalixConfig:
    vocab: int
    width: int
    eps: float
    logit_scale: float
    layers: tuple          # of dicts as config.json holds them, checked
    eos_token_ids: tuple = ()

    @classmethod
    def from_dict(cls, raw: dict) -> "VovalixConfig":
        vocab = _positive(_get(raw, "vocab", int, "the model"), "vocab")
        width = _positive(_get(raw, "width", int, "the model"), "width")
        eps = _positive(_get(raw.get("norm"), "eps", float, "norm"), "norm.eps")
        scale = float(raw["logit_scale"]) if raw.get("logit_scale") is not None else 1.0
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        checked = []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            kind = _get(layer, "type", str, where)
            if kind not in LAYER_TYPES:
                raise ConfigError(f"config.json: {where}.type = {kind!r} is not one of {', '.join(LAYER_TYPES)}")
            if not isinstance(layer.get("mixer"), dict):
                raise ConfigError(f"config.json: {where} lacks its mixer's sizes")
            entry = {"type": kind, "mixer": cls._check_mixer(kind, layer["mixer"], where + ".mixer"),
                     "mlp": cls._check_mlp(layer.get("mlp"), where + ".mlp")}
            if layer.get("weights_of") is not None:
                j = _get(layer, "weights_of", int, where)
                if not 0 <= j < len(layers) or j == i:
                    raise ConfigError(f"config.json: {where}.weights_of = {j} names no other layer")
                entry["weights_of"] = j
            checked.append(entry)
        for i, entry in enumerate(checked):
            j = cls._source(checked, i)
            if j != i and any(entry[k] != checked[j][k] for k in ("type", "mixer", "mlp")):
                raise ConfigError(f"config.json: layers[{i}] borrows the weights of layers[{j}], which is another layer in more than its weights")
        eos = raw.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        return cls(vocab, width, eps, scale, tuple(checked), eos_ids)

    @staticmethod
    def _source(layers, i: int) -> int:
        """The layer whose tensors layer i uses (itself, unless it borrows)."""
        seen = set()
        while layers[i].get("weights_of") is not None:
            if i in seen:
                raise ConfigError(f"config.json: layers[{i}].weights_of leads back to itself")
            seen.add(i)
            i = layers[i]["weights_of"]
        return i

    @staticmethod
    def _check_mixer(kind: str, m: dict, where: str) -> dict:
        keys = ("heads", "dim", "vdim") if kind == "gla" else ("heads", "kv_heads", "dim", "vdim")
        out = {k: _positive(_get(m, k, int, where), f"{where}.{k}") for k in keys}
        if "kv_heads" in out and out["heads"] % out["kv_heads"]:
            raise ConfigError(f"config.json: {where}: {out['heads']} heads are not a multiple of {out['kv_heads']} kv heads")
        most = 256 if kind == "attention" else 1024
        if out["dim"] > 256 or out["vdim"] > most:
            raise ConfigError(f"config.json: {where}: {kind} takes key sizes up to 256 and value sizes up to {most}")
        if kind == "gla":
            out["tau"] = _positive(_get(m, "tau", float, where), where + ".tau")
            if m.get("decay_rank") is not None:
                out["decay_rank"] = _positive(_get(m, "decay_rank", int, where), where + ".decay_rank")
        elif kind == "attention":
            out["scale"] = _get(m, "scale", float, where)
            if m.get("mask"):
                out["mask"] = {"size": _positive(_get(m["mask"], "size", int, where + ".mask"), where + ".mask.size")}
        else:
            out["conv"] = _positive(_get(m, "conv", int, where), where + ".conv")
            if out["conv"] > MAX_TAPS:
                raise ConfigError(f"config.json: {where}.conv = {out['conv']}; the convolution takes up to {MAX_TAPS} taps")
        return out

    @staticmethod
    def _check_mlp(f, where: str):
        if f is None:
            return None
        kind = _get(f, "kind", str, where)
        if kind != "moe":
            raise ConfigError(f"config.json: {where}.kind = {kind!r}; this design's feed-forwards are routed experts ('moe')")

        def expert(t, at):
            return {"ff": _positive(_get(t, "ff", int, at), at + ".ff"), "limit": _positive(_get(t, "limit", float, at), at + ".limit")}

        r = f.get("router")
        router = {k: _positive(_get(r, k, int, where + ".router"), f"{where}.router.{k}") for k in ("experts", "top")}
        E, top = router["experts"], router["top"]
        if E > MAX_EXPERTS or top > min(E, MAX_TOP):
            raise ConfigError(f"config.json: {where}.router: {top} of {E} experts (at most {MAX_TOP} of {MAX_EXPERTS})")
        count = keep = 1
        if r.get("groups"):
            count, keep = (_positive(_get(r["groups"], k, int, where + ".router.groups"), f"{where}.router.groups.{k}") for k in ("count", "keep"))
            router["groups"] = {"count": count, "keep": keep}
        if E % count or keep > count or keep * (E // count) < top:
            raise ConfigError(f"config.json: {where}.router: {E} experts in {count} groups of which {keep} are kept cannot give {top} choices")
        out = {"kind": kind, "expert": expert(f.get("expert"), where + ".expert"), "router": router}
        if f.get("shared"):
            out["shared"] = expert(f["shared"], where + ".shared")
        return out

    def with_tensor_shapes(self, shapes: dict) -> "VovalixConfig":
        """The configuration with the size that a checkpoint's tensors give: the rank of a gla layer's decays (rows of
        ``l<i>.mix.a1``)."""
        layers = []
        for i, layer in enumerate(self.layers):
            name = f"l{self._source(self.layers, i)}.mix.a1"
            if layer["type"] == "gla" and len(shapes.get(name, ())) == 2:
                layer = dict(layer, mixer=dict(layer["mixer"], decay_rank=int(shapes[name][0])))
            layers.append(layer)
        return replace(self, layers=tuple(layers))

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "logit_scale": self.logit_scale, "layers": [dict(layer) for layer in self.layers]}
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return d

    # ------------------------------------------------------------------------------------------
    def _mixer(self, i: int, kind: str, m: dict):
        """(description, pieces of the layer's joined input matrix, pieces of its joined matrix with a 32-bit result)."""
        W, p, H, d, dv = self.width, f"l{i}.mix.", m["heads"], m["dim"], m["vdim"]
        out = tensor(p + "o", (W, H * dv), "matrix", ("normal", 0.0, (H * dv) ** -0.5))
        if kind == "attention":
            G = m["kv_heads"]
            part = PartSpec("mixer", "sink_attention",
                            {"hidden_size": W, "num_heads": H, "num_kv_heads": G, "key_dim": d, "value_dim": dv, "scale": m["scale"],
                             "window": m["mask"]["size"] if m.get("mask") else None, "mask": "chunked" if m.get("mask") else "sliding",
                             "distance_bias": "halving", "eps": self.eps, "qk_norm": "head_unit", "sink": None, "gate": None, "input": "shared"},
                            {"out": out})
            return part, [(p + "q", H * d), (p + "k", G * d), (p + "v", G * dv)], []
        norm = tensor(p + "norm", (dv,), "vector", _AROUND_ONE)
        if kind == "gla":
            if "decay_rank" not in m:
                raise ConfigError(f"layers[{i}].mixer: the rank of the decays' low-rank map is given by the shape of {p}a1, or by decay_rank where "
                                  "there is no checkpoint")
            R = m["decay_rank"]
            part = PartSpec("mixer", "gla",
                            {"hidden_size": W, "num_heads": H, "key_dim": d, "value_dim": dv, "decay_rank": R, "tau": m["tau"],
                             "query_scale": d ** -0.5, "eps": self.eps, "input": "shared"},
                            {"decay_up": tensor(p + "a2", (H * d, R), "vector", ("normal", 0.0, R ** -0.5)),
                             "decay_bias": tensor(p + "a2.b", (H * d,), "vector", ("normal", 2.0, 1.0)), "norm": norm, "out": out})
            return part, [(p + "q", H * d), (p + "k", H * d), (p + "v", H * dv), (p + "g", H * dv)], [(p + "a1", R)]
        G, taps = m["kv_heads"], m["conv"]
        part = PartSpec("mixer", "delta_rule_head",
                        {"hidden_size": W, "num_heads": H, "num_qk_heads": G, "key_dim": d, "value_dim": dv, "taps": taps, "eps": self.eps,
                         "input": "shared"},
                        {"conv": joined([p + n + ".conv" for n in "qkv"], [(G * d, taps), (G * d, taps), (H * dv, taps)], "vector", ("normal", 0.0, 0.5)),
                         "a_log": tensor(p + "A_log", (H,), "vector", ("normal", -1.0, 0.5)),
                         "dt_bias": tensor(p + "dt_bias", (H,), "vector", ("normal", -2.0, 1.0)), "norm": norm, "out": out})
        return part, [(p + "q", G * d), (p + "k", G * d), (p + "v", H * dv), (p + "g", H * dv)], [(p + "b", H), (p + "a", H)]

    def _feed_forward(self, p: str, f: dict):
        """(description, pieces of the layer's joined input matrix, pieces of its joined matrix with a 32-bit result)."""
        W, r, F = self.width, f["router"], f["expert"]["ff"]
        E, groups = r["experts"], r.get("groups") or {"count": 1, "keep": 1}
        params = {"hidden_size": W, "intermediate_size": F, "num_experts": E, "top": r["top"], "scale": 1.0, "groups": groups["count"],
                  "keep": groups["keep"], "score": "softmax", "group_score": "largest", "form": "capped_gated", "limit": f["expert"]["limit"],
                  "slope": GATE_SLOPE, "shift": UP_SHIFT, "input": "shared"}
        names = [f"{p}e{e}.{n}" for e in range(E) for n in ("gate", "up")]
        tensors = {"up": joined(names, [(F, W)] * (2 * E), "matrix", ("normal", 0.0, W ** -0.5)),
                   "down": joined([f"{p}e{e}.down" for e in range(E)], [(W, F)] * E, "matrix", ("normal", 0.0, F ** -0.5))}
        rows = []
        if f.get("shared"):
            S = f["shared"]["ff"]
            params.update(shared_size=S, shared_limit=f["shared"]["limit"], shared_gate=False)
            tensors["shared_down"] = tensor(p + "shared.down", (W, S), "matrix", ("normal", 0.0, S ** -0.5))
            rows = [(p + "shared.gate", S), (p + "shared.up", S)]
        return PartSpec("feed_forward", "routed_scored", params, tensors), rows, [(p + "router", E)]

    def spec(self, tensor_names=None) -> ModelSpec:
        W, V, eps = self.width, self.vocab, self.eps

        def norm(name: str, **more) -> PartSpec:
            return PartSpec("norm", "rms", {"width": W, "eps": eps, "offset": 1.0, **more}, {"weight": tensor(name, (W,), "vector", _AROUND_ZERO)})

        layers, index = [], {}                       # layers with tensors of their own; config layer -> its place there
        for i, layer in enumerate(self.layers):
            if layer.get("weights_of") is not None:
                continue
            mixer, rows, exact = self._mixer(i, layer["type"], layer["mixer"])
            parts = {"norm": norm(f"l{i}.norm1"), "mixer": mixer}
            if layer["mlp"] is not None:
                parts["feed_forward"], more_rows, more_exact = self._feed_forward(f"l{i}.mlp.", layer["mlp"])
                rows, exact = rows + more_rows, exact + more_exact
            # both branches read one norm's output: one product makes the rows of both, one what must stay 32-bit
            tensors = {"in": joined([n for n, _ in rows], [(r, W) for _, r in rows], "matrix", ("normal", 0.0, 1.5 * W ** -0.5))}
            if exact:
                tensors["in_exact"] = joined([n for n, _ in exact], [(r, W) for _, r in exact], "matrix", ("normal", 0.0, 1.5 * W ** -0.5))
            index[i] = len(layers)
            layers.append(PartSpec("block", "parallel_pre_norm", {"hidden_size": W}, tensors, parts))
        order = tuple(LayerCall(index[self._source(self.layers, i)]) for i in range(len(self.layers)))

        table = tensor("embed", (V, W), "table", ("normal", 0.0, 1.0))
        return ModelSpec(
            architecture=self.architecture, vocab_size=V, hidden_size=W, max_positions=None,
            embedding=PartSpec("embedding", "token_table", {"vocab_size": V, "hidden_size": W}, {"table": table}),
            # the logits' scale goes into the norm whose rows the head reads
            layers=tuple(layers), order=order, final_norm=norm("final.norm", gain=self.logit_scale),
            head=PartSpec("head", "linear", {"vocab_size": V, "hidden_size": W}, {"weight": table}),
            stop_token_ids=self.eos_token_ids,
        )
