"""The typed configuration of the Nirotar decoder and its description as parts.

A Nirotar model is a list of pre-norm layers, x += mixer(norm(x)); x += ff(norm(x)), each with a mixer of one of two kinds:

  attention         softmax attention with grouped key/value heads of a key size and a value size of their own, no biases, a
                    rotation of the first ``rot.dims`` dimensions of each head in neighbouring pairs (2i with 2i + 1) whose
                    slow frequencies are stretched by wavelength, a sliding window, a learned sink score per head in the
                    softmax's denominator
  latent_attention  softmax attention whose keys and values are made from one normed latent and one rotated key part (shared by
                    all heads, the same pairs) per position, a learned sink score per head, every earlier position in sight.
                    A layer with ``kv_from``: j has no latents of its own: it reads those that layer j cached, with its own
                    queries and its own matrices from latents to keys and values.

A layer's feed-forward is a mixture of small experts down(relu(up(h))^2) that a table chooses by token id (no router; the
chosen experts weigh the same), plus a shared expert of the same form for every token; or the layer has none.  The head is a
matrix of its own.

config.json: ``architecture`` "Nirotar", ``vocab``, ``width``, ``norm.eps`` and ``layers``, a list of ``{"type": "attention",
"mixer": {heads, kv_heads, dim, vdim, scale, mask: {size}, rot: {dims, base, scaling: {factor, low, high, original}}}, "mlp":
..}`` and ``{"type": "latent_attention", "mixer": {heads, dim, rot_dim, vdim, kv_rank, scale, rot: {dims, base}, kv_from},
"mlp": ..}`` with ``mlp`` null or ``{"kind": "moe", "expert": {ff}, "router": {experts, top}, "shared": {ff}}``.  A missing
``mask`` is no window, a missing ``rot.scaling`` plain frequencies, a missing ``rot`` (attention) no rotation, a missing ``shared``
no shared expert.  Tensor names: ``embed``, ``head``, ``final.norm``, ``l<i>.norm1``, ``l<i>.norm2``, ``l<i>.mix.{q,sink,o}``
(both), ``l<i>.mix.{k,v}`` (attention), ``l<i>.mix.{uk,uv}`` and, without ``kv_from``, ``l<i>.mix.dkv`` with ``dkv.norm``
(latent_attention), ``l<i>.mlp.table`` (integers [vocab, top]), ``l<i>.mlp.e<k>.{up,down}``, ``l<i>.mlp.shared.{up,down}``.
"""
from __future__ import annotations

from dataclasses import dataclass

from .registry import ConfigError, register_architecture
from .spec import LayerCall, ModelSpec, PartSpec, joined, tensor

LAYER_TYPES = ("attention", "latent_attention")
MAX_EXPERTS, MAX_TOP = 512, 64
_NORM_INIT = ("normal", 1.0, 0.1)


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


@register_architecture("Nirotar", model_type="nirotar")
@dataclass(frozen=True)
class NirotarConfig:
    vocab: int
    width: int
    eps: float
    layers: tuple          # of dicts as config.json holds them, checked
    eos_token_ids: tuple = ()

    @classmethod
    def from_dict(cls, raw: dict) -> "NirotarConfig":
        vocab = _positive(_get(raw, "vocab", int, "the model"), "vocab")
        width = _positive(_get(raw, "width", int, "the model"), "width")
        eps = _positive(_get(raw.get("norm"), "eps", float, "norm"), "norm.eps")
        layers = raw.get("layers")
        if not isinstance(layers, list) or not layers:
            raise ConfigError("config.json: 'layers' must be a list with at least one layer")
        checked = []
        for i, layer in enumerate(layers):
            where = f"layers[{i}]"
            kind = _get(layer, "type", str, where)
            if kind not in LAYER_TYPES:
                raise ConfigError(f"config.json: {where}.type = {kind!r} is not one of {', '.join(LAYER_TYPES)}")
            m = layer.get("mixer")
            if not isinstance(m, dict):
                raise ConfigError(f"config.json: {where} lacks its mixer's sizes")
            check = cls._check_attention if kind == "attention" else cls._check_latent
            checked.append({"type": kind, "mixer": check(m, where + ".mixer"), "mlp": cls._check_mlp(layer.get("mlp"), where + ".mlp")})
        for i, layer in enumerate(checked):
            j = layer["mixer"].get("kv_from")
            if j is None:
                continue
            where = f"layers[{i}].mixer"
            if not 0 <= j < i or checked[j]["type"] != "latent_attention" or checked[j]["mixer"].get("kv_from") is not None:
                raise ConfigError(f"config.json: {where}.kv_from = {j} must name an earlier latent_attention layer with latents of its own")
            a, b = layer["mixer"], checked[j]["mixer"]
            if any(a.get(k) != b.get(k) for k in ("kv_rank", "rot_dim", "rot")):
                raise ConfigError(f"config.json: {where} reads layer {j}'s latents but has another kv_rank, rot_dim or rotation")
        eos = raw.get("eos_token_id")
        eos_ids = () if eos is None else tuple(int(e) for e in (eos if isinstance(eos, (list, tuple)) else [eos]))
        return cls(vocab, width, eps, tuple(checked), eos_ids)

    @staticmethod
    def _check_mask(m: dict, out: dict, where: str) -> None:
        if m.get("mask"):
            out["mask"] = {"size": _positive(_get(m["mask"], "size", int, where + ".mask"), where + ".mask.size")}

    @staticmethod
    def _check_rot(rot, where: str) -> dict:
        out = {"dims": _get(rot, "dims", int, where), "base": _positive(_get(rot, "base", float, where), where + ".base")}
        if out["dims"] <= 0 or out["dims"] % 2:
            raise ConfigError(f"config.json: {where}.dims = {out['dims']} must be even and positive")
        if rot.get("scaling"):
            sc = {k: _positive(_get(rot["scaling"], k, float, where + ".scaling"), f"{where}.scaling.{k}")
                  for k in ("factor", "low", "high", "original")}
            if sc["high"] <= sc["low"]:
                raise ConfigError(f"config.json: {where}.scaling: high = {sc['high']} must lie above low = {sc['low']}")
            out["scaling"] = sc
        return out

    @classmethod
    def _check_attention(cls, m: dict, where: str) -> dict:
        out = {k: _positive(_get(m, k, int, where), f"{where}.{k}") for k in ("heads", "kv_heads", "dim", "vdim")}
        if out["heads"] % out["kv_heads"]:
            raise ConfigError(f"config.json: {where}: {out['heads']} heads are not a multiple of {out['kv_heads']} kv heads")
        if out["dim"] > 256 or out["vdim"] > 256:
            raise ConfigError(f"config.json: {where}: the attention kernels take key and value sizes up to 256")
        out["scale"] = _get(m, "scale", float, where)
        cls._check_mask(m, out, where)
        if m.get("rot"):
            out["rot"] = cls._check_rot(m["rot"], where + ".rot")
            if out["rot"]["dims"] > out["dim"]:
                raise ConfigError(f"config.json: {where}.rot.dims = {out['rot']['dims']} exceeds the key size {out['dim']}")
        return out

    @classmethod
    def _check_latent(cls, m: dict, where: str) -> dict:
        out = {k: _positive(_get(m, k, int, where), f"{where}.{k}") for k in ("heads", "dim", "vdim", "kv_rank", "rot_dim")}
        out["scale"] = _get(m, "scale", float, where)
        if out["kv_rank"] > 1024 or out["kv_rank"] + out["rot_dim"] > 1280 or out["dim"] > 512:
            raise ConfigError(f"config.json: {where}: the attention kernels take latents up to 1024 (with the rotated part 1280) and "
                              "unrotated key sizes up to 512")
        cls._check_mask(m, out, where)
        out["rot"] = cls._check_rot(m.get("rot"), where + ".rot")
        if out["rot"]["dims"] != out["rot_dim"]:
            raise ConfigError(f"config.json: {where}.rot.dims = {out['rot']['dims']}: the whole rotated part of {out['rot_dim']} is rotated")
        if m.get("kv_from") is not None:
            out["kv_from"] = _get(m, "kv_from", int, where)
        return out

    @staticmethod
    def _check_mlp(f, where: str):
        if f is None:
            return None
        kind = _get(f, "kind", str, where)
        if kind != "moe":
            raise ConfigError(f"config.json: {where}.kind = {kind!r}; this design's feed-forwards are chosen experts ('moe')")
        experts = _positive(_get(f.get("router"), "experts", int, where + ".router"), where + ".router.experts")
        top = _positive(_get(f.get("router"), "top", int, where + ".router"), where + ".router.top")
        if experts > MAX_EXPERTS or top > min(experts, MAX_TOP):
            raise ConfigError(f"config.json: {where}.router: {top} of {experts} experts (at most {MAX_TOP} of {MAX_EXPERTS})")
        out = {"kind": kind, "expert": {"ff": _positive(_get(f.get("expert"), "ff", int, where + ".expert"), where + ".expert.ff")},
               "router": {"experts": experts, "top": top}}
        if f.get("shared"):
            out["shared"] = {"ff": _positive(_get(f["shared"], "ff", int, where + ".shared"), where + ".shared.ff")}
        return out

    def to_dict(self) -> dict:
        d = {"architecture": self.architecture, "vocab": self.vocab, "width": self.width, "norm": {"eps": self.eps},
             "layers": [dict(layer) for layer in self.layers]}
        if self.eos_token_ids:
            d["eos_token_id"] = self.eos_token_ids[0] if len(self.eos_token_ids) == 1 else list(self.eos_token_ids)
        return d

    # ------------------------------------------------------------------------------------------
    @staticmethod
    def _position(rot: dict) -> PartSpec:
        scaling = dict(rot["scaling"], kind="wavelength") if rot.get("scaling") else None
        return PartSpec("position", "rotary", {"rotary_dim": rot["dims"], "theta": rot["base"], "pairing": "interleaved", "scaling": scaling,
                                               "exact_frequencies": True})

    def _attention(self, p: str, m: dict) -> PartSpec:
        W, H, G, d, dv = self.width, m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        return PartSpec(
            "mixer", "sink_attention",
            {"hidden_size": W, "num_heads": H, "num_kv_heads": G, "key_dim": d, "value_dim": dv, "scale": m["scale"],
             "window": m["mask"]["size"] if m.get("mask") else None, "eps": self.eps, "qk_norm": None, "sink": "learned", "gate": None},
            {"qkvg": joined([p + n for n in "qkv"], [(H * d, W), (G * d, W), (G * dv, W)], "matrix", ("normal", 0.0, 1.5 * W ** -0.5)),
             "sink_scores": tensor(p + "sink", (H,), "vector", ("normal", 0.0, 1.0)),
             "out": tensor(p + "o", (W, H * dv), "matrix", ("normal", 0.0, (H * dv) ** -0.5))},
            {"position": self._position(m["rot"])} if m.get("rot") else {})

    def _storage_window(self, i: int):
        """By which window layer i's latents are kept: the longest of its own and its readers' (None: all)."""
        sizes = [layer["mixer"].get("mask") for k, layer in enumerate(self.layers)
                 if k == i or (layer["type"] == "latent_attention" and layer["mixer"].get("kv_from") == i)]
        return None if any(s is None for s in sizes) else max(int(s["size"]) for s in sizes)

    def _latent(self, i: int, p: str, m: dict) -> PartSpec:
        W, H, d, dr, dv, R = self.width, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        borrows = m.get("kv_from") is not None
        names, shapes = [p + "q"], [(H * (d + dr), W)]
        params = {"hidden_size": W, "num_heads": H, "key_dim": d, "rot_dim": dr, "value_dim": dv, "kv_rank": R, "q_rank": None,
                  "scale": m["scale"], "window": m["mask"]["size"] if m.get("mask") else None, "eps": self.eps, "gated": False,
                  "sink": "learned", "kv": "borrowed" if borrows else "own"}
        tensors = {"uk": tensor(p + "uk", (H * d, R), "matrix", ("normal", 0.0, 1.5 * R ** -0.5)),
                   "uv": tensor(p + "uv", (H * dv, R), "matrix", ("normal", 0.0, R ** -0.5)),
                   "sink_scores": tensor(p + "sink", (H,), "vector", ("normal", 0.0, 1.0)),
                   "out": tensor(p + "o", (W, H * dv), "matrix", ("normal", 0.0, (H * dv) ** -0.5))}
        if not borrows:
            names.append(p + "dkv")
            shapes.append((R + dr, W))
            params["storage_window"] = self._storage_window(i)
            tensors["kv_norm"] = tensor(p + "dkv.norm", (R,), "vector", _NORM_INIT)
        tensors["down"] = joined(names, shapes, "matrix", ("normal", 0.0, 1.5 * W ** -0.5))
        return PartSpec("mixer", "latent_attention", params, tensors, {"position": self._position(m["rot"])})

    def _feed_forward(self, p: str, f: dict) -> PartSpec:
        W, F, E, top = self.width, f["expert"]["ff"], f["router"]["experts"], f["router"]["top"]
        params = {"hidden_size": W, "intermediate_size": F, "num_experts": E, "top": top, "vocab_size": self.vocab, "form": "relu_squared"}
        tensors = {"table": tensor(p + "table", (self.vocab, top), "integer", ("distinct", E)),
                   "up": joined([f"{p}e{e}.up" for e in range(E)], [(F, W)] * E, "matrix", ("normal", 0.0, W ** -0.5)),
                   "down": joined([f"{p}e{e}.down" for e in range(E)], [(W, F)] * E, "matrix", ("normal", 0.0, F ** -0.5))}
        if f.get("shared"):
            S = params["shared_size"] = f["shared"]["ff"]
            tensors["shared_up"] = tensor(p + "shared.up", (S, W), "matrix", ("normal", 0.0, W ** -0.5))
            tensors["shared_down"] = tensor(p + "shared.down", (W, S), "matrix", ("normal", 0.0, S ** -0.5))
        return PartSpec("feed_forward", "routed_table", params, tensors)

    def spec(self, tensor_names=None) -> ModelSpec:
        W, V = self.width, self.vocab
        names = set(tensor_names) if tensor_names is not None else set()

        def norm(name: str) -> PartSpec:
            return PartSpec("norm", "rms", {"width": W, "eps": self.eps}, {"weight": tensor(name, (W,), "vector", _NORM_INIT)})

        layers, order = [], []
        for i, layer in enumerate(self.layers):
            p, m = f"l{i}.", layer["mixer"]
            mixer = self._attention(p + "mix.", m) if layer["type"] == "attention" else self._latent(i, p + "mix.", m)
            parts, spare = {"mixer_norm": norm(p + "norm1"), "mixer": mixer}, {}
            if layer["mlp"] is not None:
                parts["feed_forward_norm"] = norm(p + "norm2")
                parts["feed_forward"] = self._feed_forward(p + "mlp.", layer["mlp"])
            elif p + "norm2" in names:
                # a checkpoint that holds the second norm of a layer without a feed-forward: bound, and not used
                spare = {"spare_norm2": tensor(p + "norm2", (W,), "vector", _NORM_INIT)}
            layers.append(PartSpec("block", "pre_norm", {}, spare, parts))
            order.append(LayerCall(i, cache_of=m.get("kv_from")))

        return ModelSpec(
            architecture=self.architecture, vocab_size=V, hidden_size=W, max_positions=None,
            embedding=PartSpec("embedding", "token_table", {"vocab_size": V, "hidden_size": W}, {"table": tensor("embed", (V, W), "table", ("normal", 0.0, 1.0))}),
            layers=tuple(layers), order=tuple(order), final_norm=norm("final.norm"),
            head=PartSpec("head", "linear", {"vocab_size": V, "hidden_size": W}, {"weight": tensor("head", (V, W), "matrix", ("normal", 0.0, W ** -0.5))}),
            stop_token_ids=self.eos_token_ids)
