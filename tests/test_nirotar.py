"""The Nirotar design in the engine against the plain implementation (tests/plain_nirotar.py).

Without a GPU: the configuration, its description as parts, the run order and cache plan, tables of random models, the oracle's
own mechanisms against closed forms, and that a mistake planted in any mechanism of the oracle moves the logits far beyond what
the comparisons allow.  On the GPU: every mechanism alone (one-layer models, and the kernels called directly with inputs made so
that one far key, one key at a window's or a page's edge, or a sink decides the result), whole prompts, prompts cut into
portions down to two tokens, prefill against token-by-token decoding from the first token, batches of unequal requests against
each alone, slots and pages that are used again, long decoding over several pages and windows, a prompt longer than a step takes
at once, recorded against launched steps, and greedy generation through ``generate``, the command line and the trace replay.  In
float32 and in bfloat16.
"""
import json
import math

import pytest
import torch

import nirotar_tiny as S
import plain_nirotar as P
from palm_infra_amd.config import ConfigError, config_from_dict

gpu = pytest.mark.gpu
DTYPES = ("float32", "bfloat16")
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
LENGTHS = {"A": [1, 2, 63, 64, 65, 130, 200, 37], "B": [129, 3, 70, 71, 1, 191], "C": [300, 9, 140], "D": [5, 66, 128, 31], "E": [67, 1, 20]}


# ---- without a GPU ---------------------------------------------------------------------------------------

def test_registry_picks_the_design_by_its_config_key():
    cfg = config_from_dict(S.CONFIGS["A"])
    assert type(cfg).__name__ == "NirotarConfig"
    again = config_from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again.to_dict() == cfg.to_dict() and again.to_dict()["layers"] == S.CONFIGS["A"]["layers"]


def test_spec_names_every_tensor():
    spec = config_from_dict(S.CONFIGS["A"]).spec()
    names = spec.expected_tensors()
    assert names["embed"][0] == names["head"][0] == (211, 64) and names["final.norm"][0] == names["l0.norm1"][0] == names["l0.norm2"][0] == (64,)
    assert names["l0.mix.q"][0] == (144, 64) and names["l0.mix.k"][0] == (48, 64) and names["l0.mix.v"][0] == (80, 64)
    assert names["l0.mix.sink"] == ((6,), "vector") and names["l0.mix.o"][0] == (64, 240)
    assert names["l0.mlp.table"] == ((211, 3), "integer") and names["l0.mlp.e7.up"][0] == (24, 64) and names["l0.mlp.e0.down"][0] == (64, 24)
    assert names["l0.mlp.shared.up"][0] == (40, 64) and names["l0.mlp.shared.down"][0] == (64, 40)
    assert names["l1.mix.q"][0] == (120, 64) and names["l1.mix.dkv"][0] == (48, 64) and names["l1.mix.dkv.norm"][0] == (40,)
    assert names["l1.mix.uk"][0] == (80, 40) and names["l1.mix.uv"][0] == (120, 40) and names["l1.mix.sink"][0] == (5,)
    # a layer that reads another's latents makes none; a layer without a feed-forward has no tensors for it
    assert names["l3.mix.q"][0] == (96, 64) and names["l3.mix.uk"][0] == (72, 40) and names["l3.mix.uv"][0] == (120, 40)
    assert not any(n.startswith(("l3.mix.dkv", "l2.mlp", "l2.norm2", "l3.mlp.shared")) or n.endswith("router") for n in names)
    assert spec.layers[0].parts["mixer"].tensors["qkvg"].shape == (144 + 48 + 80, 64)
    assert spec.layers[1].parts["mixer"].tensors["down"].shape == (120 + 48, 64)


def test_second_norm_of_a_feed_forward_that_is_not_there_is_bound_if_the_file_has_it():
    cfg = config_from_dict(S.CONFIGS["A"])
    names = list(cfg.spec().expected_tensors())
    assert "l2.norm2" in cfg.spec(names + ["l2.norm2"]).expected_tensors() and "l2.norm2" not in cfg.spec(names).expected_tensors()


def test_run_order_and_cache_plan():
    from palm_infra_amd.cache import KVNeed, RowsNeed
    from palm_infra_amd.parts import cache_needs, cache_needs_beside_shared
    spec = config_from_dict(S.CONFIGS["A"]).spec()
    assert [(c.layer, c.cache_of) for c in spec.order] == [(0, None), (1, None), (2, None), (3, 1)]
    assert cache_needs(spec.layers[0]) == [KVNeed(2, 24, 37, value_dim=40)]
    assert cache_needs(spec.layers[1]) == [RowsNeed("latent", (48,), None, None), RowsNeed("latent_t", (40,), "bfloat16", None)]
    assert cache_needs(spec.layers[2]) == [KVNeed(3, 40, 70, value_dim=24)]
    assert cache_needs_beside_shared(spec.layers[3]) == []
    with pytest.raises(ValueError, match="another entry"):
        cache_needs(spec.layers[3])
    b = config_from_dict(S.CONFIGS["B"]).spec()
    assert [c.cache_of for c in b.order] == [None, 0, None, 0]
    assert cache_needs(b.layers[2]) == [KVNeed(1, 40, None, value_dim=72)]


@pytest.mark.parametrize("change,what", [
    (lambda c: c["layers"][0].update(type="retention"), "type"),
    (lambda c: c["layers"][0].pop("mixer"), "mixer"),
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=4), "kv heads"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"].update(dim=300), "key and value sizes"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=26), "rot.dims"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=7), "even"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].pop("low"), "low"),
    (lambda c: c["layers"][0]["mixer"]["rot"]["scaling"].update(high=1.0), "high"),
    (lambda c: c["layers"][1]["mixer"].pop("rot"), "dims"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=4), "whole rotated part"),
    (lambda c: c["layers"][1]["mixer"].update(kv_rank=2000), "latents"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=0), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_from=3), "kv_from"),
    (lambda c: c["layers"][3]["mixer"].update(kv_rank=48), "another kv_rank"),
    (lambda c: c["layers"][3]["mixer"]["rot"].update(base=7.0), "rotation"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"].pop("expert"), "ff"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "experts"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_bad_configurations_are_refused(change, what):
    raw = json.loads(json.dumps(S.CONFIGS["A"]))
    change(raw)
    with pytest.raises(ConfigError, match=what):
        config_from_dict(raw)


def test_random_model_folder_is_read_by_the_plain_implementation(tmp_path):
    from palm_infra_amd.weights import write_random_model
    write_random_model(S.CONFIGS["D"], 3, tmp_path, "bfloat16")
    cfg, w = P.read_model(tmp_path)
    layers = []
    logits = P.forward(cfg, w, [1, 2, 3, 4, 5], layers)
    assert logits.shape == (5, 97) and torch.isfinite(logits).all() and len(layers) == 3
    assert w["l0.mlp.table"].dtype == torch.int32


@pytest.mark.parametrize("count,n", [(1, 7), (3, 3), (4, 9), (2, 2), (6, 64)])
def test_random_tables_hold_different_entries_of_every_expert(count, n):
    from palm_infra_amd.weights.random_numbers import distinct_rows, tensor_key
    rows = distinct_rows(tensor_key(5, "table"), 900, count, n)
    assert rows.shape == (900, count) and all(len(set(r)) == count for r in rows.tolist())
    share = torch.bincount(torch.from_numpy(rows).long().reshape(-1), minlength=n).double() / (900 * count)
    assert share.shape == (n,) and float((share * n - 1).abs().max()) < 0.6
    assert (distinct_rows(tensor_key(5, "table"), 12, count, n) == rows[:12]).all()


def test_plain_frequencies_in_their_three_bands():
    """dims 4, base 16: frequencies 1 and 1/4, wavelengths 6.28 and 25.1."""
    rot = lambda low, high, original: {"dims": 4, "base": 16.0, "scaling": {"factor": 5.0, "low": low, "high": high, "original": original}}
    assert torch.allclose(P.frequencies({"dims": 4, "base": 16.0}), torch.tensor([1.0, 0.25], dtype=P.F64))
    assert torch.allclose(P.frequencies(rot(1.0, 2.0, 100)), torch.tensor([1.0, 0.25], dtype=P.F64))          # both below 50
    assert torch.allclose(P.frequencies(rot(1.0, 2.0, 4)), torch.tensor([0.2, 0.05], dtype=P.F64))            # both above 4
    s = (40 / (8 * math.pi) - 1.0) / (4.0 - 1.0)                                                              # 25.1 between 10 and 40
    assert torch.allclose(P.frequencies(rot(1.0, 4.0, 40)), torch.tensor([1.0, (1 - s) * 0.05 + s * 0.25], dtype=P.F64))
    x = torch.zeros(3, 1, 5, dtype=P.F64)
    x[:, 0, 0], x[:, 0, 4] = 1.0, 9.0
    y = P.rotate_pairs(x, {"dims": 4, "base": 16.0})
    assert torch.allclose(y[2, 0], torch.tensor([math.cos(2.0), math.sin(2.0), 0.0, 0.0, 9.0], dtype=P.F64))


def test_the_position_part_makes_the_same_frequencies():
    from palm_infra_amd.config.spec import PartSpec
    from palm_infra_amd.parts import Builder
    for dims, base, sc in [(16, 500.0, (4.0, 1.0, 4.0, 256)), (40, 1e4, None), (32, 20.0, (8.0, 1.0, 2.0, 64)), (48, 3e5, (8.0, 1.0, 4.0, 8192))]:
        rot = S.rotation(dims, base, sc)
        scaling = dict(rot["scaling"], kind="wavelength") if sc else None
        part = Builder(None, torch.float32, "cpu").build(PartSpec("position", "rotary", {"rotary_dim": dims, "theta": base, "pairing": "interleaved",
                                                                                         "scaling": scaling, "exact_frequencies": True}))
        assert torch.equal(part.inv_freq, P.frequencies(rot).float()) and part.magnitude == 1.0


def test_plain_sink_takes_weight_and_gives_nothing_and_the_window_ends():
    T = 7
    scores = torch.zeros(2, T, T, dtype=P.F64)
    p = P.sink_softmax_heads(scores, torch.tensor([math.log(2.0), -40.0], dtype=P.F64), 3)
    for i in range(T):
        seen = min(i + 1, 3)
        assert torch.allclose(p[0, i, max(0, i - 2):i + 1], torch.full((seen,), 1.0 / (seen + 2), dtype=P.F64))
        assert float(p[0, i].sum()) == pytest.approx(seen / (seen + 2)) and float(p[1, i].sum()) == pytest.approx(1.0)


def test_plain_latent_attention_equals_its_absorbed_form():
    """Scores through U_k^T q against the latents, and U_v applied to the weighted latents, give the same outputs."""
    torch.manual_seed(3)
    raw = S.SINGLE["latent"]
    m, w = raw["layers"][0]["mixer"], {k: t.to(P.F64) for k, t in S.tensors_of(raw, 7, "float32").items()}
    T, H, d, dr, dv, R = 12, m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
    h = torch.randn(T, raw["width"], dtype=P.F64)
    want = P.latent_mixer(h, w, "l0.mix.", m, 1e-6, {})
    c, r = P.latent_rows(h, w, "l0.mix.", m, 1e-6)
    q = (h @ w["l0.mix.q"].T).reshape(T, H, d + dr)
    a = torch.stack([q[:, x, :d] @ w["l0.mix.uk"].reshape(H, d, R)[x] for x in range(H)])
    scores = (a @ c.T + P.rotate_pairs(q[..., d:], m["rot"]).transpose(0, 1) @ r.T) * m["scale"]
    p = P.sink_softmax_heads(scores, w["l0.mix.sink"], None)
    o = torch.stack([(p[x] @ c) @ w["l0.mix.uv"].reshape(H, dv, R)[x].T for x in range(H)], 1)
    assert torch.allclose(o.reshape(T, -1) @ w["l0.mix.o"].T, want)


def test_plain_table_experts():
    w = {"table": torch.tensor([[1, 0], [2, 1], [0, 2]]), "shared.up": torch.tensor([[1.0]], dtype=P.F64), "shared.down": torch.tensor([[100.0]], dtype=P.F64)}
    for e, (u, d) in enumerate([(1.0, 1.0), (-1.0, 10.0), (2.0, 1000.0)]):
        w[f"e{e}.up"], w[f"e{e}.down"] = torch.tensor([[u]], dtype=P.F64), torch.tensor([[d]], dtype=P.F64)
    h = torch.tensor([[3.0], [-2.0], [1.0]], dtype=P.F64)
    got = P.table_experts(h, [2, 1, 0], w, "", {"router": {"experts": 3, "top": 2}, "shared": {"ff": 1}})
    assert got[:, 0].tolist() == [(9 + 36000) / 2 + 900.0, (0 + 40) / 2 + 0.0, (0 + 1) / 2 + 100.0]


# A mistake in any mechanism must show: each of these, planted in the oracle, moves some logits by more than twenty times what a
# float32 comparison allows.
def _plant(monkeypatch, what):
    soft, rotate, freq, rows, experts = P.sink_softmax_heads, P.rotate_pairs, P.frequencies, P.latent_rows, P.table_experts
    if what == "window one longer":
        monkeypatch.setattr(P, "sink_softmax_heads", lambda s, z, w: soft(s, z, w and w + 1))
    elif what == "window one shorter":
        monkeypatch.setattr(P, "sink_softmax_heads", lambda s, z, w: soft(s, z, w and w - 1))
    elif what == "no sink":
        monkeypatch.setattr(P, "sink_softmax_heads", lambda s, z, w: soft(s, z * 0 - 1e9, w))
    elif what == "scaled sink":
        monkeypatch.setattr(P, "sink_softmax_heads", lambda s, z, w: soft(s, z * 0.2, w))
    elif what == "halves":
        def halves(x, rot):
            n = rot["dims"]
            order = torch.tensor([i // 2 + (i % 2) * (n // 2) for i in range(n)] + list(range(n, x.shape[-1])))
            y = torch.empty_like(x)
            y[..., order] = rotate(x[..., order], rot)
            return y
        monkeypatch.setattr(P, "rotate_pairs", halves)
    elif what == "plain frequencies":
        monkeypatch.setattr(P, "frequencies", lambda rot: freq({k: rot[k] for k in ("dims", "base")}))
    elif what == "all stretched":
        monkeypatch.setattr(P, "frequencies", lambda rot: freq({k: rot[k] for k in ("dims", "base")}) / (rot["scaling"]["factor"] if rot.get("scaling") else 1.0))
    elif what == "positions from one":
        monkeypatch.setattr(P, "frequencies", freq)
        def late(h, w, p, m, eps):
            c, r = rows(torch.cat([h[:1], h]), w, p, m, eps)
            return c[1:], r[1:]
        monkeypatch.setattr(P, "latent_rows", late)                     # the keys turn by one position more than the queries
    elif what == "latent not normed":
        monkeypatch.setattr(P, "latent_rows", lambda h, w, p, m, eps: ((h @ w[p + "dkv"].T)[:, :m["kv_rank"]] * w[p + "dkv.norm"], rows(h, w, p, m, eps)[1]))
    elif what == "wrong shelf":
        latent = P.latent_mixer
        def fresh(h, w, p, m, eps, shelf):
            if m.get("kv_from") is None:
                return latent(h, w, p, m, eps, shelf)
            j = f"l{m['kv_from']}.mix."
            return latent(h, w, p, m, eps, {j: P.latent_rows(h, w, j, m, eps)})      # the other layer's matrix on this layer's input
        monkeypatch.setitem(P.MIXERS, "latent_attention", fresh)
    elif what == "next token's experts":
        monkeypatch.setattr(P, "table_experts", lambda h, ids, w, p, f: experts(h, list(ids[1:]) + [ids[0]], w, p, f))
    elif what == "weights of one":
        monkeypatch.setattr(P, "table_experts", lambda h, ids, w, p, f: experts(h, ids, w, p, f) + (f["router"]["top"] - 1) * experts(h, ids, w, p, {k: f[k] for k in ("router",)}))
    elif what == "no shared expert":
        monkeypatch.setattr(P, "table_experts", lambda h, ids, w, p, f: experts(h, ids, w, p, {k: f[k] for k in ("router",)}))
    elif what == "relu":
        monkeypatch.setattr(P, "squared_relu_expert", lambda h, w, p: torch.clamp(h @ w[p + "up"].T, min=0.0) @ w[p + "down"].T)
    elif what == "eps outside":
        monkeypatch.setattr(P, "rms_norm", lambda x, w, eps: x / (torch.sqrt((x * x).mean(-1, keepdim=True)) + 40 * math.sqrt(eps)) * w)
    else:
        raise KeyError(what)


@pytest.mark.parametrize("what", ["window one longer", "window one shorter", "no sink", "scaled sink", "halves", "plain frequencies", "all stretched",
                                  "positions from one", "latent not normed", "wrong shelf", "next token's experts", "weights of one",
                                  "no shared expert", "relu", "eps outside"])
def test_a_planted_mistake_shows(monkeypatch, what):
    raw = S.CONFIGS["A"]
    w = S.tensors_of(raw, S.SEEDS["A"], "float32")
    ids = S.prompts(raw, [90], seed=3)[0]
    right = P.forward(raw, w, ids)
    _plant(monkeypatch, what)
    wrong = P.forward(raw, w, ids)
    scale = float(right.pow(2).mean().sqrt())
    assert float((wrong - right).abs().max()) > 20 * 1e-4 * max(1.0, scale), what


# ---- on the GPU ------------------------------------------------------------------------------------------

_dirs, _engines, _refs = {}, {}, {}


def raw_of(name: str) -> dict:
    return S.CONFIGS.get(name) or S.SINGLE[name]


def model_dir(tmp_path_factory, name: str, store: str):
    key = (name, store)
    if key not in _dirs:
        _dirs[key] = S.write_model(raw_of(name), S.SEEDS.get(name, 101), tmp_path_factory.mktemp(f"nirotar_{name}_{store}"), store)
    return _dirs[key]


def engine_for(tmp_path_factory, name: str, dtype: str, **options):
    from palm_infra_amd.engine import Engine
    key = (name, dtype, tuple(sorted(options.items())))
    if key not in _engines:
        _engines[key] = Engine.from_dir(model_dir(tmp_path_factory, name, dtype), dtype=dtype, max_tokens=64 * 24, **options)
    return _engines[key]


def reference(tmp_path_factory, name: str, dtype: str, ids):
    key = (name, dtype, tuple(ids))
    if key not in _refs:
        cfg, w = P.read_model(model_dir(tmp_path_factory, name, dtype))
        _refs[key] = P.forward(cfg, w, ids)
    return _refs[key]


def assert_close(got, ref, dtype: str, what: str = "") -> None:
    """float32: 1e-4 of the logits' scale, the gate that shows faults.  bfloat16: every row's root mean square error within a
    twentieth of the logits' scale, half of the rows within a fiftieth."""
    got = torch.as_tensor(got).double().cpu().reshape(ref.shape)
    assert torch.isfinite(got).all(), f"{what}: logits are not finite"
    err = (got - ref.double()).abs().reshape(-1, ref.shape[-1])
    scale = float(ref.double().pow(2).mean().sqrt())
    if dtype == "float32":
        worst = float(err.max())
        assert worst <= 1e-4 * max(1.0, scale), f"{what}: float32 logits differ by {worst:.3e} (their scale is {scale:.3e})"
        return
    rows = err.pow(2).mean(-1).sqrt()
    worst, middle = float(rows.max()), float(rows.median())
    assert worst <= 0.05 * scale, f"{what}: bfloat16 rms error {worst:.3e} of a row vs {scale:.3e}"
    assert rows.numel() < 8 or middle <= 0.02 * scale, f"{what}: bfloat16 median rms error {middle:.3e} vs {scale:.3e}"


CASES = [(n, d) for n in ("A", "B", "C", "D", "E") for d in DTYPES]


def _step_context(lengths_before, new_counts, slots=None, ids=None):
    """A cache-less context for kernels that only need the packed layout."""
    from palm_infra_amd.parts import make_context
    slots = list(range(len(new_counts))) if slots is None else list(slots)
    tokens = [[0] * c for c in new_counts] if ids is None else ids
    return make_context(slots, list(lengths_before), tokens, torch.float32, "cuda")


# ---- every mechanism alone -------------------------------------------------------------------------------

@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", sorted(S.SINGLE))
def test_one_layer_of_one_kind(tmp_path_factory, kind, dtype):
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, kind, dtype)
    ids = S.prompts(raw_of(kind), [120], seed=1)[0]
    ref = reference(tmp_path_factory, kind, dtype, ids)
    slot = eng.open()
    got = [eng.step([StepEntry(slot, ids[:100], list(range(100)))])] + [eng.step([StepEntry(slot, [t], [0])]) for t in ids[100:]]
    eng.close(slot)
    assert_close(torch.cat(got), ref, dtype, kind)


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,window", [(4, 2, 24, 40, 37), (3, 3, 40, 72, 70), (6, 1, 16, 12, None), (16, 2, 64, 32, 130), (4, 2, 96, 56, 64)])
def test_attention_far_keys_page_borders_window_edges_and_sinks(dtype, H, G, d, dv, window):
    """Keys and values straight into the pages.  One key is made to stand out at places that matter: the first positions, far
    back, a page's last and first key, just inside and just outside the window, the query's own; one head's sink outweighs
    every key, one's is absent in all but name.  Prompts (the matrix cores in bfloat16), portions, and single tokens in slices."""
    from palm_infra_amd.kernels import ops
    torch.manual_seed(H * 100 + d)
    dt = TORCH[dtype]
    T, scale, per = 300, 0.3, H // G
    pages = [3, 0, 5, 2, 4]
    table = torch.tensor([[6] * 5, pages], dtype=torch.int32, device="cuda")
    sinks = torch.randn(H)
    sinks[H - 1], sinks[0] = 60.0, -50.0
    targets = [0, 1, 63, 64, 127, 128, T - (window or 200), T - 1 - (window or 200), T - 1]
    for target in sorted(set(t for t in targets if 0 <= t < T)):
        k, v, q = torch.randn(T, G, d) * 0.3, torch.randn(T, G, dv), torch.randn(T, H, d) * 0.3
        k[target] = torch.nn.functional.normalize(torch.randn(G, d), dim=-1) * 4.0
        for h in range(H):
            q[T - 1, h] = k[target, h // per] / 16.0 * 40.0 / scale
        q, k, v = (t.to(dt) for t in (q, k, v))
        kc, vc = torch.full((7, G, 64, d), float("nan"), dtype=dt), torch.full((7, G, dv, 64), float("nan"), dtype=dt)
        for p in range(T):
            kc[pages[p // 64], :, p % 64] = k[p]
            vc[pages[p // 64], :, :, p % 64] = v[p]
        vc[pages[T // 64], :, :, T % 64:] = 0
        kc[pages[T // 64], :, T % 64:] = 0
        scores = torch.stack([q.double()[:, h] @ k.double()[:, h // per].T * scale for h in range(H)])
        pr = P.sink_softmax_heads(scores, sinks.double(), window)
        want = torch.stack([pr[h] @ v.double()[:, h // per] for h in range(H)], 1)
        tol = dict(atol=2e-4, rtol=2e-4) if dtype == "float32" else dict(atol=3e-2, rtol=3e-2)
        run = lambda fn, a, b, **kw: fn(q[a:b].cuda(), kc.cuda(), vc.cuda(), table, _step_context([a], [b - a], slots=[1]), H, G, d, dv, scale, window,
                                        sinks.cuda(), None, **kw).cpu().double().reshape(b - a, H, dv)
        for cuts in ((0, T), (0, 170, T), (0, 2, 66, T)):
            got = torch.cat([run(ops.sink_attention, a, b) for a, b in zip(cuts, cuts[1:])])
            assert torch.allclose(got, want, **tol), (target, cuts)
        for slices in (None, 1, 3):
            assert torch.allclose(run(ops.sink_attention_exact, T - 1, T, slices=slices)[0], want[T - 1], **tol), (target, slices)
        seen = window is None or T - 1 - target < window
        assert bool((want[T - 1, 0] - v[target, 0].double()).abs().max() < 0.05) == seen, target
        assert float(want[T - 1, H - 1].abs().max()) < 1e-3


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("heads,R,dr,window", [(3, 40, 8, None), (17, 96, 16, None), (5, 33, 2, 40), (2, 200, 32, 64), (16, 256, 32, 129), (1, 512, 64, None), (20, 24, 16, 70)])
def test_latent_attention_far_keys_page_borders_window_edges_and_sinks(dtype, heads, R, dr, window):
    """Two sequences through pages in a scrambled order, NaN wherever a page belongs to nobody: a prompt portion, and single
    tokens in one and several slices.  For chosen queries one row carries a large score: the first positions, either side of a
    page border, the last row inside a window and the first outside it, the query's own; the row after a query is larger still
    and must stay unseen.  One head's sink outweighs every row."""
    from palm_infra_amd.kernels import ops
    td = TORCH[dtype]
    g = torch.Generator().manual_seed(R + dr)
    lens, scale, dk, dv = [330, 200], 0.7, R + dr, 12
    sinks = torch.randn(heads, generator=g)
    if heads > 1:
        sinks[heads - 1] = 80.0
    uv = (torch.randn(heads * dv, R, generator=g) * 0.2).to(td)
    pages_of, pages_t = [[7, 6, 5, 4, 3, 2], [9, 12, 8, 10]], [[3, 11, 0, 5, 7, 1], [2, 4, 12, 6]]
    w = window or 10 ** 9
    for counts in ([70, 2], [1, 1]):
        starts = [ln - c for ln, c in zip(lens, counts)]
        for offset in ((0,) if counts[0] > 1 else (0, 1, "border", "own", "inside", "outside")):
            rows = [(torch.randn(ln + 1, dk, generator=g) * 0.3).to(td) for ln in lens]        # one row beyond each length: never seen
            n = sum(counts)
            qa = torch.randn(n, heads, dk, generator=g) * 0.3
            marks = []
            for b, (s, c) in enumerate(zip(starts, counts)):
                pos = s + c - 1
                if counts[0] == 1:
                    marks.append((b, pos, {0: 0, 1: 1, "border": 128, "own": pos, "inside": max(0, pos - w + 1), "outside": max(0, pos - w)}[offset]))
                elif b == 0:
                    marks += [(b, pos, max(0, pos - w + 1)), (b, s + 3, max(0, s + 3 - w)), (b, s + 10, (s + 10) // 64 * 64 - 1),
                              (b, s + 20, (s + 20) // 64 * 64), (b, s + 30, s + 30), (b, s + 40, 0), (b, s + 45, 1)]
            for b, pos, key in marks:
                direction = torch.nn.functional.normalize(torch.randn(dk, generator=g), dim=0)
                qa[sum(counts[:b]) + pos - starts[b]] = direction * 6.0
                rows[b][key] = (direction * 6.0).to(td)
                rows[b][pos + 1] = (direction * 12.0).to(td)
            want, o = [], 0
            for b, (s, c) in enumerate(zip(starts, counts)):
                r = rows[b][:-1].double()
                for i in range(c):
                    full = torch.full((heads, lens[b], lens[b]), 0.0, dtype=P.F64)
                    full[:, s + i] = qa[o + i].double() @ r.T * scale
                    want.append(P.sink_softmax_heads(full, sinks.double(), window)[:, s + i] @ r[:, :R])
                o += c
            want = torch.stack(want)
            cache, turned = torch.full((14, 64, dk), float("nan"), dtype=td), torch.full((14, R, 64), float("nan"), dtype=torch.bfloat16)
            table, table_t = torch.full((3, 8), 13, dtype=torch.int32), torch.full((3, 8), 13, dtype=torch.int32)
            for b in range(2):
                table[b + 1, :len(pages_of[b])] = torch.tensor(pages_of[b], dtype=torch.int32)
                table_t[b + 1, :len(pages_t[b])] = torch.tensor(pages_t[b], dtype=torch.int32)
                for j in range(lens[b] + 1):
                    cache[pages_of[b][j // 64], j % 64] = rows[b][j]
                    if j < lens[b]:
                        turned[pages_t[b][j // 64], :, j % 64] = rows[b][j, :R].bfloat16()
            cache, turned, table, table_t = cache.cuda(), turned.cuda(), table.cuda(), table_t.cuda()
            ctx = _step_context(starts, counts, slots=[1, 2])
            args = (qa.cuda(), cache, table, ctx, heads, R, dr, scale, window)
            got = ops.latent_attention(*args, sink=sinks.cuda()).double().cpu()
            tol = dict(atol=1e-4, rtol=1e-3) if dtype == "float32" else dict(atol=2e-2, rtol=2e-2)
            assert torch.isfinite(got).all() and torch.allclose(got, want, **tol), (counts, offset, float((got - want).abs().max()))
            if heads > 1:
                assert float(want[:, heads - 1].abs().max()) < 1e-2
            if dtype != "bfloat16" or not ops.latent_mfma_serves(cache, R, dr):
                continue
            out = torch.stack([want[:, h] @ uv.double().reshape(heads, dv, R)[h].T for h in range(heads)], 1).reshape(n, heads * dv)
            if ctx.is_decode:
                for slices in (None, 1, 2, 4, 50):
                    fast = ops.latent_attention_decode(*args, turned, table_t, uv.cuda(), None, dv, sink=sinks.cuda(), slices=slices).double().cpu()
                    assert torch.isfinite(fast).all() and torch.allclose(fast, out, atol=4e-2, rtol=4e-2), (offset, slices, float((fast - out).abs().max()))
                gate = torch.randn(n, heads + 3, generator=g).to(td)
                fast = ops.latent_attention_decode(*args, turned, table_t, uv.cuda(), gate.cuda()[:, 3:], dv, sink=sinks.cuda()).double().cpu()
                gated = out.reshape(n, heads, dv) * torch.sigmoid(gate.double()[:, 3:, None])
                assert torch.allclose(fast, gated.reshape(n, -1), atol=4e-2, rtol=4e-2)
                plain = ops.latent_attention_decode(*args, turned, table_t, uv.cuda(), None, dv).double().cpu()
                exact = ops.latent_output(ops.latent_attention(*args), uv.cuda(), None, heads, R, dv, torch.bfloat16).double().cpu()
                assert torch.allclose(plain, exact, atol=4e-2, rtol=4e-2)
            else:
                fast = ops.latent_attention(*args, rows_t=turned, table_t=table_t, sink=sinks.cuda()).double().cpu()
                assert torch.isfinite(fast).all() and torch.allclose(fast, want, atol=3e-2, rtol=3e-2), float((fast - want).abs().max())
                fast = ops.latent_attention_fused(*args, turned, table_t, uv.cuda(), None, dv, sink=sinks.cuda()).double().cpu()
                assert torch.isfinite(fast).all() and torch.allclose(fast, out, atol=4e-2, rtol=4e-2), float((fast - out).abs().max())


@gpu
@pytest.mark.parametrize("heads,d,dr,dv,R,window", [(3, 16, 8, 24, 64, None), (5, 64, 32, 128, 256, None), (2, 32, 16, 40, 96, 70), (1, 128, 64, 128, 512, None), (4, 24, 8, 72, 136, 64)])
def test_latent_attention_with_expanded_keys_and_values(heads, d, dr, dv, R, window):
    """A prompt's portions of three sequences (one from its start, two further on) over cached rows in scrambled pages, NaN wherever
    a page belongs to nobody; the queries come unrotated as columns of a wider product.  For chosen queries one position's key
    stands out: the first ones, a page's borders, a window's edges, the query's own.  One head's sink outweighs every key."""
    from palm_infra_amd.kernels import ops
    g = torch.Generator().manual_seed(R + d)
    bf, dk, scale = torch.bfloat16, R + dr, 0.4
    lens, counts = [330, 100, 290], [150, 100, 70]
    starts = [ln - c for ln, c in zip(lens, counts)]
    n = sum(counts)
    sinks = torch.randn(heads, generator=g)
    if heads > 1:
        sinks[heads - 1] = 90.0
    uk, uv = (torch.randn(heads * d, R, generator=g) * R ** -0.5).to(bf), (torch.randn(heads * dv, R, generator=g) * R ** -0.5).to(bf)
    rot = {"dims": dr, "base": 40.0}
    q = torch.randn(n, heads * (d + dr) + 24, generator=g) * 0.3
    rows = [(torch.randn(ln, dk, generator=g) * 0.5).to(bf) for ln in lens]
    w = window or 10 ** 9
    at = 0
    for b, (s, c) in enumerate(zip(starts, counts)):
        for i in range(0, c, 9):
            pos = s + i
            key = [0, 1, pos // 64 * 64 - 1, pos // 64 * 64, max(0, pos - w + 1), pos - w, pos][i // 9 % 7]
            if 0 <= key <= pos:
                r = rows[b][key].double()
                for h in range(heads):                              # the query points along that position's unrotated key
                    k = uk[h * d:(h + 1) * d].double() @ r[:R]
                    q[at + i, h * (d + dr):h * (d + dr) + d] = (k / k.norm() ** 2 * 30.0 / scale).float()
        at += c
    q = q.to(bf)
    pages_of = [[7, 6, 5, 4, 3, 2], [9, 12], [8, 10, 0, 13, 11]]
    cache = torch.full((16, 64, dk), float("nan"), dtype=bf)
    table = torch.full((4, 8), 15, dtype=torch.int32)
    for b in range(3):
        table[b + 1, :len(pages_of[b])] = torch.tensor(pages_of[b], dtype=torch.int32)
        for j in range(lens[b]):
            if window is None or j // 64 >= max(0, starts[b] - window + 1) // 64:              # (pages that no query sees may be gone)
                cache[pages_of[b][j // 64], j % 64] = rows[b][j]
    ctx = _step_context(starts, counts, slots=[1, 2, 3])
    ang = ctx.positions.cpu().double()[:, None] * P.frequencies(rot)
    cos, sin = torch.cos(ang).float().cuda(), torch.sin(ang).float().cuda()
    gate = torch.randn(n, heads + 5, generator=g).to(bf)
    want, at = [], 0
    for b, (s, c) in enumerate(zip(starts, counts)):
        r = rows[b].double()
        qs = torch.zeros(lens[b], heads, d + dr, dtype=P.F64)
        qs[s:] = q[at:at + c, :heads * (d + dr)].double().reshape(c, heads, d + dr)
        qt = P.rotate_pairs(qs[..., d:], rot)
        kp, v = (r[:, :R] @ uk.double().T).reshape(-1, heads, d), (r[:, :R] @ uv.double().T).reshape(-1, heads, dv)
        scores = torch.stack([(qs[:, h, :d] @ kp[:, h].T + qt[:, h] @ r[:, R:].T) * scale for h in range(heads)])
        p = P.sink_softmax_heads(scores, sinks.double(), window)
        want.append(torch.stack([p[h] @ v[:, h] for h in range(heads)], 1)[s:])
        at += c
    want = torch.cat(want)
    qc = q.cuda()[:, :heads * (d + dr)]
    serves = ops.latent_expanded_serves(qc, cache.cuda(), uk.cuda(), uv.cuda(), ctx, heads, d, dr, R, dv, window)
    assert serves or R < 100                                          # (a small latent: it may not pay, which the next line overrides)
    plan, ops.latent_expand_plan = ops.latent_expand_plan, lambda ctx, window: (64, 1e12)
    try:
        args = (qc, uk.cuda(), uv.cuda(), cos, sin, heads, d, dr, R, dv, "interleaved", ctx, None, cache.cuda(), table.cuda(), scale, window, sinks.cuda())
        got = ops.latent_attention_expanded(*args, None).double().cpu().reshape(n, heads, dv)
        assert torch.isfinite(got).all()
        assert torch.allclose(got, want, atol=4e-2, rtol=4e-2), float((got - want).abs().max())
        gated = ops.latent_attention_expanded(*args, gate.cuda()[:, 5:]).double().cpu().reshape(n, heads, dv)
        assert torch.allclose(gated, want * torch.sigmoid(gate.double()[:, 5:, None]), atol=4e-2, rtol=4e-2)
    finally:
        ops.latent_expand_plan = plan
    if heads > 1:
        assert float(want[:, heads - 1].abs().max()) < 1e-2


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dr,R", [(3, 12, 6, 24), (1, 40, 2, 70), (20, 16, 8, 136), (3, 72, 24, 56)])
def test_direct_queries_through_the_key_matrix_and_cache_rows_in_one_launch(dtype, H, d, dr, R):
    """Queries as columns of a wider product, neighbouring pairs turned, the latent normed and written to its page and to the
    transposed copy's page; a part that reads another's rows writes none."""
    from palm_infra_amd.kernels import ops
    td = TORCH[dtype]
    tol = dict(atol=1e-4, rtol=1e-4) if dtype == "float32" else dict(atol=0.06, rtol=0.02)
    g = torch.Generator().manual_seed(R)
    n, q_size = 11, H * (d + dr)
    ctx = _step_context([60, 0], [8, 3], slots=[0, 1])
    assert (ops.latent_key_transposes(torch.zeros(H * d, R, dtype=td), H, d, R) is not None) == (dtype == "bfloat16" and d % 8 == R % 8 == 0)
    down = torch.randn(n, q_size + R + dr, generator=g).to(td)
    wk = 1 + 0.2 * torch.randn(R, generator=g)
    uk = (torch.randn(H * d, R, generator=g) * 0.3).to(td)
    rot = {"dims": dr, "base": 50.0}
    pos = ctx.positions.cpu().double()
    ang = pos[:, None] * P.frequencies(rot)
    cos, sin = torch.cos(ang).float().cuda(), torch.sin(ang).float().cuda()

    def turn(x):                                                    # rows at the positions of this step
        long = torch.zeros((int(pos.max()) + 1,) + tuple(x.shape[1:]), dtype=P.F64)
        out = torch.empty_like(x)
        for i, p in enumerate(pos.long().tolist()):
            long[p] = x[i]
            out[i] = P.rotate_pairs(long, rot)[p]
        return out
    table = torch.tensor([[2, 1], [0, 3], [3, 3]], dtype=torch.int32, device="cuda")
    table_t = torch.tensor([[1, 3], [2, 0], [3, 3]], dtype=torch.int32, device="cuda")
    dd, dc = down.double(), down.cuda()
    q = dd[:, :q_size].reshape(n, H, d + dr)
    want_qa = torch.cat([torch.stack([q[:, h, :d] @ uk.double().reshape(H, d, R)[h] for h in range(H)], 1), turn(q[..., d:])], -1)
    want_rows = torch.cat([P.rms_norm(dd[:, q_size:q_size + R], wk.double(), 1e-5), turn(dd[:, None, q_size + R:])[:, 0]], 1)
    for writes in (True, False):
        cache = torch.zeros((4, 64, R + dr), dtype=td, device="cuda")
        turned = torch.zeros((4, R, 64), dtype=torch.bfloat16, device="cuda")
        store = ops.LatentStore(dc[:, q_size:], wk.cuda(), 1e-5, cache, table, turned, table_t) if writes else None
        qa = ops.latent_query(dc[:, :q_size], uk.cuda(), cos, sin, H, d, dr, R, pairing="interleaved", ctx=ctx, store=store,
                              uk_t=ops.latent_key_transposes(uk.cuda(), H, d, R)).double().cpu()
        assert torch.allclose(qa, want_qa, **tol)
        plain = ops.latent_query(dc[:, :q_size], uk.cuda(), cos, sin, H, d, dr, R, pairing="interleaved").double().cpu()
        assert torch.allclose(plain, want_qa, **tol)
        where = [(1, 60 + i - 64) if 60 + i >= 64 else (2, 60 + i) for i in range(8)] + [(0, i) for i in range(3)]
        where_t = [(3, 60 + i - 64) if 60 + i >= 64 else (1, 60 + i) for i in range(8)] + [(2, i) for i in range(3)]
        if not writes:
            assert not cache.any() and not turned.any()
            continue
        assert torch.allclose(torch.stack([cache[p, j] for p, j in where]).double().cpu(), want_rows, **tol)
        assert torch.allclose(torch.stack([turned[p, :, j] for p, j in where_t]).double().cpu(), want_rows[:, :R], atol=0.03, rtol=0.02)
        assert int((cache.abs().sum(-1) > 0).sum()) == n and int((turned.abs().sum(1) > 0).sum()) == n       # and nothing else was written


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("E,top,W,F,shared", [(6, 2, 48, 24, 40), (5, 1, 64, 32, 32), (4, 4, 40, 16, None), (9, 5, 50, 7, 11), (33, 3, 72, 40, 8), (7, 2, 264, 136, 64)])
def test_table_experts_for_few_rows_and_many(dtype, E, top, W, F, shared):
    """The part alone, with the step's token ids choosing: one row, a few (the shared expert rides along), a decode batch's
    and a prompt's; also when all tokens choose the same experts and when an expert is chosen by nobody."""
    from palm_infra_amd.kernels import ops
    from palm_infra_amd.parts.feedforward import RoutedTableFeedForward
    from palm_infra_amd.config.spec import PartSpec, tensor
    g = torch.Generator().manual_seed(E + F)
    dt, V = TORCH[dtype], 37
    t = {"up": (torch.randn(E * F, W, generator=g) * W ** -0.5).to(dt), "down": (torch.randn(E * W, F, generator=g) * F ** -0.5).to(dt),
         "table": torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(V)]).to(torch.int32)}
    w = {"table": t["table"]}
    for e in range(E):
        w[f"e{e}.up"], w[f"e{e}.down"] = t["up"][e * F:(e + 1) * F].double(), t["down"][e * W:(e + 1) * W].double()
    params = {"hidden_size": W, "intermediate_size": F, "num_experts": E, "top": top, "vocab_size": V}
    if shared:
        t["shared_up"], t["shared_down"] = (torch.randn(shared, W, generator=g) * W ** -0.5).to(dt), (torch.randn(W, shared, generator=g) * shared ** -0.5).to(dt)
        w["shared.up"], w["shared.down"] = t["shared_up"].double(), t["shared_down"].double()
        params["shared_size"] = shared

    class Build:
        dtype, device = dt, torch.device("cuda")

        @staticmethod
        def tensor(spec, name):
            return t[name].cuda()
    part = RoutedTableFeedForward(PartSpec("feed_forward", "routed_table", params, {n: tensor(n, tuple(x.shape)) for n, x in t.items()}), Build)
    f = {"router": {"experts": E, "top": top}, **({"shared": {"ff": shared}} if shared else {})}
    # (squares of bfloat16 numbers summed over few inner values: outputs of several units)
    tol = dict(atol=1e-4, rtol=1e-4) if dtype == "float32" else dict(atol=8e-2, rtol=3e-2)
    for n, same in ((1, False), (9, False), (16, True), (17, False), (128, False), (128, True), (129, True), (200, False)):
        ids = [5] * n if same else torch.randint(0, V, (n,), generator=g).tolist()
        h = torch.randn(n, W, generator=g).to(dt)
        want = P.table_experts(h.double(), ids, w, "", f)
        ctx = _step_context([0], [n], ids=[ids])
        got = part.forward(h.cuda(), ctx)
        assert torch.allclose(got.cpu().double(), want, **tol), (n, same, float((got.cpu().double() - want).abs().max()))
    chosen, weight = ops.moe_route_table(torch.tensor([3, 36, 0], dtype=torch.int32).cuda(), t["table"].cuda())
    assert torch.equal(chosen.cpu(), t["table"][[3, 36, 0]]) and torch.allclose(weight.cpu(), torch.full((3, top), 1.0 / top))
    t["table"][2, 0] = E
    with pytest.raises(ValueError, match="names expert"):
        RoutedTableFeedForward(PartSpec("feed_forward", "routed_table", params, {n: tensor(n, tuple(x.shape)) for n, x in t.items()}), Build)


# ---- whole models ----------------------------------------------------------------------------------------

@gpu
@pytest.mark.parametrize("name,dtype", CASES)
def test_each_request_alone_and_whole(tmp_path_factory, name, dtype):
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    for ids in S.prompts(raw_of(name), LENGTHS[name]):
        slot = eng.open()
        got = eng.step([StepEntry(slot, ids, list(range(len(ids))))])
        eng.close(slot)
        assert_close(got, reference(tmp_path_factory, name, dtype, ids), dtype, f"{name} whole {len(ids)}")
    eng.cache.check()


@gpu
@pytest.mark.parametrize("name", ["A", "C"])
def test_the_stream_after_every_layer(tmp_path_factory, name):
    """The residual stream after each layer, in float32: a hook on the blocks reads it (a branch's output joins the stream in
    the pass of the norm that reads it next; the last layer's only for the wanted rows: the logits of the other tests cover it)."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, "float32", graphs=False)
    ids = S.prompts(raw_of(name), [40], seed=2)[0]
    cfg, w = P.read_model(model_dir(tmp_path_factory, name, "float32"))
    want, seen = [], []
    P.forward(cfg, w, ids, want)
    originals = [b.forward for b in eng.model.layers]
    for b in eng.model.layers:
        def hooked(x, h, ctx, sink, _f=b.forward):
            out = _f(x, h, ctx, sink)
            seen.append(x.detach().clone())
            return out
        b.forward = hooked
    try:
        slot = eng.open()
        eng.step([StepEntry(slot, ids, list(range(len(ids))))])
        eng.close(slot)
    finally:
        for b, f in zip(eng.model.layers, originals):
            b.forward = f
    assert len(seen) == len(want) == 4
    for i, (a, b) in enumerate(zip(seen[:-1], want[:-1])):
        assert torch.allclose(a.cpu().double(), b, atol=2e-4, rtol=1e-4), (i, float((a.cpu().double() - b).abs().max()))


@gpu
def test_a_checkpoint_with_the_second_norm_of_a_layer_without_a_feed_forward(tmp_path):
    from palm_infra_amd.engine import Engine, StepEntry
    from palm_infra_amd.weights import write_safetensors
    raw = raw_of("A")
    tensors = S.tensors_of(raw, 7, "float32")
    tensors["l2.norm2"] = torch.full((64,), 3.0)
    (tmp_path / "config.json").write_text(json.dumps(raw))
    write_safetensors(tmp_path / "model.safetensors", tensors)
    eng = Engine.from_dir(tmp_path, dtype="float32", max_tokens=256)
    ids = S.prompts(raw, [40], seed=12)[0]
    slot = eng.open()
    got = eng.step([StepEntry(slot, ids, list(range(len(ids))))])
    eng.close(slot)
    cfg, w = P.read_model(tmp_path)
    assert_close(got, P.forward(cfg, w, ids), "float32", "spare norm")


@gpu
@pytest.mark.parametrize("name,dtype", CASES)
def test_prompt_then_every_token_alone_from_the_first(tmp_path_factory, name, dtype):
    """Token-by-token decoding from the very first token, through recorded steps, across page borders and past the windows."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    ids = S.prompts(raw_of(name), [150], seed=4)[0]
    ref = reference(tmp_path_factory, name, dtype, ids)
    slot = eng.open()
    got = []
    for t, tok in enumerate(ids):
        got.append(eng.step([StepEntry(slot, [tok], [0])]))
        assert eng.length(slot) == t + 1
    eng.close(slot)
    assert_close(torch.cat(got), ref, dtype, f"{name} one by one")


@gpu
@pytest.mark.parametrize("name,dtype", CASES)
@pytest.mark.parametrize("portion", [2, 3, 7, 64, 65])
def test_prompt_in_portions(tmp_path_factory, name, dtype, portion):
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    ids = S.prompts(raw_of(name), [140], seed=5)[0]
    ref = reference(tmp_path_factory, name, dtype, ids)
    slot = eng.open()
    got = []
    for lo in range(0, len(ids), portion):
        piece = ids[lo:lo + portion]
        got.append(eng.step([StepEntry(slot, piece, list(range(len(piece))))]))
    eng.close(slot)
    assert_close(torch.cat(got), ref, dtype, f"{name} in portions of {portion}")


@gpu
@pytest.mark.parametrize("name,dtype", CASES)
def test_portions_with_one_place_wanted_are_recorded_too(tmp_path_factory, name, dtype):
    """Short portions of one sequence with their last place wanted replay a recorded prompt step, whose padding is a sequence of
    its own; the tokens' experts come from the ids laid into the recording's buffer."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    for seed in (14, 15):
        ids = S.prompts(raw_of(name), [132], seed=seed)[0]
        ref = reference(tmp_path_factory, name, dtype, ids)
        slot, got = eng.open(), []
        for lo in range(0, len(ids), 11):
            got.append(eng.step([StepEntry(slot, ids[lo:lo + 11], [10])]))
        eng.close(slot)
        assert_close(torch.cat(got), ref[10::11], dtype, f"{name} recorded portions")


@gpu
@pytest.mark.parametrize("name,dtype", CASES)
def test_batches_of_unequal_requests_and_reused_slots(tmp_path_factory, name, dtype):
    """Two batches through the same slots and pages: prompts of unequal lengths in one step minus their last tokens, which
    come one a step; a request that has no tokens left ends and gives its slot and pages back at once."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    for turn, (seed, tails) in enumerate([(6, [0, 1, 9, 3, 20, 5, 2, 11]), (7, [12, 0, 2, 7, 30, 1, 1, 4])]):
        lengths = LENGTHS[name] if turn == 0 else LENGTHS[name][::-1]
        reqs = S.prompts(raw_of(name), lengths, seed=seed)
        tails = [min(t, len(r) - 1) for t, r in zip(tails, reqs)]
        slots = [eng.open() for _ in reqs]
        assert sorted(slots) == list(range(len(reqs)))                # the second batch gets the first one's slots
        cuts = [len(r) - t for r, t in zip(reqs, tails)]
        got = {i: [] for i in range(len(reqs))}
        out = eng.step([StepEntry(s, r[:c], list(range(c))) for s, r, c in zip(slots, reqs, cuts)])
        o = 0
        for i, c in enumerate(cuts):
            got[i].append(out[o:o + c])
            o += c
        live, fed = list(range(len(reqs))), list(cuts)
        while True:
            for i in [i for i in live if fed[i] == len(reqs[i])]:
                eng.close(slots[i])
                live.remove(i)
            if not live:
                break
            out = eng.step([StepEntry(slots[i], [reqs[i][fed[i]]], [0]) for i in live])
            for r, i in enumerate(live):
                got[i].append(out[r:r + 1])
                fed[i] += 1
        for i, r in enumerate(reqs):
            assert_close(torch.cat(got[i]), reference(tmp_path_factory, name, dtype, r), dtype,
                         f"{name} batch {turn} request {i} ({len(r)} tokens, {tails[i]} one by one)")
        eng.cache.check()
        assert all(g.table.pages.held_count == 0 for g in eng.cache.paged_groups)


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_padded_recorded_step_of_many_sequences(tmp_path_factory, dtype):
    """Nineteen sequences of unequal lengths decode together (the recorded step is padded to twenty-four rows), more rows than
    share the shared expert in the experts' kernels, then fewer."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, "A", dtype)
    reqs = S.prompts(raw_of("A"), [3 + 4 * i for i in range(19)], seed=16)
    refs = [reference(tmp_path_factory, "A", dtype, r) for r in reqs]
    slots = [eng.open() for _ in reqs]
    eng.step([StepEntry(s, r[:-2], []) for s, r in zip(slots, reqs)])
    got = eng.step([StepEntry(s, [r[-2]], [0]) for s, r in zip(slots, reqs)])
    assert_close(got, torch.stack([r[-2] for r in refs]), dtype, "nineteen")
    for s in slots[7:]:
        eng.close(s)
    got = eng.step([StepEntry(s, [r[-1]], [0]) for s, r in zip(slots[:7], reqs)])
    assert_close(got, torch.stack([r[-1] for r in refs[:7]]), dtype, "seven of them")
    for s in slots[:7]:
        eng.close(s)


@gpu
@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("B", "bfloat16"), ("C", "bfloat16"), ("D", "float32")])
def test_long_decoding(tmp_path_factory, name, dtype):
    """A short prompt, then some hundred tokens one by one over several pages and windows, two sequences side by side that
    started at different lengths; a windowed layer gives pages back on the way, a latent layer keeps them all."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    a, b = S.prompts(raw_of(name), [330, 270], seed=8)
    refs = [reference(tmp_path_factory, name, dtype, a), reference(tmp_path_factory, name, dtype, b)]
    sa, sb = eng.open(), eng.open()
    got = [eng.step([StepEntry(sa, a[:70], [69]), StepEntry(sb, b[:10], [9])])]
    want = [torch.stack([refs[0][69], refs[1][9]])]
    for i in range(260):
        got.append(eng.step([StepEntry(sa, [a[70 + i]], [0]), StepEntry(sb, [b[10 + i]], [0])]))
        want.append(torch.stack([refs[0][70 + i], refs[1][10 + i]]))
    for g in eng.cache.paged_groups:
        held = 2 * (g.table.window // 64 + 2) if g.table.window else 6 + 5
        assert g.table.pages.held_count <= held and (g.table.window or g.table.pages.held_count == held)
    eng.close(sa)
    eng.close(sb)
    assert_close(torch.cat(got), torch.cat(want), dtype, f"{name} long decoding")


@gpu
@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("C", "bfloat16")])
def test_a_prompt_longer_than_a_step_takes_at_once(tmp_path_factory, name, dtype):
    """A windowed model cuts a long prompt into pieces between which pages go back."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    assert eng.step_tokens_per_seq == 1024
    ids = S.prompts(raw_of(name), [1100], seed=13)[0]
    want = [0, 1, 511, 1023, 1024, 1025, 1099]
    slot = eng.open()
    got = eng.step([StepEntry(slot, ids, want)])
    more = eng.step([StepEntry(slot, [ids[5]], [0])])                       # and a single token after it
    eng.close(slot)
    ref = reference(tmp_path_factory, name, dtype, ids + [ids[5]])
    assert_close(torch.cat([got, more]), ref[want + [1100]], dtype, f"{name} long prompt")


@gpu
@pytest.mark.parametrize("name", ["A", "D"])
def test_recorded_and_launched_steps_agree(tmp_path_factory, name):
    """Decode steps replayed from a HIP graph against the same steps launched kernel by kernel, several replays with other
    work between them."""
    from palm_infra_amd.engine import StepEntry
    ids = S.prompts(raw_of(name), [90], seed=9)[0]
    for dtype in DTYPES:
        outs = []
        for graphs in (True, False):
            eng = engine_for(tmp_path_factory, name, dtype, graphs=graphs)
            assert eng.model.capturable
            slot = eng.open()
            got = [eng.step([StepEntry(slot, ids[:50], [49])])]
            for t in range(50, 90):
                got.append(eng.step([StepEntry(slot, [ids[t]], [0])]))
                torch.cuda.synchronize()
            eng.close(slot)
            outs.append(torch.cat(got).cpu())
        # (a recorded step is cut into slices for the longest sequence it serves: sums in another order)
        assert torch.allclose(outs[0], outs[1], atol=1e-5 if dtype == "float32" else 5e-2)
        assert_close(outs[0], reference(tmp_path_factory, name, dtype, ids)[49:], dtype, f"{name} recorded steps")


@gpu
@pytest.mark.parametrize("name", ["A", "B", "C", "D"])
def test_greedy_generation_through_generate(tmp_path_factory, name):
    from palm_infra_amd.sampling import GREEDY
    eng = engine_for(tmp_path_factory, name, "float32")
    cfg, w = P.read_model(model_dir(tmp_path_factory, name, "float32"))
    prompts = S.prompts(raw_of(name), [5, 1, 66, 19], seed=10)
    results, metrics = eng.generate(prompts, GREEDY, max_new_tokens=12, ignore_eos=True, max_batch=3)
    for p, r in zip(prompts, results):
        assert r.token_ids == P.greedy(cfg, w, p, 12), f"{name}: prompt of {len(p)} tokens"
    eng.cache.check()
    assert eng.cache.slots.held_count == 0


@gpu
def test_command_line_generates_for_the_design(tmp_path_factory, capsys):
    from palm_infra_amd.engine.cli import chat_main
    d = model_dir(tmp_path_factory, "D", "float32")
    cfg, w = P.read_model(d)
    rc = chat_main(["--package", str(d), "--prompt-ids", "5,6,7", "--max-new-tokens", "6", "--temperature", "0",
                    "--dtype", "float32", "--ignore-eos"])
    assert rc == 0
    assert " ".join(str(t) for t in P.greedy(cfg, w, [5, 6, 7], 6)) in capsys.readouterr().out


@gpu
def test_random_weights_on_the_device_are_those_of_the_written_folder(tmp_path):
    """Also the integer tables, which the device gets from the host's function."""
    from palm_infra_amd.engine import Engine, StepEntry
    from palm_infra_amd.weights import write_random_model
    write_random_model(S.CONFIGS["A"], 21, tmp_path, "bfloat16")
    ids = S.prompts(S.CONFIGS["A"], [30], seed=17)[0]
    outs = []
    for eng in (Engine.from_dir(tmp_path, max_tokens=256), Engine.from_config(S.CONFIGS["A"], seed=21, max_tokens=256)):
        assert int(eng.model.layers[0].feed_forward.table.max()) == 7
        outs.append(eng.step([StepEntry(eng.open(), ids, list(range(30)))]).cpu())
    assert torch.equal(outs[0], outs[1])


@gpu
def test_trace_replay_of_a_batch_then_single_tokens(tmp_path_factory, tmp_path):
    """bin/trace_run as a child process: four requests of unequal lengths in one batch, then one token each while the
    shorter ones end; the files it writes against the plain implementation."""
    import subprocess
    import sys
    from pathlib import Path
    import numpy as np
    d = model_dir(tmp_path_factory, "A", "float32")
    reqs = S.prompts(raw_of("A"), [75, 4, 140, 1], seed=11)
    heads = [70, 2, 130, 1]
    steps = [{"step": 0, "entries": [{"id": f"r{i}", "tokens": r[:h], "want": [0, h - 1]} for i, (r, h) in enumerate(zip(reqs, heads))],
              "end": ["r3"]}]
    fed = list(heads)
    for s in range(1, 11):
        live = [i for i in range(3) if fed[i] < len(reqs[i])]
        steps.append({"step": s, "entries": [{"id": f"r{i}", "tokens": [reqs[i][fed[i]]], "want": [0] if s % 2 else []} for i in live],
                      "end": [f"r{i}" for i in live if fed[i] + 1 == len(reqs[i])]})
        for i in live:
            fed[i] += 1
    root = Path(__file__).resolve().parent.parent
    out = tmp_path / "out"
    run = subprocess.run([sys.executable, str(root / "bin" / "trace_run"), "--model", str(d), "--dtype", "float32", "--out", str(out),
                          "--max-tokens", "320"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=110)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == [f"done {s}" for s in range(11)]
    refs = [reference(tmp_path_factory, "A", "float32", r) for r in reqs]
    first = np.fromfile(out / "0.f32", dtype="<f4").reshape(8, -1)
    want = torch.stack([refs[i][p] for i, h in enumerate(heads) for p in (0, h - 1)])
    assert_close(torch.from_numpy(first.copy()), want, "float32", "trace step 0")
    fed = list(heads)
    for s in range(1, 11):
        live = [i for i in range(3) if fed[i] < len(reqs[i])]
        if s % 2 and live:
            got = np.fromfile(out / f"{s}.f32", dtype="<f4").reshape(len(live), -1)
            assert_close(torch.from_numpy(got.copy()), torch.stack([refs[i][fed[i]] for i in live]), "float32", f"trace step {s}")
        else:
            assert not (out / f"{s}.f32").exists()
        for i in live:
            fed[i] += 1
