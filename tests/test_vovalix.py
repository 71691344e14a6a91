"""The Vovalix design in the engine against the plain implementation (tests/plain_vovalix.py).

Without a GPU: the configuration, its description as parts, the run order and cache plan, pages by chunks, the oracle's own
mechanisms against closed forms, and that a mistake planted in any mechanism of the oracle moves the logits far beyond what
the comparisons allow.  On the GPU: every mechanism alone (one-layer models, and the kernels called directly with inputs made
so that one far key, one key at a chunk's or a page's edge, a far write into a state or a group of experts decides the result),
whole prompts, prompts cut into portions down to two tokens, prefill against token-by-token decoding from the first token,
batches of unequal requests against each alone, slots and pages that are used again, long decoding over several pages and
chunks, a prompt longer than a step takes at once, recorded against launched steps, and greedy generation through ``generate``,
the command line and the trace replay.  In float32 and in bfloat16.
"""
import json
import math

import pytest
import torch

import plain_vovalix as P
import vovalix_tiny as S
from palm_infra_amd.config import ConfigError, config_from_dict

gpu = pytest.mark.gpu
DTYPES = ("float32", "bfloat16")
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}
LENGTHS = {"A": [1, 2, 63, 64, 65, 130, 200, 37], "B": [129, 3, 70, 71, 1, 191], "C": [300, 9, 140], "D": [5, 66, 128, 31], "E": [67, 1, 20]}


# ---- without a GPU ---------------------------------------------------------------------------------------

def test_registry_picks_the_design_by_its_config_key():
    cfg = config_from_dict(S.CONFIGS["A"])
    assert type(cfg).__name__ == "VovalixConfig"
    again = config_from_dict(json.loads(json.dumps(cfg.to_dict())))
    assert again.to_dict() == cfg.to_dict() and again.logit_scale == 0.7


def test_spec_names_every_tensor():
    names = config_from_dict(S.CONFIGS["A"]).spec().expected_tensors()
    assert names["embed"][0] == (211, 64) and names["final.norm"][0] == (64,) and names["l0.norm1"][0] == (64,)
    assert names["l0.mix.q"][0] == names["l0.mix.k"][0] == (48, 64) and names["l0.mix.v"][0] == names["l0.mix.g"][0] == (240, 64)
    assert names["l0.mix.q.conv"][0] == (48, 3) and names["l0.mix.v.conv"][0] == (240, 3) and names["l0.mix.o"][0] == (64, 240)
    assert names["l0.mix.a"][0] == names["l0.mix.b"][0] == (6, 64) and names["l0.mix.A_log"][0] == names["l0.mix.dt_bias"][0] == (6,)
    assert names["l0.mix.norm"][0] == (40,)
    assert names["l1.mix.q"][0] == (144, 64) and names["l1.mix.k"][0] == (48, 64) and names["l1.mix.v"][0] == (80, 64) and "l1.mix.norm" not in names
    assert names["l1.mlp.e11.gate"][0] == names["l1.mlp.e0.up"][0] == (24, 64) and names["l1.mlp.e3.down"][0] == (64, 24)
    assert names["l1.mlp.router"][0] == (12, 64) and names["l1.mlp.shared.up"][0] == (40, 64) and names["l1.mlp.shared.down"][0] == (64, 40)
    assert names["l2.mix.a1"][0] == (5, 64) and names["l2.mix.a2"][0] == (48, 5) and names["l2.mix.a2.b"][0] == (48,) and names["l2.mix.norm"][0] == (24,)
    # a layer without a feed-forward, and layers that use another layer's weights, have no tensors for them
    assert not any(n.startswith(("l2.mlp", "l3.", "l4.")) for n in names) and "head" not in names


def test_ranks_come_from_the_tensors_shapes():
    raw = json.loads(json.dumps(S.CONFIGS["A"]))
    for entry in raw["layers"]:
        entry["mixer"].pop("decay_rank", None)
    cfg = config_from_dict(raw)
    with pytest.raises(ConfigError, match="rank"):
        cfg.spec()
    shapes = {n: s for n, (s, _) in config_from_dict(S.CONFIGS["A"]).spec().expected_tensors().items()}
    assert cfg.with_tensor_shapes(shapes).spec() == config_from_dict(S.CONFIGS["A"]).spec()


def test_run_order_and_cache_plan():
    from palm_infra_amd.cache import KVNeed, StateNeed
    from palm_infra_amd.parts import cache_needs
    spec = config_from_dict(S.CONFIGS["A"]).spec()
    assert [c.layer for c in spec.order] == [0, 1, 2, 1, 2] and all(c.cache_of is None for c in spec.order) and len(spec.layers) == 3
    assert cache_needs(spec.layers[0]) == [StateNeed("delta", (6, 24, 40)), StateNeed("delta_conv", (2, 2 * 48 + 240))]
    assert cache_needs(spec.layers[1]) == [KVNeed(2, 24, 37, value_dim=40, chunked=True)]
    assert cache_needs(spec.layers[2]) == [StateNeed("gla", (3, 16, 24))]
    d = config_from_dict(S.CONFIGS["D"]).spec()
    assert [c.layer for c in d.order] == [1, 0, 1, 2] and len(d.layers) == 3              # layer 0 uses layer 2's weights
    c = config_from_dict(S.CONFIGS["C"]).spec()
    assert cache_needs(c.layers[3]) == [KVNeed(4, 32, None, value_dim=96)]                # no chunks: every key is kept


def test_pages_below_the_current_chunk_go_back():
    from palm_infra_amd.cache.pool import PageTable
    t = PageTable(8, 1, 8, window=100, chunked=True)
    t.grow(0, 100)
    t.trim(0, 100)                                   # the next query, at 100, begins a chunk: page 0 lies wholly below it, page 1 does not
    assert [p >= 0 for p in t.slot_pages[0]] == [False, True]
    t.grow(0, 199)
    t.trim(0, 199)                                   # still the chunk from 100 on
    assert [p >= 0 for p in t.slot_pages[0]] == [False, True, True, True]
    t.trim(0, 200)                                   # the chunk from 200 on: pages 1 and 2 (64 .. 191) go back, page 3 holds 192 .. 255
    assert [p >= 0 for p in t.slot_pages[0]] == [False, False, False, True]
    t.check()
    with pytest.raises(ValueError, match="size"):
        PageTable(8, 1, 8, chunked=True)


@pytest.mark.parametrize("change,what", [
    (lambda c: c["layers"][0].update(type="retention"), "type"),
    (lambda c: c["layers"][1]["mixer"].update(kv_heads=4), "kv heads"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].update(mask={}) or c["layers"][1]["mixer"]["mask"].update(size=0), "mask.size"),
    (lambda c: c["layers"][0]["mixer"].update(conv=40), "conv"),
    (lambda c: c["layers"][2]["mixer"].pop("tau"), "tau"),
    (lambda c: c["layers"][2]["mixer"].update(tau=-1), "tau"),
    (lambda c: c["layers"][2]["mixer"].update(dim=300), "key sizes"),
    (lambda c: c["layers"][3].update(weights_of=3), "weights_of"),
    (lambda c: c["layers"][3].update(weights_of=0), "another layer"),
    (lambda c: c["layers"][1].update(weights_of=3), "leads back"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "kind"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "experts"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=3), "choices"),
    (lambda c: c["layers"][0]["mlp"]["router"]["groups"].update(count=5), "groups"),
    (lambda c: c["norm"].pop("eps"), "eps"),
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
    assert logits.shape == (5, 97) and torch.isfinite(logits).all() and len(layers) == 4


def test_plain_attention_sees_its_own_chunk_and_loses_by_the_distance():
    T, size = 11, 4
    q, k = torch.zeros(T, 2, 3, dtype=P.F64), torch.randn(T, 1, 3, dtype=P.F64)
    v = torch.eye(T, dtype=P.F64).reshape(T, 1, T)
    slopes = P.head_slopes(2)
    assert slopes == [2.0 ** -4, 2.0 ** -8]
    out = P.chunk_softmax_heads(q, k, v, 1.0, slopes, size)
    for i in range(T):
        for h in range(2):
            want = torch.zeros(T, dtype=P.F64)
            for j in range(i // size * size, i + 1):
                want[j] = math.exp(-slopes[h] * (i - j))
            assert torch.allclose(out[i, h], want / want.sum())


def test_plain_gla_is_a_decayed_sum_over_its_past():
    torch.manual_seed(0)
    T, H, d, dv = 9, 2, 3, 4
    q, k, a = (torch.randn(T, H, d, dtype=P.F64) for _ in range(3))
    a, v = torch.sigmoid(a), torch.randn(T, H, dv, dtype=P.F64)
    out, _ = P.gla_recurrence(q, k, v, a)
    for t in range(T):
        for h in range(H):
            want = sum(float((q[t, h] * k[j, h] * a[j + 1:t + 1, h].prod(0)).sum()) * v[j, h] for j in range(t + 1))
            assert torch.allclose(out[t, h], want)
    w = {"a1": torch.tensor([[1.0]], dtype=P.F64), "a2": torch.tensor([[2.0], [0.0]], dtype=P.F64), "a2.b": torch.tensor([0.5, -1.0], dtype=P.F64)}
    got = P.channel_decays(torch.tensor([[3.0]], dtype=P.F64), w, "", 4.0)
    assert torch.allclose(got, torch.tensor([[(1 / (1 + math.exp(-6.5))) ** 0.25, (1 / (1 + math.exp(1.0))) ** 0.25]], dtype=P.F64))


def test_plain_delta_rule_recalls_what_it_wrote_and_reads_its_own_write():
    """With orthonormal keys, full write strength and no decay a key's value is whatever was written last; the token's own
    write is already in what it reads."""
    k = torch.eye(3, dtype=P.F64)[[0, 1, 0, 2]].reshape(4, 1, 3)
    v = torch.arange(1.0, 9.0, dtype=P.F64).reshape(4, 1, 2)
    one = torch.ones(4, 1, dtype=P.F64)
    assert torch.allclose(P.delta_recurrence(k, k, v, one, one), v)
    q = torch.eye(3, dtype=P.F64)[[0, 0, 1, 0]].reshape(4, 1, 3)
    assert torch.allclose(P.delta_recurrence(q, k, v, one, one)[:, 0], v[[0, 0, 1, 2], 0])
    half = P.delta_recurrence(q, k, v, one, 0.5 * one)[:, 0]                # g is applied before the write: once a token since
    assert torch.allclose(half, torch.stack([v[0, 0], 0.5 * v[0, 0], 0.5 * v[1, 0], 0.5 * v[2, 0]]))
    u = torch.arange(1.0, 11.0, dtype=P.F64).reshape(5, 2)
    y = P.short_convolution(u, torch.tensor([[1.0, 10.0, 100.0], [0.0, 0.0, 2.0]], dtype=P.F64))
    assert y[:, 1].tolist() == [4.0, 8.0, 12.0, 16.0, 20.0] and y[:, 0].tolist() == [100.0, 310.0, 531.0, 753.0, 975.0]


def test_plain_routing_by_the_groups_largest_score():
    """Two groups of two, one kept.  The group with the largest single score wins, though the other's two sum higher."""
    z = torch.tensor([[2.0, -9.0, 1.8, 1.7]], dtype=P.F64)
    r = {"experts": 4, "top": 2, "groups": {"count": 2, "keep": 1}}
    chosen, weights = P.route(z, r)
    assert chosen[0].tolist() == [0, 1]
    assert torch.allclose(weights[0], torch.tensor([1.0, math.exp(-11.0)], dtype=P.F64) / (1 + math.exp(-11.0)))
    chosen, weights = P.route(z, {"experts": 4, "top": 2})
    assert chosen[0].tolist() == [0, 2] and math.isclose(float(weights.sum()), 1.0)
    w = {"gate": torch.tensor([[5.0], [-3.0]], dtype=P.F64), "up": torch.tensor([[9.0], [-9.0]], dtype=P.F64), "down": torch.eye(2, dtype=P.F64)}
    got = P.capped_expert(torch.tensor([[1.0]], dtype=P.F64), w, "", 2.0)[0]
    s = lambda x: 1 / (1 + math.exp(-1.702 * x))
    assert torch.allclose(got, torch.tensor([2.0 * s(2.0) * 3.0, -3.0 * s(-3.0) * -1.0], dtype=P.F64))


# A mistake in any mechanism must show: each of these, planted in the oracle, moves some logits by more than twenty times what a
# float32 comparison allows (and most by more than a bfloat16 one does).
def _plant(monkeypatch, what):
    if what == "slope":
        monkeypatch.setattr(P, "head_slopes", lambda H: [2.0 ** (-8.0 * h / H) for h in range(H)])
    elif what in ("chunk one longer", "chunk one shorter", "window"):
        plain, by = P.chunk_softmax_heads, 1 if what == "chunk one longer" else -1
        if what == "window":
            def windowed(q, k, v, scale, slopes, size):
                keep = torch.stack([plain(q[max(0, t - size + 1):t + 1], k[max(0, t - size + 1):t + 1], v[max(0, t - size + 1):t + 1], scale, slopes, None)[-1]
                                    for t in range(q.shape[0])])
                return keep
            monkeypatch.setattr(P, "chunk_softmax_heads", windowed)
        else:
            monkeypatch.setattr(P, "chunk_softmax_heads", lambda q, k, v, scale, slopes, size: plain(q, k, v, scale, slopes, size + by))
    elif what == "no unit heads":
        unit = P.unit_rms
        monkeypatch.setattr(P, "unit_rms", lambda x, eps: x if x.dim() == 3 and x.shape[-1] == 24 else unit(x, eps))
    elif what == "tau":
        decays = P.channel_decays
        monkeypatch.setattr(P, "channel_decays", lambda h, w, p, tau: decays(h, w, p, 1.0))
    elif what == "lost state":
        rec = P.gla_recurrence
        monkeypatch.setattr(P, "gla_recurrence", lambda q, k, v, a: (torch.cat([rec(q[:64], k[:64], v[:64], a[:64])[0], rec(q[64:], k[64:], v[64:], a[64:])[0]]), None))
    elif what == "read before write":
        rec = P.delta_recurrence
        monkeypatch.setattr(P, "delta_recurrence", lambda q, k, v, b, g: rec(q, k, v, b, g) - (q * k).sum(-1).repeat_interleave(v.shape[1] // q.shape[1], 1)[..., None] * b[..., None] * v)
    elif what == "convolution shifted":
        conv = P.short_convolution
        monkeypatch.setattr(P, "short_convolution", lambda u, w: conv(u, w.roll(1, 1)))
    elif what == "group sums":
        def by_sum(z, r):
            s = torch.softmax(z, -1)
            if not r.get("groups"):
                return route(z, r)
            c, keep = r["groups"]["count"], r["groups"]["keep"]
            g = s.reshape(len(z), c, -1)
            best = g.topk(min(2, g.shape[2]), 2).values.sum(2).topk(keep, 1).indices
            allowed = torch.zeros(len(z), c, dtype=torch.bool).scatter_(1, best, True)
            chosen = g.masked_fill(~allowed[..., None], -math.inf).reshape(len(z), -1).topk(r["top"], 1).indices
            picked = s.gather(1, chosen)
            return chosen, picked / picked.sum(1, keepdim=True)
        route = P.route
        monkeypatch.setattr(P, "route", by_sum)
    elif what == "one limit for both":
        routed = P.routed_feed_forward
        monkeypatch.setattr(P, "routed_feed_forward", lambda h, w, p, f: routed(h, w, p, dict(f, shared=dict(f["shared"], limit=f["expert"]["limit"])) if f.get("shared") else f))
    elif what == "weights not normed":
        route = P.route
        monkeypatch.setattr(P, "route", lambda z, r: (route(z, r)[0], torch.softmax(z, -1).gather(1, route(z, r)[0])))
    elif what == "norm weight":
        monkeypatch.setattr(P, "norm_around_zero", lambda x, w, eps: P.unit_rms(x, eps) * (1.0 - w))
    else:
        raise KeyError(what)


@pytest.mark.parametrize("what", ["slope", "chunk one longer", "chunk one shorter", "window", "no unit heads", "tau", "lost state", "read before write",
                                  "convolution shifted", "group sums", "one limit for both", "weights not normed", "norm weight"])
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
        _dirs[key] = S.write_model(raw_of(name), S.SEEDS.get(name, 81), tmp_path_factory.mktemp(f"vovalix_{name}_{store}"), store)
    return _dirs[key]


def engine_for(tmp_path_factory, name: str, dtype: str, **options):
    from palm_infra_amd.engine import Engine
    key = (name, dtype, tuple(sorted(options.items())))
    if key not in _engines:
        _engines[key] = Engine.from_dir(model_dir(tmp_path_factory, name, dtype), dtype=dtype, max_tokens=64 * 24, **options)
    return _engines[key]


class Rows:
    """Logits of the plain implementation, and which of the rows lie before the request's first close call of a router."""
    CLOSE = 0.03                                                   # of router logits, whose own scale is about one

    def __init__(self, logits, clean):
        self.logits, self.clean = logits, clean

    def __getitem__(self, at):
        at = [at] if isinstance(at, int) else at
        return Rows(self.logits[at], self.clean[at])

    @staticmethod
    def joined(parts):
        return Rows(torch.cat([p.logits for p in parts]), torch.cat([p.clean for p in parts]))


def reference(tmp_path_factory, name: str, dtype: str, ids) -> Rows:
    key = (name, dtype, tuple(ids))
    if key not in _refs:
        cfg, w = P.read_model(model_dir(tmp_path_factory, name, dtype))
        margins = []
        logits = P.forward(cfg, w, ids, margins=margins)
        close = torch.stack(margins).min(0).values < Rows.CLOSE if margins else torch.zeros(len(ids), dtype=torch.bool)
        _refs[key] = Rows(logits, close.cumsum(0) == 0)
    return _refs[key]


def assert_close(got, ref, dtype: str, what: str = "") -> None:
    """float32: 1e-4 of the logits' scale, the gate that shows faults.  bfloat16: a row's root mean square error within a
    tenth of the logits' scale (half of the rows within a fiftieth: a head whose output nearly vanishes is scaled up again with
    its rounding by its unit norm) for every row before the request's first close call (a choice between two experts or groups
    of nearly equal scores may fall the other way, for that token and for what later ones read of it); of all rows one in four
    may lie beyond.  The float32 runs hold every row, and so do the kernels'
    own tests below in bfloat16."""
    ref, clean = (ref.logits, ref.clean) if isinstance(ref, Rows) else (ref, torch.ones(len(ref), dtype=torch.bool))
    got = torch.as_tensor(got).double().cpu().reshape(ref.shape)
    assert torch.isfinite(got).all(), f"{what}: logits are not finite"
    err = (got - ref.double()).abs().reshape(-1, ref.shape[-1])
    scale = float(ref.double().pow(2).mean().sqrt())
    if dtype == "float32":
        worst = float(err.max())
        assert worst <= 1e-4 * max(1.0, scale), f"{what}: float32 logits differ by {worst:.3e} (their scale is {scale:.3e})"
        return
    rows = err.pow(2).mean(-1).sqrt()
    over = rows > 0.1 * scale
    assert int(over.sum()) <= max(1, rows.numel() // 4), f"{what}: {int(over.sum())} of {rows.numel()} rows beyond the bfloat16 bound"
    if clean.any():
        worst = float(rows[clean].max())
        assert worst <= 0.1 * scale, f"{what}: bfloat16 rms error {worst:.3e} before the first close call, vs {scale:.3e}"
        assert float(err[clean].max()) <= 0.4 * scale, f"{what}: bfloat16 max error {float(err[clean].max()):.3e} vs {scale:.3e}"
        middle = float(rows[clean].median())
        assert int(clean.sum()) < 8 or middle <= 0.02 * scale, f"{what}: bfloat16 median rms error {middle:.3e} vs {scale:.3e}"


CASES = [(n, d) for n in ("A", "B", "C", "D", "E") for d in DTYPES]


def _step_context(lengths_before, new_counts, slots=None):
    """A cache-less context for kernels that only need the packed layout."""
    from palm_infra_amd.parts import make_context
    slots = list(range(len(new_counts))) if slots is None else list(slots)
    return make_context(slots, list(lengths_before), [[0] * c for c in new_counts], torch.float32, "cuda")


def _run_schedule(lengths, cuts, slots, step):
    """Two sequences through ``step(ctx, live, fed, counts)`` in portions ``cuts[b]``; the outputs of each, joined."""
    got, fed = [[] for _ in lengths], [0] * len(lengths)
    for i in range(max(len(c) for c in cuts)):
        live = [b for b in range(len(lengths)) if i < len(cuts[b])]
        counts = [cuts[b][i] for b in live]
        out = step(_step_context([fed[b] for b in live], counts, slots=[slots[b] for b in live]), live, list(fed), counts)
        o = 0
        for b, c in zip(live, counts):
            got[b].append(out[o:o + c].cpu())
            o += c
            fed[b] += c
    assert fed == [sum(c) for c in cuts]
    return [torch.cat(g).double() for g in got]


# ---- every mechanism alone -------------------------------------------------------------------------------

@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", sorted(S.SINGLE))
def test_one_layer_of_one_kind(tmp_path_factory, kind, dtype):
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, kind, dtype)
    for ids in S.prompts(raw_of(kind), [1, 7, 64, 131], seed=1):
        slot = eng.open()
        got = eng.step([StepEntry(slot, ids, list(range(len(ids))))])
        eng.close(slot)
        assert_close(got, reference(tmp_path_factory, kind, dtype, ids), dtype, f"{kind} whole {len(ids)}")


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_unit_heads_of_q_and_k_go_to_their_pages(dtype):
    from palm_infra_amd.kernels import ops
    torch.manual_seed(4)
    dt, H, G, d, dv, eps, n = TORCH[dtype], 6, 3, 20, 12, 1e-3, 70
    rows = torch.randn(n, 2 + H * d + G * (d + dv) + 3).to(dt)                       # two columns before, three after
    k_cache = torch.full((4, G, 64, d), float("nan"), dtype=dt, device="cuda")
    v_cache = torch.full((4, G, dv, 64), float("nan"), dtype=dt, device="cuda")
    table = torch.tensor([[3, 3], [2, 0]], dtype=torch.int32, device="cuda")
    ctx = _step_context([0], [n], slots=[1])
    q = ops.sink_qkv_store(rows.cuda(), H, G, d, dv, None, "head_unit", None, None, eps, None, None, 0, k_cache, v_cache, table, ctx, col0=2).cpu()
    r = rows.double()[:, 2:]
    tol = dict(atol=1e-5, rtol=1e-5) if dtype == "float32" else dict(atol=2e-2, rtol=1e-2)
    assert torch.allclose(q.double(), P.unit_rms(r[:, :H * d].reshape(n, H, d), eps), **tol)
    want_k, want_v = P.unit_rms(r[:, H * d:(H + G) * d].reshape(n, G, d), eps), r[:, (H + G) * d:(H + G) * d + G * dv].reshape(n, G, dv)
    for p in range(n):
        page = (2, 0)[p // 64]
        assert torch.allclose(k_cache[page, :, p % 64].cpu().double(), want_k[p], **tol)
        assert torch.allclose(v_cache[page, :, :, p % 64].cpu().double(), want_v[p], **tol)


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,chunk", [(4, 2, 24, 40, 37), (3, 3, 40, 72, 70), (6, 1, 8, 12, None), (16, 2, 64, 32, 130), (6, 2, 32, 96, 64), (5, 5, 9, 15, 100),
                                            (18, 2, 16, 16, 299), (4, 4, 128, 256, 128)])
def test_attention_kernels_far_keys_page_borders_and_chunk_edges(dtype, H, G, d, dv, chunk):
    """Keys and values straight into the pages.  One key is made to stand out (its score far above the others' and above what
    the distance costs) at places that matter: the first position, far back, a page's last and first key, a chunk's first key
    and the last one of the chunk before.  Prompts (the matrix cores in bfloat16) and single tokens (the exact kernel, in slices)."""
    from palm_infra_amd.kernels import ops
    torch.manual_seed(H * 100 + d)
    dt = TORCH[dtype]
    T, scale = 300, 0.3
    per = H // G
    pages = [3, 0, 5, 2, 4]
    table = torch.tensor([[6] * 5, pages], dtype=torch.int32, device="cuda")
    slopes = P.head_slopes(H)
    first = (T - 1) // chunk * chunk if chunk else 0                      # the last query's chunk begins here
    slopes_dev = torch.tensor(slopes, dtype=torch.float32, device="cuda")
    kw = dict(chunked=chunk is not None, slopes=slopes_dev)
    targets = [0, 5, 63, 64, 127, 128, 190, first - 1, first, first + 1, (first + T - 1) // 2, T - 1]
    for target in sorted(set(t for t in targets if 0 <= t < T)):
        k = torch.randn(T, G, d) * 0.3
        v = torch.randn(T, G, dv)
        q = torch.randn(T, H, d) * 0.3
        # the last query points at the target key with a score of some 40 beyond what the distance takes from it
        k[target] = torch.nn.functional.normalize(torch.randn(G, d), dim=-1) * 4.0
        for h in range(H):
            q[T - 1, h] = k[target, h // per] / 16.0 * (40.0 + slopes[h] * (T - 1 - target)) / scale
        q, k, v = (t.to(dt) for t in (q, k, v))
        kc = torch.full((7, G, 64, d), float("nan"), dtype=dt)
        vc = torch.full((7, G, dv, 64), float("nan"), dtype=dt)
        for p in range(T):
            kc[pages[p // 64], :, p % 64] = k[p]
            vc[pages[p // 64], :, :, p % 64] = v[p]
        vc[pages[T // 64], :, :, T % 64:] = 0                              # (beyond the sequence: whatever a page held, made finite here)
        kc[pages[T // 64], :, T % 64:] = 0
        want = P.chunk_softmax_heads(q.double(), k.double(), v.double(), scale, slopes, chunk)
        tol = dict(atol=2e-4, rtol=2e-4) if dtype == "float32" else dict(atol=4e-2, rtol=3e-2)
        for cuts in ([T], [170, 130]):                                     # a prompt of all T tokens, and one in two portions
            got, at = [], 0
            for c in cuts:
                ctx = _step_context([at], [c], slots=[1])
                got.append(ops.sink_attention(q[at:at + c].cuda(), kc.cuda(), vc.cuda(), table, ctx, H, G, d, dv, scale, chunk, None, None, **kw).cpu())
                at += c
            assert torch.allclose(torch.cat(got).double().reshape(T, H, dv), want, **tol), (target, cuts)
        for p in (T - 1, T - 2, first, max(0, first - 1)):                 # single tokens: the exact kernel in slices
            ctx = _step_context([p], [1], slots=[1])
            for slices in (None, 1, 3):
                got = ops.sink_attention_exact(q[p:p + 1].cuda(), kc.cuda(), vc.cuda(), table, ctx, H, G, d, dv, scale, chunk, None, None,
                                               slices=slices, **kw).cpu()
                assert torch.allclose(got.double().reshape(H, dv), want[p], **tol), (target, p, slices)
        # the target decides the last query's output where it is seen, and counts for nothing where it is not
        assert bool((want[T - 1, 0] - v[target, 0].double()).abs().max() < 0.05) == (target >= first), target


SCHEDULES = {"whole": ([[260], [75]], 0), "chunks of 32": ([[260], [75]], 32), "chunks of 40": ([[200, 60], [75]], 40),
             "portions": ([[1, 2, 1, 64, 65, 127], [70, 1, 1, 1, 2]], None)}


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,tau,rank", [(3, 16, 24, 8.0, 5), (1, 40, 130, 1.0, 16), (2, 128, 64, 16.0, 33), (5, 32, 16, 2.5, 1), (2, 24, 70, 4.0, 3), (2, 200, 300, 16.0, 4)])
def test_gla_keeps_a_far_write_in_its_channels_whole_in_portions_and_in_chunks(dtype, H, d, dv, tau, rank):
    """Half of the key channels hardly forget, the others forget quickly: a large write of a far token stays in the first half
    and is gone from the second.  The last query reads each half.  Whole, in portions down to one token, and cut into chunks
    that run side by side; two sequences of unequal lengths in slots that were used before; the decays' inputs and the rows as
    views of wider tensors."""
    from palm_infra_amd.kernels import ops
    torch.manual_seed(d + dv)
    dt = TORCH[dtype]
    lengths, far, eps = [260, 75], 3, 1e-6
    rows = [torch.randn(n, 4 + H * (2 * d + 2 * dv)) * 0.2 for n in lengths]
    r0, k0 = rows[0], 4 + H * d
    half = d // 2
    for h in range(H):
        r0[far, k0 + h * d:k0 + (h + 1) * d] = 4.0                            # the far token's key fills every channel ..
        r0[far, k0 + H * d + h * dv:k0 + H * d + (h + 1) * dv] *= 60.0        # .. with a large value
        r0[258, 4 + h * d:4 + (h + 1) * d] = torch.cat([torch.ones(half), torch.zeros(d - half)])       # reads what hardly forgets
        r0[259, 4 + h * d:4 + (h + 1) * d] = torch.cat([torch.zeros(half), torch.ones(d - half)])       # reads what forgets
    rows = [r.to(dt) for r in rows]
    low = [torch.randn(n, rank + 3) * 0.1 for n in lengths]
    w2 = torch.randn(rank, H * d)
    bias = torch.cat([torch.full((half,), 9.0 + math.log(tau)), torch.full((d - half,), -1.5 * tau)]).repeat(H)
    norm_w = torch.randn(dv) * 0.2 + 1.5
    want, wgt = [], {"a1": torch.eye(rank, dtype=P.F64), "a2": w2.T.double(), "a2.b": bias.double()}
    for r, lo in zip(rows, low):
        n = r.shape[0]
        r = r.double()[:, 4:]
        q, k = r[:, :H * d].reshape(n, H, d) * d ** -0.5, r[:, H * d:2 * H * d].reshape(n, H, d)
        v, g = r[:, 2 * H * d:2 * H * d + H * dv].reshape(n, H, dv), r[:, 2 * H * d + H * dv:]
        a = P.channel_decays(lo.double()[:, 2:2 + rank], wgt, "", tau).reshape(n, H, d)
        o, _ = P.gla_recurrence(q, k, v, a)
        if n == 260:                                                          # the far value is what the one query finds and the other does not
            vf = v[far, 0]
            assert float(torch.nn.functional.cosine_similarity(o[258, 0], vf, dim=0)) > 0.95
            assert abs(float(o[259, 0] @ vf / vf.norm())) < 0.02 * abs(float(o[258, 0] @ vf / vf.norm()))
        want.append((P.unit_rms(o, eps) * norm_w.double()).reshape(n, -1) * P.silu(g))
    tol = dict(atol=5e-4, rtol=5e-4) if dtype == "float32" else dict(atol=3e-2, rtol=3e-2)
    for what, (cuts, chunk) in SCHEDULES.items():
        state = torch.randn(3, H, d, dv, device="cuda")                       # stale from an earlier sequence
        state[1:].zero_()

        def step(ctx, live, fed, counts):
            packed = torch.cat([rows[b][fed[b]:fed[b] + c] for b, c in zip(live, counts)]).cuda()
            lo = torch.cat([low[b][fed[b]:fed[b] + c] for b, c in zip(live, counts)]).cuda()
            return ops.gla(packed, lo[:, 2:2 + rank], w2.cuda(), bias.cuda(), tau, norm_w.cuda(), H, d, dv, d ** -0.5, eps, state, ctx, col0=4, chunk=chunk)

        for b, got in enumerate(_run_schedule(lengths, cuts, [1, 2], step)):
            assert torch.allclose(got, want[b], **tol), (what, b, float((got - want[b]).abs().max()))


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,taps", [(4, 2, 16, 24, 4), (3, 1, 40, 130, 2), (2, 2, 128, 64, 3), (6, 6, 32, 16, 1), (3, 3, 24, 70, 5), (2, 1, 200, 300, 4), (8, 2, 33, 5, 16)])
def test_delta_rule_with_a_decay_a_head_keeps_a_far_write(dtype, H, G, d, dv, taps):
    """Decays near one and small write strengths but for one far token, whose value the queries that point at its key find
    again at the end.  Whole, in portions down to one token (shorter than the convolution reaches back), and in chunks that
    run side by side; two sequences in slots that were used before; rows as columns of wider ones."""
    from palm_infra_amd.kernels import ops
    torch.manual_seed(d + dv)
    dt = TORCH[dtype]
    lengths, far, eps, unit_eps = [260, 75], 20, 1e-6, 1e-6
    C = 2 * G * d + H * dv
    rows = [(torch.randn(n, 3 + C + H * dv + 2)).to(dt) for n in lengths]
    conv = torch.randn(C, taps) * 0.3
    conv[:, -1] += 1.0
    with torch.no_grad():
        key = rows[0][far - taps + 1:far + 1, 3 + G * d:3 + 2 * G * d].clone()
        rows[0][260 - taps:, 3:3 + G * d] = key                                # the last query's window is the far key's
        conv[:G * d] = conv[G * d:2 * G * d]
    ab = [torch.randn(n, 1 + 2 * H) for n in lengths]
    ab[0][:, 1:1 + H] = -5.0 + 0.3 * torch.randn(260, H)
    ab[0][far, 1:1 + H] = 4.0
    a_log, dt_bias = torch.full((H,), -2.0) + 0.2 * torch.randn(H), torch.full((H,), -4.0) + 0.2 * torch.randn(H)
    norm_w = torch.randn(dv) * 0.2 + 1.5
    want = []
    for r, z in zip(rows, ab):
        n = r.shape[0]
        r, z = r.double(), z.double()[:, 1:]
        u = P.silu(P.short_convolution(r[:, 3:3 + C], conv.double()))
        q = P.unit_vectors(u[:, :G * d].reshape(n, G, d)) * d ** -0.5
        k = P.unit_vectors(u[:, G * d:2 * G * d].reshape(n, G, d))
        v = u[:, 2 * G * d:].reshape(n, H, dv)
        g = torch.exp(-torch.exp(a_log.double()) * P.softplus(z[:, H:] + dt_bias.double()))
        o = P.delta_recurrence(q, k, v, torch.sigmoid(z[:, :H]), g)
        if n == 260 and d >= 24 and dv >= 16:
            assert float(torch.nn.functional.cosine_similarity(o[-1, 0], v[far, 0], dim=0)) > 0.5
        want.append((P.unit_rms(o, eps) * norm_w.double()).reshape(n, -1) * P.silu(r[:, 3 + C:3 + C + H * dv]))
    tol = dict(atol=1e-3, rtol=1e-3) if dtype == "float32" else dict(atol=6e-2, rtol=3e-2)
    for what, (cuts, chunk) in SCHEDULES.items():
        state, kept = torch.randn(3, H, d, dv, device="cuda"), torch.randn(3, taps - 1, C, device="cuda")
        state[1:].zero_()
        kept[1:].zero_()

        def step(ctx, live, fed, counts):
            packed = torch.cat([rows[b][fed[b]:fed[b] + c] for b, c in zip(live, counts)]).cuda()
            z = torch.cat([ab[b][fed[b]:fed[b] + c] for b, c in zip(live, counts)]).cuda()
            return ops.delta_head(packed, z[:, 1:], conv.cuda(), kept, a_log.cuda(), dt_bias.cuda(), norm_w.cuda(), H, G, d, dv, d ** -0.5, unit_eps,
                                  eps, state, ctx, col0=3, chunk=chunk)

        for b, got in enumerate(_run_schedule(lengths, cuts, [1, 2], step)):
            assert torch.allclose(got, want[b], **tol), (what, b, float((got - want[b]).abs().max()))
            if taps > 1:
                assert torch.allclose(kept[b + 1].cpu().double(), rows[b][-taps + 1:, 3:3 + C].double(), atol=1e-6), (what, b, "kept inputs")


@gpu
def test_softmax_routing_by_the_groups_largest_against_the_plain_choice():
    """Random logits for several shapes of groups, and rows made so that the group with the largest score differs from the one
    whose two largest sum highest; the kernel's experts and weights against the plain ones, as columns of wider rows.  Logits
    that are no numbers choose experts that exist."""
    from palm_infra_amd.kernels import ops
    torch.manual_seed(3)
    for E, top, groups, keep in ((12, 3, 3, 2), (16, 4, 4, 2), (8, 2, 2, 1), (6, 1, 1, 1), (5, 5, 1, 1), (64, 6, 8, 3), (130, 7, 10, 4), (9, 3, 9, 3), (512, 64, 4, 1)):
        n = 200
        logits = torch.randn(n, E + 3) * 1.5
        r = {"experts": E, "top": top, **({"groups": {"count": groups, "keep": keep}} if groups > 1 else {})}
        if groups > 1 and E // groups > 1:
            size = E // groups
            logits[:50, 2:2 + E] -= 6.0
            logits[:50, 2] = 1.0                                              # one large score in the first group ..
            logits[:50, 2 + size:4 + size] = 0.9                              # .. two nearly as large in the second
        chosen_ref, weight_ref = P.route(logits[:, 2:2 + E].double(), r)
        chosen, weight = ops.moe_route_scored(logits.cuda()[:, 2:2 + E], E, top, None, groups, keep, 1.0, score="softmax", group_score="largest")
        for t in range(n):
            a = dict(zip(chosen[t].tolist(), weight[t].tolist()))
            b = dict(zip(chosen_ref[t].tolist(), weight_ref[t].tolist()))
            assert sorted(a) == sorted(b), (E, t)
            assert all(abs(a[e] - b[e]) < 1e-5 for e in a), (E, t)
    nan = torch.full((2, 8), float("nan"), device="cuda")
    for chosen in (ops.moe_route_scored(nan, 8, 3, None, 2, 1, 1.0, score="softmax", group_score="largest")[0], ops.moe_route(nan, 3)[0]):
        assert int(chosen.min()) >= 0 and int(chosen.max()) < 8


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_capped_experts_for_few_rows_and_many_with_rows_of_other_branches(dtype):
    """The experts alone, with given choices and caps that bite: a decode step's rows (every pair reads its expert itself), a
    prompt's rows (grouped on the device in bfloat16), with none, one or two rows of other branches added; and the shared
    expert's gate over columns of wider rows."""
    from palm_infra_amd.kernels import ops
    torch.manual_seed(11)
    dt = TORCH[dtype]
    E, top, W, F, limit = 6, 2, 48, 24, 0.8
    up, down = (torch.randn(E * 2 * F, W) * W ** -0.5).to(dt), (torch.randn(E * W, F) * F ** -0.5).to(dt)
    tol = dict(atol=1e-4, rtol=1e-4) if dtype == "float32" else dict(atol=5e-2, rtol=4e-2)
    weights = {}
    for e in range(E):
        first = up[e * 2 * F:(e + 1) * 2 * F].double()
        weights.update({f"e{e}.gate": first[:F], f"e{e}.up": first[F:], f"e{e}.down": down[e * W:(e + 1) * W].double()})
    for n in (1, 9, 128, 200):
        h = torch.randn(n, W).to(dt)
        chosen = torch.stack([torch.randperm(E)[:top] for _ in range(n)]).to(torch.int32)
        weight = torch.rand(n, top)
        extra = [torch.randn(n, W).to(dt) for _ in range(2)]
        for add in ([], extra[:1], extra):
            want = sum((y.double() for y in add), torch.zeros(n, W, dtype=P.F64))
            for t in range(n):
                for c in range(top):
                    want[t] += weight[t, c].double() * P.capped_expert(h[t:t + 1].double(), weights, f"e{int(chosen[t, c])}.", limit)[0]
            args = (h.cuda(), up.cuda(), down.cuda(), chosen.cuda(), weight.cuda(), F, "capped_gated", (limit, P.GATE_SLOPE, 1.0), [y.cuda() for y in add])
            if n <= 128:
                assert torch.allclose(ops.moe_experts(*args).cpu().double(), want, **tol), (n, len(add))
            if dtype == "bfloat16":
                assert torch.allclose(ops.moe_grouped(*args).cpu().double(), want, **tol), (n, len(add))
        for ff, col in ((24, 4), (7, 3), (300, 8)):                          # (in steps of four values, and not)
            wide = (torch.randn(n, col + 2 * ff + 5) * 2).to(dt)
            got = ops.capped_gate(wide.cuda()[:, col:col + 2 * ff], limit, P.GATE_SLOPE, 1.0).cpu().double()
            g, u = wide[:, col:col + ff].double().clamp(max=limit), wide[:, col + ff:col + 2 * ff].double().clamp(-limit, limit)
            assert torch.allclose(got, g * torch.sigmoid(P.GATE_SLOPE * g) * (u + 1.0), **tol), (n, ff)


@gpu
def test_branches_with_products_of_their_own_and_a_feed_forward_without_addend():
    """The block of parallel branches without the shared input products, around a feed-forward that knows nothing of addends:
    a model of one such layer put together here, against the same layer with shared products."""
    from palm_infra_amd.config import LayerCall, ModelSpec, PartSpec, joined, tensor
    from palm_infra_amd.engine import Engine, StepEntry
    from palm_infra_amd.weights import random_weights
    W, V, H, d, dv, R, F = 32, 50, 2, 8, 16, 3, 24
    N = ("normal", 0.0, 0.3)
    norm = lambda name: PartSpec("norm", "rms", {"width": W, "eps": 1e-6, "offset": 1.0}, {"weight": tensor(name, (W,), "vector", N)})
    mixer = PartSpec("mixer", "gla", {"hidden_size": W, "num_heads": H, "key_dim": d, "value_dim": dv, "decay_rank": R, "tau": 2.0, "query_scale": 0.5, "eps": 1e-6},
                     {"qkvg": joined(["q", "k", "v", "g"], [(H * d, W), (H * d, W), (H * dv, W), (H * dv, W)], "matrix", N), "low": tensor("a1", (R, W), "matrix", N),
                      "decay_up": tensor("a2", (H * d, R), "vector", N), "decay_bias": tensor("a2.b", (H * d,), "vector", N), "norm": tensor("mn", (dv,), "vector", N),
                      "out": tensor("o", (W, H * dv), "matrix", N)})
    ff = PartSpec("feed_forward", "dense", {"hidden_size": W, "intermediate_size": F, "activation": "gelu_tanh"},
                  {"up": tensor("up", (F, W), "matrix", N), "down": tensor("down", (W, F), "matrix", N)})
    table = tensor("embed", (V, W), "table", ("normal", 0.0, 1.0))
    spec = ModelSpec("toy", V, W, None, PartSpec("embedding", "token_table", {"vocab_size": V, "hidden_size": W}, {"table": table}),
                     (PartSpec("block", "parallel_pre_norm", {"hidden_size": W}, {}, {"norm": norm("n1"), "mixer": mixer, "feed_forward": ff}),), (LayerCall(0), LayerCall(0)),
                     norm("fn"), PartSpec("head", "linear", {"vocab_size": V, "hidden_size": W}, {"weight": table}))
    weights = random_weights(spec, 5, torch.float32, "cuda:0")
    eng = Engine(None, spec, weights, torch.float32, 256)
    w = {name: weights.get(ref).double().cpu() for ref in spec.tensor_refs() for name in ref.names if len(ref.names) == 1}
    qkvg = weights.get(mixer.tensors["qkvg"]).double().cpu()
    for name, rows in (("q", qkvg[:16]), ("k", qkvg[16:32]), ("v", qkvg[32:64]), ("g", qkvg[64:])):
        w[name] = rows
    w["norm"] = w["mn"]
    ids = S.prompts({"vocab": V}, [21], seed=1)[0]
    x = w["embed"][ids]
    for _ in range(2):
        h = P.norm_around_zero(x, w["n1"], 1e-6)
        a = P.channel_decays(h, w, "", 2.0).reshape(21, H, d)
        o, _ = P.gla_recurrence((h @ w["q"].T).reshape(21, H, d) * 0.5, (h @ w["k"].T).reshape(21, H, d), (h @ w["v"].T).reshape(21, H, dv), a)
        z = h @ w["up"].T
        x = x + P.gated_heads(o, w, "", h, 1e-6) + torch.nn.functional.gelu(z, approximate="tanh") @ w["down"].T
    want = P.norm_around_zero(x, w["fn"], 1e-6) @ w["embed"].T
    slot = eng.open()
    got = eng.step([StepEntry(slot, ids[:20], list(range(20)))])
    got = torch.cat([got, eng.step([StepEntry(slot, ids[20:], [0])])])
    eng.close(slot)
    assert_close(got, want, "float32", "branches with products of their own")


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
def test_the_residual_stream_after_every_layer(tmp_path_factory):
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, "A", "float32", graphs=False)
    ids = S.prompts(raw_of("A"), [40], seed=2)[0]
    cfg, w = P.read_model(model_dir(tmp_path_factory, "A", "float32"))
    want, seen = [], []
    P.forward(cfg, w, ids, want)
    originals = {id(b): b.forward for b in eng.model.layers}
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
        for b in eng.model.layers:
            b.forward = originals[id(b)]
    assert len(seen) == len(want) == 5
    for i, (a, b) in enumerate(zip(seen[:-1], want[:-1])):              # (the last layer's sum is made only for the rows that the final norm reads)
        assert torch.allclose(a.cpu().double(), b, atol=2e-4, rtol=1e-4), (i, float((a.cpu().double() - b).abs().max()))


@gpu
@pytest.mark.parametrize("name,dtype", CASES)
def test_prompt_then_every_token_alone_from_the_first(tmp_path_factory, name, dtype):
    """Token-by-token decoding from the very first token (every state starts from zero, the convolution from zeros, the chunk
    from an empty page), through recorded steps, across page borders and chunks; against the whole prompt in one step."""
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
def test_batches_of_unequal_requests_and_reused_slots(tmp_path_factory, name, dtype):
    """Two batches through the same slots and pages: prompts of unequal lengths in one step minus their last tokens, which
    come one a step; a request that has no tokens left ends and gives its slot and pages back at once."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    for round_no, (seed, tails) in enumerate([(6, [0, 1, 9, 3, 20, 5, 2, 11]), (7, [12, 0, 2, 7, 30, 1, 1, 4])]):
        lengths = LENGTHS[name] if round_no == 0 else LENGTHS[name][::-1]
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
                         f"{name} batch {round_no} request {i} ({len(r)} tokens, {tails[i]} one by one)")
        eng.cache.check()
        assert all(g.table.pages.held_count == 0 for g in eng.cache.paged_groups)


@gpu
@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("A", "bfloat16"), ("B", "float32"), ("C", "bfloat16"), ("D", "float32")])
def test_long_decoding(tmp_path_factory, name, dtype):
    """A short prompt, then some hundred tokens one by one over several pages and several chunks, two sequences side by
    side that started at different lengths; a chunked layer gives pages back on the way."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    a, b = S.prompts(raw_of(name), [330, 270], seed=8)
    refs = [reference(tmp_path_factory, name, dtype, a), reference(tmp_path_factory, name, dtype, b)]
    sa, sb = eng.open(), eng.open()
    got = [eng.step([StepEntry(sa, a[:70], [69]), StepEntry(sb, b[:10], [9])])]
    want = [refs[0][69], refs[1][9]]
    for i in range(260):
        got.append(eng.step([StepEntry(sa, [a[70 + i]], [0]), StepEntry(sb, [b[10 + i]], [0])]))
        want += [refs[0][70 + i], refs[1][10 + i]]
    chunked = [g for g in eng.cache.paged_groups if g.table.window]
    assert all(g.table.pages.held_count <= 2 * (g.table.window // 64 + 2) for g in chunked)      # two sequences' chunks, not their lengths
    eng.close(sa)
    eng.close(sb)
    assert_close(torch.cat(got), Rows.joined(want), dtype, f"{name} long decoding")


@gpu
@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("C", "bfloat16")])
def test_a_prompt_longer_than_a_step_takes_at_once(tmp_path_factory, name, dtype):
    """A chunked model cuts a long prompt into pieces between which pages go back; the recurrences' long runs go through in
    chunks of their own; logits on both sides of a piece's edge and at the end."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, name, dtype)
    assert eng.step_tokens_per_seq == 1024
    ids = S.prompts(raw_of(name), [1300], seed=13)[0]
    want = [0, 1, 511, 1023, 1024, 1025, 1200, 1299]
    slot = eng.open()
    got = eng.step([StepEntry(slot, ids, want)])
    more = eng.step([StepEntry(slot, [ids[5]], [0])])                       # and a single token after it
    eng.close(slot)
    ref = reference(tmp_path_factory, name, dtype, ids + [ids[5]])
    assert_close(torch.cat([got, more]), ref[want + [1300]], dtype, f"{name} long prompt")


@gpu
@pytest.mark.parametrize("name", ["A", "D"])
def test_recorded_and_launched_steps_agree(tmp_path_factory, name):
    """Decode steps and a short prompt replayed from HIP graphs against the same steps launched kernel by kernel, several
    replays with other work between them."""
    from palm_infra_amd.engine import StepEntry
    ids = S.prompts(raw_of(name), [90], seed=9)[0]
    outs = []
    for graphs in (True, False):
        eng = engine_for(tmp_path_factory, name, "float32", graphs=graphs)
        assert eng.model.capturable
        got = []
        for _ in range(3):
            slot = eng.open()
            got.append(eng.step([StepEntry(slot, ids[:50], [49])]))
            for t in range(50, 90):
                got.append(eng.step([StepEntry(slot, [ids[t]], [0])]))
                torch.cuda.synchronize()
            eng.close(slot)
        outs.append(torch.cat(got).cpu())
    assert torch.allclose(outs[0], outs[1], atol=1e-5)
    ref = reference(tmp_path_factory, name, "float32", ids)[list(range(49, 90))]
    assert_close(outs[0], Rows.joined([ref] * 3), "float32", f"{name} recorded steps")


@gpu
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_decode_step_of_many_sequences_padded_to_its_bucket(tmp_path_factory, dtype):
    """Nineteen sequences decode side by side (a recorded step of 24 rows, five of them padding): each as if alone."""
    from palm_infra_amd.engine import StepEntry
    eng = engine_for(tmp_path_factory, "D", dtype)
    reqs = S.prompts(raw_of("D"), [3 + i for i in range(19)], seed=21)
    slots = [eng.open() for _ in reqs]
    eng.step([StepEntry(s, r[:-3], []) for s, r in zip(slots, reqs) if len(r) > 3])
    eng.step([StepEntry(s, [r[-3]], []) for s, r in zip(slots, reqs)])
    got = [eng.step([StepEntry(s, [r[at]], [0]) for s, r in zip(slots, reqs)]).cpu() for at in (-2, -1)]
    for s in slots:
        eng.close(s)
    ref = Rows.joined([reference(tmp_path_factory, "D", dtype, r)[at] for at in (-2, -1) for r in reqs])
    assert_close(torch.cat(got), ref, dtype, "nineteen sequences")


@gpu
@pytest.mark.parametrize("name", ["A", "B", "C", "D", "E"])
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
                          "--max-tokens", "320"], input="\n".join(json.dumps(s) for s in steps) + "\n", capture_output=True, text=True, timeout=600)
    assert run.returncode == 0, run.stderr[-2000:]
    assert [ln for ln in run.stdout.splitlines() if ln.startswith("done")] == [f"done {s}" for s in range(11)]
    refs = [reference(tmp_path_factory, "A", "float32", r) for r in reqs]
    first = np.fromfile(out / "0.f32", dtype="<f4").reshape(8, -1)
    want = Rows.joined([refs[i][p] for i, h in enumerate(heads) for p in (0, h - 1)])
    assert_close(torch.from_numpy(first.copy()), want, "float32", "trace step 0")
    fed = list(heads)
    for s in range(1, 11):
        live = [i for i in range(3) if fed[i] < len(reqs[i])]
        if s % 2 and live:
            got = np.fromfile(out / f"{s}.f32", dtype="<f4").reshape(len(live), -1)
            assert_close(torch.from_numpy(got.copy()), Rows.joined([refs[i][fed[i]] for i in live]), "float32", f"trace step {s}")
        else:
            assert not (out / f"{s}.f32").exists()
        for i in live:
            fed[i] += 1
