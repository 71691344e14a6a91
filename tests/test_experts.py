"""The routed experts' kernels alone, in every form an expert can have, against a plain sum over the chosen experts in float64:
the kernels for a decode step's rows, the grouped products whose operands cross LDS (sizes in whole cache lines, enough rows
an expert) and those that read their fragments from memory (other sizes, few rows an expert), with uneven choices (an expert
that everybody chose, one that nobody did), and rows of other branches added."""
import math

import pytest
import torch

gpu = pytest.mark.gpu
F64 = torch.float64
CAP = (1.3, 1.702, 1.0)


def plain_expert(form, z, ff):
    if form == "gelu":
        return 0.5 * z * (1 + torch.erf(z / math.sqrt(2.0)))
    if form == "relu_squared":
        return torch.clamp(z, min=0.0) ** 2
    g, u = z[..., :ff], z[..., ff:]
    if form == "gated_silu":
        return g * torch.sigmoid(g) * u
    limit, slope, shift = CAP
    g, u = torch.clamp(g, max=limit), torch.clamp(u, -limit, limit)
    return g * torch.sigmoid(slope * g) * (u + shift)


def plain_mixture(form, h, up, down, chosen, weight, ff):
    E, W = down.shape[0] // h.shape[1], h.shape[1]
    per = up.shape[0] // E
    out = torch.zeros(h.shape, dtype=F64)
    for e in range(E):
        for c in range(chosen.shape[1]):
            rows = (chosen[:, c] == e).nonzero().flatten()
            if rows.numel():
                z = h[rows].double() @ up[e * per:(e + 1) * per].double().T
                out[rows] += weight[rows, c, None].double() * (plain_expert(form, z, ff) @ down[e * W:(e + 1) * W].double().T)
    return out


def case(form, E, top, W, F, n, uneven, seed, dt):
    g = torch.Generator().manual_seed(seed)
    per = (2 if form in ("gated_silu", "capped_gated") else 1) * F
    up, down = (torch.randn(E * per, W, generator=g) * W ** -0.5).to(dt), (torch.randn(E * W, F, generator=g) * F ** -0.5).to(dt)
    h = torch.randn(n, W, generator=g).to(dt)
    chosen = torch.stack([torch.randperm(E - 1 if uneven and E > top else E, generator=g)[:top] for _ in range(n)]).to(torch.int32)
    if uneven:                                    # expert 0 is everybody's (once a token), the last one nobody's
        chosen = torch.where(chosen == 0, chosen[:, :1], chosen)
        chosen[:, 0] = 0
    weight = torch.rand(n, top, generator=g)
    return h, up, down, chosen, weight


@gpu
@pytest.mark.parametrize("form", ["gated_silu", "gelu", "capped_gated", "relu_squared"])
@pytest.mark.parametrize("E,top,W,F,n,uneven", [(4, 2, 64, 64, 300, False), (3, 1, 128, 192, 131, True), (8, 3, 320, 128, 400, True), (5, 5, 192, 320, 150, False),
                                                (2, 1, 64, 448, 700, False), (33, 2, 128, 64, 160, False), (6, 2, 72, 40, 200, True)])
def test_grouped_products(form, E, top, W, F, n, uneven):
    from palm_infra_amd.kernels import ops
    h, up, down, chosen, weight = case(form, E, top, W, F, n, uneven, E * n + F, torch.bfloat16)
    want = plain_mixture(form, h, up, down, chosen, weight, F)
    args = [t.cuda() for t in (h, up, down, chosen, weight)]
    got = ops.moe_grouped(*args, F, form, CAP if form == "capped_gated" else ops.NO_CAP)
    tol = 0.02 * float(want.abs().max())
    assert float((got.cpu().double() - want).abs().max()) <= tol
    y = torch.randn(n, W).to(torch.bfloat16)
    more = ops.moe_grouped(*args, F, form, CAP if form == "capped_gated" else ops.NO_CAP, add=[y.cuda()])
    assert torch.allclose(more - got, y.cuda().float(), atol=1e-4)


@gpu
@pytest.mark.parametrize("form", ["gated_silu", "gelu", "capped_gated", "relu_squared"])
@pytest.mark.parametrize("E,top,W,F,shared", [(4, 2, 64, 64, 40), (3, 1, 72, 24, None), (33, 4, 320, 264, 264), (5, 5, 8, 8, 16), (512, 3, 48, 16, None), (6, 2, 2056, 520, 1032)])
def test_few_rows(form, E, top, W, F, shared):
    """One row, a decode batch's rows, and as many as a recorded step holds: both kernels for few rows, with a shared expert and
    with planes of partial sums."""
    from palm_infra_amd.kernels import ops
    cap = CAP if form == "capped_gated" else ops.NO_CAP
    for n, uneven in ((1, False), (8, False), (17, True), (40, False), (70, True), (128, True), (128, False)):
        h, up, down, chosen, weight = case(form, E, top, W, F, n, uneven, E + F + n, torch.bfloat16)
        want = plain_mixture(form, h, up, down, chosen, weight, F)
        extra = None
        if shared:
            per = (2 if form in ("gated_silu", "capped_gated") else 1) * shared
            extra = ((torch.randn(per, W) * W ** -0.5).to(torch.bfloat16), (torch.randn(W, shared) * shared ** -0.5).to(torch.bfloat16))
            want += plain_expert(form, h.double() @ extra[0].double().T, shared) @ extra[1].double().T
            extra = tuple(t.cuda() for t in extra)
        args = [t.cuda() for t in (h, up, down, chosen, weight)]
        tol = 0.02 * float(want.abs().max())
        got = ops.moe_few(*args, F, form, cap, shared=extra)
        assert float((got.cpu().double() - want).abs().max()) <= tol, (n, uneven)
        again = ops.moe_few(*args, F, form, cap, shared=extra)
        assert torch.equal(got, again)
        planes = ops.moe_few(*args, F, form, cap, shared=extra, planes_ok=True)
        planes = planes if planes.dim() == 2 else planes.sum(0)
        assert torch.allclose(planes, got, atol=1e-4 * float(want.abs().max()), rtol=1e-4)
        exact = ops.moe_experts(*args, F, form, cap, shared=extra)
        assert float((exact.cpu().double() - want).abs().max()) <= tol, (n, uneven)
        y = [torch.randn(n, W).to(torch.bfloat16).cuda() for _ in range(2)]
        more = ops.moe_few(*args, F, form, cap, add=y, shared=extra)
        assert torch.allclose(more, got + y[0].float() + y[1].float(), atol=1e-3, rtol=1e-4)
