"""The kernel set of routed experts: both products on the matrix cores, in tiles of 64 and of 128 rows and in the form for
few rows, against the formula in float32, with every activation between them and the weight on either side."""
import pytest
import torch

pytestmark = pytest.mark.gpu
DEV = "cuda:0"


def between(act, pre, F):
    if not act.gated:
        return torch.nn.functional.relu(pre) ** 2 if act.kind == "relu2" else torch.nn.functional.silu(pre)
    g, u = pre[:, :F], pre[:, F:]
    if act.limit is None:
        return torch.nn.functional.silu(g) * u
    g, u = g.clamp(max=act.limit), u.clamp(-act.limit, act.limit)
    return g * torch.sigmoid(act.alpha * g) * (u + act.shift)


@pytest.mark.parametrize("activation", ["silu", "clamped", "relu2"])
@pytest.mark.parametrize("on_input", [False, True])
@pytest.mark.parametrize("n,W,E,top,F", [(9, 64, 5, 2, 48), (40, 96, 12, 3, 64), (100, 64, 3, 2, 272), (400, 128, 4, 2, 136), (700, 320, 6, 4, 32), (257, 64, 1, 1, 64)])
def test_tuned_experts_against_the_formula(activation, on_input, n, W, E, top, F):
    from flambeau_amd.engine import Runtime
    from flambeau_amd.kernels import ops
    from flambeau_amd.kernels.experts import ExpertActivation
    rt = Runtime(DEV, torch.bfloat16, 1024, True)
    ks = rt.kernels("routed_experts")
    act = {"silu": ExpertActivation(True), "clamped": ExpertActivation(True, limit=0.9, alpha=1.5, shift=0.7), "relu2": ExpertActivation(False, "relu2")}[activation]
    g = torch.Generator().manual_seed(n + F)
    mat = lambda r, c: (torch.randn(r, c, generator=g) * 0.2).to(torch.bfloat16).to(DEV)
    up, gate, down = [mat(F, W) for _ in range(E)], [mat(F, W) for _ in range(E)], [mat(W, F) for _ in range(E)]
    x = torch.randn(n, W, generator=g).to(torch.bfloat16).to(DEV)
    z = torch.randn(n, E, generator=g).to(DEV)
    first = ks.prepare(up, gate if act.gated else None)
    second = ks.prepare(down)
    P = n * top
    tile_rows = ks.tile_rows(P, E, first, second)
    packed = first.packed is not None and second.packed is not None
    assert tile_rows == (128 if packed and P >= 48 * E else 64) and (second.packed is not None) == (F % 32 == 0)
    i32 = lambda *s: torch.empty(*s, dtype=torch.int32, device=DEV)
    place, src_row, tiles = i32(P), i32(P), i32(ops.moe_max_tiles(P, E, tile_rows), 4)
    scale, pair_w = torch.empty(P, device=DEV), torch.empty(P, device=DEV)
    ops.moe_route(z, 0, E, top, place, src_row, scale, pair_w, tiles, "softmax", tile_rows=tile_rows)
    expert = torch.full((P,), -1, dtype=torch.long)
    for e, p0, m, _ in tiles.cpu().tolist():
        if e >= 0:
            assert 0 < m <= tile_rows and (expert[p0:p0 + m] == -1).all()
            expert[p0:p0 + m] = e
    assert (expert >= 0).all() and torch.equal(torch.sort(src_row.cpu())[0], torch.arange(n).repeat_interleave(top).int())
    s = torch.softmax(z, dim=1).cpu()
    assert (scale.cpu() - s[src_row.cpu().long(), expert]).abs().max() < 1e-6
    a = torch.full((P, F), float("nan"), dtype=torch.bfloat16, device=DEV)
    ks.first(x, first, act, a, tiles, tile_rows, P, src_row, scale if on_input else None)
    y = torch.full((P, W), float("nan"), device=DEV)
    ks.product(a, second, y, tiles, tile_rows, None, None if on_input else scale)
    xf, sc = x.float().cpu(), scale.cpu()
    want_a, want_y = torch.empty(P, F), torch.empty(P, W)
    for p in range(P):
        e, r = int(expert[p]), int(src_row[p])
        w1 = torch.cat([gate[e], up[e]]) if act.gated else up[e]
        pre = (xf[r] * (sc[p] if on_input else 1.0)) @ w1.float().cpu().T
        want_a[p] = between(act, pre[None], F)[0]
        want_y[p] = want_a[p] @ down[e].float().cpu().T * (1.0 if on_input else sc[p])
    assert (a.float().cpu() - want_a).abs().max() < 2e-2 * want_a.abs().max()
    assert (y.cpu() - want_y).abs().max() < 2e-2 * want_y.abs().max()
