"""Fipitar on the GPU against the plain implementation: every mechanism alone, the layers one by one, and whole
models in every cutting (whole prompts, single tokens, portions down to two tokens, mixed batches over a small
poisoned pool whose pages and slots are used again), in 32-bit and in bfloat16, at sizes of the tests' own."""
import json

import numpy as np
import pytest
import torch

import plain_fipitar as pf
import replay_helpers as rh
from fipitar_configs import CONFIGS, left, long_memory, read_model, right, rot, write_model
from test_bugidra_gpu import CUTS, TOL, _x, run_mixer, runner_for
from test_bugidra_gpu import bound_part as _bound_part
from test_kuvidra_gpu import close, make_rt, make_step

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    base = tmp_path_factory.mktemp("fipitar")
    out = {}
    for name in CONFIGS:
        for store in DTYPES:
            out[(name, store)] = write_model(name, base / f"{name}-{store}", store)
    for store in DTYPES:          # (weights are stored in the dtype they are run in: the plain side reads the same numbers)
        out[("sharp", store)] = write_model("A", base / f"A-sharp-{store}", store, sharpen=6.0)
        out[("memory", store)] = write_model("A", base / f"A-memory-{store}", store, edit=long_memory)
    return out


_refs = {}


def reference(d, reqs):
    out = {}
    cfg = t = None
    for rid, toks in reqs.items():
        key = (str(d), tuple(toks))
        if key not in _refs:
            if cfg is None:
                cfg, t = read_model(d)
            _refs[key] = pf.forward(cfg, t, toks)
        out[rid] = _refs[key]
    return out


dev = lambda v: v.to(DEV).contiguous() if v is not None else None


def bound_part(*args, **kw):
    part, plain = _bound_part(*args, **kw)
    return part, {k.replace("_norm", ".norm") if k.endswith("_norm") else k: v for k, v in plain.items()}


# ---------------------------------------------------------------- each mechanism alone: around the recurrences
@pytest.mark.parametrize("C,taps,H", [(40, 3, 4), (37, 1, 1), (64, 5, 300), (300, 2, 7), (2052, 4, 16), (36, 7, 2)])
def test_the_convolution_ahead_of_a_state_space_walk_alone(C, taps, H):
    """Two requests side by side, cut into portions shorter and longer than the convolution reaches, in slots whose
    neighbours hold NaN; rows without a slot write nothing; not a bit depends on the cutting; the steps and decays too."""
    from flambeau_amd.kernels import ops
    g = torch.Generator().manual_seed(C + taps)
    n, at_ring = 40, 8
    width = 4 + C + H
    xs = [torch.randn(n, width, generator=g) * 2 for _ in range(2)]
    w, b, dtb, alog = torch.randn(C, taps, generator=g), torch.randn(C, generator=g), torch.randn(H, generator=g) * 3, torch.randn(H, generator=g)
    wt = dev(w.t())
    d = lambda v: v.double().numpy()
    want = [pf.silu(pf.causal_convolution(d(x)[:, 4:4 + C], d(w), d(b))) for x in xs]
    dt = [pf.softplus(d(x)[:, 4 + C:] + d(dtb)) for x in xs]
    results = []
    for cuts in ([40], [1] * 40, [2, 1, 3, 7, 2, 1, 1, 8, 2, 13], [5, 35], [33, 1, 6]):
        state = torch.full((5, at_ring + -(-taps * C // 4) * 4), float("nan"), device=DEV)
        state[3], state[1] = 0.0, 0.0
        got = [[], []]
        at = 0
        for k in cuts:
            step = make_step([(at, k), (at, k)], 8, 20, slots=[3, 1])
            p = dev(torch.cat([x[at:at + k] for x in xs]))
            out, gates = torch.full((2 * k, C), float("nan"), device=DEV), torch.full((2 * k, 2 * H), float("nan"), device=DEV)
            for _ in range(2 if k == 1 else 1):                            # (a step of one token writes places it does not read)
                ops.conv_steps(p, 4, wt, dev(b), state, at_ring, step, out, 4 + C, H, dev(dtb), dev(alog), gates)
            both = torch.cat([out, gates], dim=1).double().cpu().numpy()
            got[0].append(both[:k]); got[1].append(both[k:])
            at += k
        assert torch.isnan(state[[0, 2, 4]]).all() and (state[[1, 3], :at_ring] == 0).all()
        results.append([np.concatenate(x) for x in got])
        for a, y, s in zip(results[-1], want, dt):
            assert np.abs(a[:, :C] - y).max() < 2e-6 * np.abs(y).max(), cuts
            assert np.abs(a[:, C + H:] - s).max() < 1e-6 * np.abs(s).max() and np.abs(a[:, C:C + H] - np.exp(-np.exp(d(alog)) * s)).max() < 2e-6
        assert all(np.array_equal(a, b_) for a, b_ in zip(results[-1], results[0])), cuts
    state = torch.full((2, at_ring + -(-taps * C // 4) * 4), 3.0, device=DEV)     # rows that pad a batch: no slot, nothing is read or written
    step = make_step([(9, 1), (0, 1)], 8, 20, slots=[-1, -1])
    out = torch.empty(2, C, device=DEV)
    ops.conv_steps(dev(xs[0][:2]), 4, wt, dev(b), state, at_ring, step, out, 4 + C, H, dev(dtb), dev(alog), torch.empty(2, 2 * H, device=DEV))
    assert (state == 3.0).all() and torch.isfinite(out).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W,parts", [(40, 1), (37, 37), (256, 2), (1024, 1), (3000, 3), (8192, 2), (9000, 1), (12288, 1)])
def test_a_gate_and_a_norm_in_parts_alone(dtype, W, parts):
    """Parts that are held in registers and parts that are not; the output as columns of a wider tensor."""
    from flambeau_amd.kernels import ops
    g = torch.Generator().manual_seed(W)
    n, eps = 5, 3e-4
    y, gate, w = torch.randn(n, W, generator=g) * 0.02, torch.randn(n, W + 9, generator=g) * 2, 1 + 0.3 * torch.randn(W, generator=g)
    both = torch.full((n, W + 16), -7.0, dtype=TORCH[dtype], device=DEV)
    ops.gated_group_norm(dev(y), dev(gate), 6, dev(w), both[:, 8:8 + W], parts, eps)
    v = (y.double().numpy() * pf.silu(gate.double().numpy()[:, 6:6 + W])).reshape(n, parts, -1)
    want = (v / np.sqrt((v * v).mean(axis=-1, keepdims=True) + eps)).reshape(n, W) * w.double().numpy()
    got = both.double().cpu().numpy()
    assert np.abs(got[:, 8:8 + W] - want).max() < (3e-6 if dtype == "float32" else 6e-3) * np.abs(want).max()
    assert (got[:, :8] == -7).all() and (got[:, 8 + W:] == -7).all()


@pytest.mark.parametrize("W", [37, 40, 256, 516, 1000, 2048, 4096, 5000, 6002, 16384, 20000])
def test_a_norm_on_its_way_into_the_stream_alone(W):
    """Rows that are held in registers by blocks of every size and rows that are not: the same bits in a step of few rows and
    of many, the stream in 32-bit and in the compute dtype beside it."""
    from flambeau_amd.kernels import ops
    g = torch.Generator().manual_seed(W)
    n, eps = 300, 3e-4
    y, x = torch.randn(n, W, generator=g) * 3 + 0.5, torch.randn(n, W, generator=g)
    w, b = 1 + 0.3 * torch.randn(W, generator=g), torch.randn(W, generator=g)
    want = x.double().numpy() + pf.layer_norm(y.double().numpy(), w.double().numpy(), b.double().numpy(), eps)
    for bias in (b, None):
        outs = []
        for rows in (n, 3):
            r, cast = dev(x[:rows]), torch.empty(rows, W, dtype=torch.bfloat16, device=DEV)
            ops.layernorm_add(dev(y[:rows]), dev(w), dev(bias), r, eps, cast=cast)
            assert torch.equal(cast, r.to(torch.bfloat16))
            ref = want[:rows] - (0 if bias is not None else b.double().numpy())
            assert np.abs(r.double().cpu().numpy() - ref).max() < 3e-6 * np.abs(want).max()
            outs.append(r)
        assert torch.equal(outs[0][:3], outs[1])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,N,R,tau", [(1, 30, 5, 4.0), (16, 700, 1, 1.0), (17, 513, 64, 16.0), (50, 33, 200, 0.5)])
def test_a_forget_gate_of_low_rank_alone(dtype, n, N, R, tau):
    """sigmoid(z)^(1 / tau) for steps of few and of many tokens, where it is near one and near zero: one minus the gate keeps
    its digits."""
    from flambeau_amd.kernels import ops
    g = torch.Generator().manual_seed(N)
    x, w, b = torch.randn(n, R + 3, generator=g), torch.randn(N, R, generator=g).to(TORCH[dtype]), torch.randn(N, generator=g) * 12
    got = ops.lowrank_gate(dev(x), 2, dev(w), dev(w.t()), dev(b), tau, torch.empty(n, N, device=DEV)).double().cpu().numpy()
    z = x.double().numpy()[:, 2:2 + R] @ w.double().numpy().T + b.double().numpy()
    want = pf.sigmoid(z) ** (1 / tau)
    assert np.abs(got - want).max() < 1e-5
    near = (1 - want < 1e-2) & (1 - want > 1e-4)
    assert near.any() and np.abs((1 - got[near]) / (1 - want[near]) - 1).max() < 2e-2
    plain = ops.lowrank_gate(dev(x), 2, dev(w), dev(w.t()), None, tau, torch.empty(n, N, device=DEV)).double().cpu().numpy()
    assert np.abs(plain - pf.sigmoid(z - b.double().numpy()) ** (1 / tau)).max() < 1e-5


# ---------------------------------------------------------------- the recurrent mixers
def gla_spec(W, H, D, Dv, R, tau, eps):
    from flambeau_amd.parts import PartSpec
    return PartSpec("gated_linear_attention", dict(hidden_size=W, n_heads=H, head_dim=D, value_dim=Dv, decay_rank=R, tau=tau, eps=eps))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("bias", [0.0, 8.0, -6.0])
@pytest.mark.parametrize("H,D,Dv,R,tau", [(3, 10, 7, 4, 4.0), (1, 1, 1, 1, 1.0), (2, 65, 33, 3, 16.0), (4, 32, 48, 16, 2.0), (2, 130, 16, 8, 16.0), (1, 300, 20, 5, 8.0)])
def test_gated_linear_attention_alone(dtype, H, D, Dv, R, tau, bias):
    """Memories that last for the whole sequence, for some tokens and hardly at all; whole, in portions and token by token."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype)
    W, n, eps = 40, 90, 2e-5
    mixer, plain = bound_part(MIXERS, gla_spec(W, H, D, Dv, R, tau, eps), dtype, rt, seed=H + D, fix={"a2.bias": lambda v: v + bias})
    x = _x(n, W, dtype, 5)
    m = dict(heads=H, dim=D, vdim=Dv, tau=tau)
    want = pf.gated_linear_attention(x.double().numpy(), m, plain, "m.", eps)
    if bias > 0 and D > 1:                            # the first token is still felt by the last
        other = x.clone(); other[0] = 0.0
        assert np.abs(pf.gated_linear_attention(other.double().numpy(), m, plain, "m.", eps)[-1] - want[-1]).max() > 1e-3 * np.abs(want).max()
    for cuts in CUTS:
        got = run_mixer(mixer, rt, x, cuts)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts


def ssd_spec(W, m, eps):
    from flambeau_amd.parts import PartSpec
    return PartSpec("state_space", dict(hidden_size=W, n_heads=m["heads"], value_dim=m["vdim"], state_dim=m["state"], n_groups=m["groups"],
                                        conv_taps=m["conv"], norm_parts=m["norm_groups"], eps=eps))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("slow", [False, True])
@pytest.mark.parametrize("m", [right(4, 6, 10, 2, 4, 3), right(1, 1, 1, 1, 1, 1), right(3, 5, 7, 3, 2, 5), right(8, 16, 64, 2, 4, 1), right(6, 33, 20, 1, 3, 2),
                               right(2, 64, 200, 2, 6, 4), right(12, 8, 300, 4, 5, 12)])
def test_the_state_space_mixer_alone(dtype, m, slow):
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype)
    W, n, eps = 40, 90, 2e-5
    fix = {"A_log": (lambda v: v * 0 - 5.0) if slow else (lambda v: v)}
    mixer, plain = bound_part(MIXERS, ssd_spec(W, m, eps), dtype, rt, seed=m["heads"] + m["state"], fix=fix)
    x = _x(n, W, dtype, 6)
    want = pf.state_space(x.double().numpy(), m, plain, "m.", eps)
    for cuts in CUTS:
        got = run_mixer(mixer, rt, x, cuts)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts


# ---------------------------------------------------------------- latent attention with neighbours turned and a sink
def latent_spec(W, H, D, Dr, Dv, Rq, R, scale, eps, r):
    from flambeau_amd.models.fipitar import _position
    from flambeau_amd.config.fipitar import RotaryConfig, RotaryScaling
    from flambeau_amd.parts import PartSpec
    cfg = RotaryConfig(r["base"], r["dims"], RotaryScaling(**r["scaling"]) if "scaling" in r else None)
    return PartSpec("latent_attention", dict(hidden_size=W, n_heads=H, head_dim=D, value_dim=Dv, q_rank=Rq, kv_rank=R, scale=scale, eps=eps, gated=False,
                                             rot_dim=Dr, position=_position(cfg, Dr, "interleaved"), sink=True))


LATENT_SHAPES = [
    # H, D, Dr, Dv, Rq, R, scaling
    (3, 10, 6, 12, 14, 24, (4.0, 20, 8.0, 1.0)), (1, 7, 2, 5, 9, 150, None), (6, 4, 8, 4, 4, 64, (2.0, 64, 32.0, 1.0)), (2, 16, 10, 16, 8, 33, None),
    # sizes that the matrix-core kernels take, all three or some of them
    (20, 32, 32, 48, 24, 96, (8.0, 64, 16.0, 2.0)), (4, 64, 16, 16, 40, 160, None), (16, 8, 64, 32, 8, 32, (16.0, 50, 4.0, 1.0)), (2, 96, 24, 16, 16, 512, None),
    (40, 40, 34, 16, 24, 256, (3.0, 4096, 32.0, 1.0)), (36, 32, 64, 16, 24, 512, None), (17, 24, 32, 32, 24, 128, (8.0, 256, 8.0, 1.0)), (3, 24, 70, 16, 16, 64, None),
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,Dr,Dv,Rq,R,scaling", LATENT_SHAPES)
def test_latent_attention_alone(dtype, H, D, Dr, Dv, Rq, R, scaling):
    """Both latents, the folded keys, the rotated parts of queries and keys and a sink that weighs as much as some keys, whole
    and in portions that cross page borders and the kernels' chunks."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype)
    W, n, eps, scale = 40, 150, 2e-5, 0.4 / max(1, R / 64)
    r = rot(Dr, 60.0, scaling)
    mixer, plain = bound_part(MIXERS, latent_spec(W, H, D, Dr, Dv, Rq, R, scale, eps, r), dtype, rt, seed=H + D, fix={"sink": lambda v: v * 4 + 2.0})
    assert mixer.graph_safe and mixer.replayable and "g.weight" not in mixer.tensors()
    x = _x(n, W, dtype, 5)
    m = dict(heads=H, dim=D, rot_dim=Dr, vdim=Dv, kv_rank=R, scale=scale, rot=r)
    h = x.double().numpy()
    want = pf.latent_attention(h, m, plain, "m.", eps)
    scale_of = np.abs(want).max()
    other = pf.latent_attention(h, m, dict(plain, **{"m.sink": plain["m.sink"] * 0 - 99.0}), "m.", eps)
    assert np.abs(other[:5] - want[:5]).max() > 0.05 * scale_of               # the sink matters
    other = pf.latent_attention(h, dict(m, rot=dict(r, base=r["base"] * 3)), plain, "m.", eps)
    assert Dr == 2 or np.abs(other - want).max() > 1e-3 * scale_of            # and so does the rotation
    for cuts in ([n], [60, 5, 1, 1, 2, 30, 2, 6, 1, 42], [1] * 90 + [60]):
        got = run_mixer(mixer, rt, x, cuts, page_size=16 if H > 3 else 8)
        assert np.abs(got - want).max() < TOL[dtype] * scale_of, cuts


@pytest.mark.parametrize("H,R,tail,ps", [(20, 128, 32, 16), (5, 128, 64, 32), (32, 256, 64, 16), (64, 256, 0, 32), (70, 512, 64, 16), (33, 512, 0, 16),
                                         (20, 96, 64, 16), (17, 192, 32, 16)])
def test_the_matrix_core_kernels_of_latent_attention_with_a_sink(H, R, tail, ps):
    """All forms (keys shared by a block, dealt out to its waves, a wave each, in parts that are joined) against the float
    kernel: unequal requests over a pool that holds NaN wherever nothing was written; sinks far below, among and far above
    the scores; one (query, key) score per request stands out."""
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.kernels import latent_attention as la
    from flambeau_amd.kernels import ops
    from flambeau_amd.parts import PagedRowSpec
    n_pages, K = -(-1600 // ps), R + tail
    store = CacheStorage([PagedRowSpec(K, 0, R)], [None], torch.device(DEV), torch.bfloat16, n_pages=n_pages, page_size=ps, max_slots=4)
    pool = store.pools[0][0]                                                # [pages, ps * (K + R)]
    g = torch.Generator().manual_seed(H + R)
    seqs = [(0, 150), (300, 7), (63, 1), (122, 70)]
    step = make_step(seqs, ps, n_pages)
    pool.fill_(float("nan"))
    for s, (st, q) in enumerate(seqs):
        for j in range(st + q):
            page, r = int(step.block_tables[0][s, j // ps]), j % ps
            v = torch.randn(K, generator=g).to(torch.bfloat16).to(DEV) * 0.7
            pool[page, r * K:(r + 1) * K] = v
            pool[page, ps * K:].view(R, ps)[:, r] = v[:R]
    n = step.n_tokens
    qa = (torch.randn(n, H, K, generator=g) * 0.4).to(torch.bfloat16).to(DEV)
    at = 0
    for s, (st, q) in enumerate(seqs):                                      # the request's last query points at its first key
        page = int(step.block_tables[0][s, 0])
        qa[at + q - 1] = pool[page, :K]
        at += q
    qa = qa.view(n, H * K).contiguous()
    sink = dev(torch.tensor([[-1e4, -2.0, 0.0, 3.0, 9.0, 1e4][h % 6] for h in range(H)]))
    cache = store.entries[0].kv
    args = (cache, step.positions, step.tok_seq, step.block_tables[0], H, 0.25, 0)
    want = ops.latent_attention(qa.float(), torch.empty(n, H * R, device=DEV), *args, sink=sink)
    bare = ops.latent_attention(qa.float(), torch.empty(n, H * R, device=DEV), *args)
    w3, b3 = want.view(n, H, R), bare.view(n, H, R)
    assert torch.equal(w3[:, 0], b3[:, 0]) and (H < 6 or (w3[:, 5] == 0).all())               # (a sink far below changes nothing, one far above takes all)
    assert w3[:, 3].norm() < 0.98 * b3[:, 3].norm()
    nan = lambda: torch.full((n, H * R), float("nan"), device=DEV)
    tiles = torch.tensor(la.shared_tiles(step.host, -(-H // 16)), dtype=torch.int32, device=DEV)
    rows = n * -(-H // 16) * 8 * 16
    po, pml = torch.empty(rows, R, device=DEV), torch.empty(rows, 2, device=DEV)
    for form, got in [("shared", la.latent_attention_shared(qa, nan(), *args, tiles, sink=sink)),
                      ("dealt", la.latent_attention_mfma(qa, nan(), *args, dealt=True, sink=sink)),
                      ("wave", la.latent_attention_mfma(qa, nan(), *args, sink=sink)),
                      ("dealt in parts", la.latent_attention_mfma(qa, nan(), *args, n_split=8, part_o=po, part_ml=pml, dealt=True, sink=sink)),
                      ("waves in parts", la.latent_attention_mfma(qa, nan(), *args, n_split=8, part_o=po, part_ml=pml, sink=sink))]:
        assert torch.isfinite(got).all(), form
        assert (got - want).abs().max().item() < 1e-2 * want.abs().max().item(), form


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R", [64, 512, 96])
def test_latent_attention_over_long_contexts(dtype, R):
    """1,400 tokens: keys in many chunks and, for single tokens behind them, in many parts; the sink counts once."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype, max_tokens=1536)
    W, n, eps, H, D, Dr, Dv, Rq = 24, 1400, 1e-5, 4, 32, 16, 16, 16
    r = rot(Dr, 1000.0, (8.0, 256, 16.0, 1.0))
    scale = 2.4 / R ** 0.5
    mixer, plain = bound_part(MIXERS, latent_spec(W, H, D, Dr, Dv, Rq, R, scale, eps, r), dtype, rt, seed=R, fix={"sink": lambda v: v + 7.0})
    x = _x(n, W, dtype, 4)
    want = pf.latent_attention(x.double().numpy(), dict(heads=H, dim=D, rot_dim=Dr, vdim=Dv, kv_rank=R, scale=scale, rot=r), plain, "m.", eps)
    for cuts in ([n], [1300, 60, 17] + [1] * 23, [900, 400, 100]):
        assert sum(cuts) == n
        got = run_mixer(mixer, rt, x, cuts, page_size=16, n_pages=100)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts[:4]


# ---------------------------------------------------------------- grouped attention: heads normed first, a cap, a sink, a gate per head
def grouped_spec(W, m, eps, **more):
    from flambeau_amd.config.fipitar import RotaryConfig
    from flambeau_amd.models.fipitar import _position
    from flambeau_amd.parts import PartSpec
    r = m.get("rot")
    position = _position(RotaryConfig(r["base"], r["dims"]) if r else None, m["dim"], "half")
    return PartSpec("normed_gqa_attention", dict(dict(hidden_size=W, n_heads=m["heads"], n_kv_heads=m["kv_heads"], head_dim=m["dim"], value_dim=m["vdim"],
                                                      scale=m["scale"], position=position, qk_norm="head_gain_first", eps=eps, softcap=m.get("softcap"),
                                                      gate="sigmoid", gate_per="head", sink=0.0), **more))


GROUPED = [left(6, 2, 12, 9, 0.4, 5.0, rot(8)), left(1, 1, 5, 5, 0.9), left(3, 3, 7, 15, 0.5, 2.0, rot(2, 30.0)), left(8, 2, 64, 40, 0.15, 10.0, rot(32, 2500.0)),
           left(34, 2, 32, 32, 0.2, None, rot(32, 700.0)), left(4, 4, 24, 56, 0.2, 30.0, rot(24, 400.0)), left(4, 1, 128, 128, 0.1, 8.0, rot(128, 1e4)),
           left(10, 5, 96, 72, 0.1, 3.0, rot(48)), left(2, 1, 200, 40, 0.1, 20.0)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", GROUPED)
def test_grouped_attention_alone(dtype, m):
    """Norms with a gain ahead of the rotation, the cap, one added to the denominator and a gate per head, whole, in portions
    and token by token."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype)
    W, n, eps = 40, 150, 2e-5
    mixer, plain = bound_part(MIXERS, grouped_spec(W, m, eps), dtype, rt, seed=m["heads"] + m["dim"])
    x = _x(n, W, dtype, 5)
    h = x.double().numpy()
    want = pf.grouped_attention(h, m, plain, "m.", eps)
    assert "sink" not in mixer.tensors() and mixer.tensors()["g.weight"].shape == (m["heads"], W)
    for cuts in ([n], [60, 5, 1, 1, 2, 30, 2, 6, 1, 42], [1] * 90 + [60]):
        got = run_mixer(mixer, rt, x, cuts, page_size=16)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts


def test_the_order_of_norm_and_rotation_and_the_sink_show():
    """Norm behind the rotation, or no sink, or a learned one of another size: other numbers, beyond any rounding."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt("float32")
    W, n, eps, m = 40, 60, 2e-5, left(4, 2, 16, 12, 0.5, 6.0, rot(16, 20.0))
    x = _x(n, W, "float32", 5)
    outs = {}
    for name, more in dict(own={}, behind=dict(qk_norm="head_gain"), none=dict(sink=None), learned=dict(sink="learned"), wide=dict(gate_per="value")).items():
        mixer, plain = bound_part(MIXERS, grouped_spec(W, m, eps, **more), "float32", rt, seed=3, fix={"sink": lambda v: v * 0})
        outs[name] = run_mixer(mixer, rt, x, [n])
    top = np.abs(outs["own"]).max()
    assert np.array_equal(outs["own"], outs["learned"])                     # (a learned sink of zero is the fixed one)
    assert all(np.abs(outs[k] - outs["own"]).max() > 1e-2 * top for k in ("behind", "none", "wide"))
    with pytest.raises(ValueError):
        MIXERS.create(grouped_spec(W, m, eps, sink="fixed"))
    with pytest.raises(ValueError):
        MIXERS.create(grouped_spec(W, m, eps, gate_per="layer"))


@pytest.mark.parametrize("cap", [0.0, 4.0])
@pytest.mark.parametrize("H,G,D,ps", [(8, 2, 64, 16), (4, 4, 128, 16), (34, 2, 32, 32), (6, 3, 128, 64), (2, 1, 256, 16)])
def test_the_tuned_attention_kernels_with_a_sink(H, G, D, ps, cap):
    """The split-K kernel of single rows and the tiled one of portions, with and without parts of the keys, against the plain
    kernel: unequal requests over a pool that holds NaN wherever nothing was written, sinks far below, among and far above the
    scores."""
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.kernels import ops, tuned
    from flambeau_amd.parts import PagedKVSpec
    rt = make_rt("bfloat16", max_tokens=1024)
    n_pages = -(-9000 // ps)
    store = CacheStorage([PagedKVSpec(G, D)], [None], torch.device(DEV), torch.bfloat16, n_pages=n_pages, page_size=ps, max_slots=6)
    kv = store.entries[0].kv
    g = torch.Generator().manual_seed(H + D)
    for seqs in ([(0, 150), (300, 7), (63, 1), (0, 1), (122, 70)], [(1500, 1), (700, 1)], [(1000, 64), (7, 1)], [(2048, 40)]):
        kv.pool.fill_(float("nan"))
        step = make_step(seqs, ps, n_pages)
        step.extra.update({k: torch.tensor(a, dtype=torch.int32, device=DEV)
                           for k, a in tuned.attention_metadata(step.host, [(tuned.decode_blocks_per_row(H, G), 0)]).items()})
        for s, (st, q) in enumerate(seqs):
            k, v = (torch.randn(st + q, G, D, generator=g).to(torch.bfloat16).to(DEV) for _ in range(2))
            for b in range(-(-(st + q) // ps)):
                page, lo, hi = int(step.block_tables[0][s, b]), b * ps, min((b + 1) * ps, st + q)
                kv.pool[page, 0, :, :hi - lo] = k[lo:hi].transpose(0, 1)
                kv.pool[page, 1].view(G, D, ps)[:, :, :hi - lo] = v[lo:hi].permute(1, 2, 0)
        n = step.n_tokens
        q = torch.randn(n, H * D, generator=g).to(torch.bfloat16).to(DEV)
        sink = dev(torch.tensor([[-1e4, -1.0, 0.0, 2.0, 6.0, 1e4][h % 6] for h in range(H)]))
        scale = 1.5 / D ** 0.5
        out = lambda: torch.full((n, H * D), float("nan"), dtype=torch.bfloat16, device=DEV)
        want = ops.attn_plain(q, out(), kv, step.positions, step.tok_seq, step.block_tables[0], H, scale, 0, softcap=cap, sink=sink).float()
        got = tuned.attention(rt, q, out(), kv, step, step.block_tables[0], H, scale, 0, softcap=cap, sink=sink).float()
        bare = tuned.attention(rt, q, out(), kv, step, step.block_tables[0], H, scale, 0, softcap=cap).float()
        assert torch.isfinite(got).all() and (got - want).abs().max().item() < 2e-2 * want.abs().max().item(), seqs
        g3, b3 = got.view(n, H, D), bare.view(n, H, D)
        assert (g3[:, 0] - b3[:, 0]).abs().max().item() < 1e-2 * b3.abs().max().item() and (H < 6 or (g3[:, 5] == 0).all())
        if H > 4:
            assert (g3[:, 4].norm() < 0.995 * b3[:, 4].norm())


@pytest.mark.parametrize("dtype", DTYPES)
def test_grouped_attention_over_long_contexts(dtype):
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype, max_tokens=1536)
    W, n, eps, m = 24, 1400, 1e-5, left(4, 2, 64, 48, 0.3, 9.0, rot(32, 1000.0))
    mixer, plain = bound_part(MIXERS, grouped_spec(W, m, eps), dtype, rt, seed=9)
    x = _x(n, W, dtype, 4)
    want = pf.grouped_attention(x.double().numpy(), m, plain, "m.", eps)
    for cuts in ([n], [1300, 60, 17] + [1] * 23, [900, 400, 100]):
        got = run_mixer(mixer, rt, x, cuts, page_size=16, n_pages=100)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts[:4]


# ---------------------------------------------------------------- one key stands out
def pointing_latent(H, D, Dr, R, r, back, by):
    """Weights under which every query points at ONE key.  ``latent``: the model width holds two vectors of R values per
    token; keys read the second, u_j, queries the first, which the test sets to the u of the key it means.  ``rotated``: the
    same query and key part at every token, the query's turned back by ``back`` positions: the score depends on the
    distance alone and is largest at ``back``."""
    W = 2 * R + 1
    dq, dkv = torch.zeros(R, W), torch.zeros(R + Dr, W)
    uq, uk = torch.zeros(H * (D + Dr), R), torch.zeros(H * D, R)
    for e in range(R):
        dq[e, e] = 1.0
        dkv[e, R + e] = 1.0
    if by == "latent":
        for h in range(H):
            for d in range(D):
                uq[h * (D + Dr) + d, (d + h) % R] = 1.0
                uk[h * D + d, (d + h) % R] = 1.0
    else:
        dq.zero_()
        dq[:, 2 * R] = 1.0                                                  # (the query latent is a vector of ones)
        for i, f in enumerate(pf.frequencies(r)[0]):
            dkv[R + 2 * i, 2 * R] = 1.0                                     # key part (1, 0) per pair
            for h in range(H):                                              # (cos, -sin) turned by p is (1, 0) turned by p - back
                uq[h * (D + Dr) + D + 2 * i, 0] = np.cos(back * f)
                uq[h * (D + Dr) + D + 2 * i + 1, 0] = -np.sin(back * f)
    return W, {"dq.weight": lambda v: dq, "dkv.weight": lambda v: dkv, "uq.weight": lambda v: uq, "uk.weight": lambda v: uk,
               "dq_norm.weight": lambda v: torch.ones_like(v), "dkv_norm.weight": lambda v: torch.ones_like(v), "sink": lambda v: v * 0 + 2.0}


BACKS = (0, 1, 7, 8, 15, 16, 17, 63, 64, 65, 200, 399)


def _pointing_cuts(n):
    return [n], [n - 60] + [1] * 60, [7, 2, 9, 16, 1, 15, 33, 3] + [n - 86 - 30] + [1] * 30


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("by,page", [("latent", 8), ("latent", 16), ("rotated", 16), ("rotated", 32)])
def test_one_latent_stands_out(dtype, by, page):
    """Every query points at the key ``back`` tokens behind it, by its latent or by its position alone, and gives it nearly all
    the weight beside the sink: itself, its neighbour, around a page's and a chunk's border, far away."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype, max_tokens=512)
    H, R, Dr, Dv, eps = 4, 32, 32, 16, 1e-6
    r = rot(Dr, 4.0, (2.0, 64, 8.0, 1.0))
    n = 420
    gen = torch.Generator().manual_seed(page)
    u = torch.randn(n, R, generator=gen)
    for back in BACKS:
        W, fix = pointing_latent(H, R, Dr, R, r, back, by)
        a = torch.roll(u, back, 0)
        a[:back] = torch.randn(back, R, generator=gen)                       # (no such key yet)
        x = torch.cat([a, u, torch.ones(n, 1)], dim=1).to(TORCH[dtype])
        scale = 1.0 if by == "latent" else 3.0
        mixer, plain = bound_part(MIXERS, latent_spec(W, H, R, Dr, Dv, R, R, scale, eps, r), dtype, rt, seed=5, fix=fix)
        m = dict(heads=H, dim=R, rot_dim=Dr, vdim=Dv, kv_rank=R, scale=scale, rot=r)
        want = pf.latent_attention(x.double().numpy(), m, plain, "m.", eps)
        if by == "latent" and back:                                          # without that key the last row is another
            y = x.double().numpy().copy()
            y[n - 1 - back, R:2 * R] = 0.0
            assert np.abs(pf.latent_attention(y, m, plain, "m.", eps)[-1] - want[-1]).max() > 0.2 * np.abs(want[-1]).max()
        for cuts in _pointing_cuts(n):
            got = run_mixer(mixer, rt, x, cuts, page_size=page, n_pages=n // page + 6)
            err = np.abs(got - want).max(axis=1)
            worst = int(err.argmax())
            assert err[worst] < (2e-4 if dtype == "float32" else 0.1) * np.abs(want).max(), (back, cuts[:3], worst)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("by,page", [("vector", 8), ("vector", 16), ("rotated", 32)])
def test_one_key_stands_out(dtype, by, page):
    """The same for grouped attention: by the keys' vectors, or by position alone (the query's projection turned back)."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype, max_tokens=512)
    H, G, D, Dv, eps, n = 4, 2, 32, 16, 1e-6, 420
    base = 4.0
    gen = torch.Generator().manual_seed(page)
    u = torch.randn(n, D, generator=gen)
    W = 2 * D + 1
    for back in BACKS:
        q, k = torch.zeros(H * D, W), torch.zeros(G * D, W)
        if by == "vector":
            for h in range(H):
                for d in range(D):
                    q[h * D + d, d] = 1.0
            for g in range(G):
                for d in range(D):
                    k[g * D + d, D + d] = 1.0
        else:
            for i, f in enumerate(pf.frequencies(rot(D, base))[0]):
                k[[g * D + i for g in range(G)], 2 * D] = 1.0
                q[[h * D + i for h in range(H)], 2 * D] = float(np.cos(back * f))
                q[[h * D + D // 2 + i for h in range(H)], 2 * D] = -float(np.sin(back * f))
        a = torch.roll(u, back, 0)
        a[:back] = torch.randn(back, D, generator=gen)
        x = torch.cat([a, u, torch.ones(n, 1)], dim=1).to(TORCH[dtype])
        m = left(H, G, D, Dv, 0.6 if by == "vector" else 1.0, 40.0, rot(D, base) if by == "rotated" else None)
        one = lambda v: torch.ones_like(v)
        mixer, plain = bound_part(MIXERS, grouped_spec(W, m, eps), dtype, rt, seed=5,
                                  fix={"q.weight": lambda v: q, "k.weight": lambda v: k, "q_norm.weight": one, "k_norm.weight": one})
        want = pf.grouped_attention(x.double().numpy(), m, plain, "m.", eps)
        for cuts in _pointing_cuts(n):
            got = run_mixer(mixer, rt, x, cuts, page_size=page, n_pages=n // page + 6)
            err = np.abs(got - want).max(axis=1)
            worst = int(err.argmax())
            assert err[worst] < (2e-4 if dtype == "float32" else 0.1) * np.abs(want).max(), (back, cuts[:3], worst)


# ---------------------------------------------------------------- the two side by side
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("l,r,fl,fr", [(left(6, 2, 12, 9, 0.4, 5.0, rot(8)), right(4, 6, 10, 2, 4, 3), 0.7, 1.3), (left(1, 1, 5, 5, 0.9), right(3, 5, 7, 3, 2, 5), 1.0, 1.0),
                                       (left(8, 2, 64, 40, 0.15, 10.0, rot(32)), right(4, 16, 32, 2, 4, 2), -0.8, 1.1),
                                       (left(2, 2, 16, 8, 0.3, None, rot(16)), right(2, 8, 8, 1, 3, 1), 0.0, 2.5)])
def test_both_side_by_side(dtype, l, r, fl, fr):
    """One projection and one product serve both members where their widths allow (alone they compute the same)."""
    from flambeau_amd.parts import MIXERS, PartSpec
    rt = make_rt(dtype)
    W, n, eps = 40, 90, 2e-5
    spec = PartSpec("side_by_side", dict(hidden_size=W, left=grouped_spec(W, l, eps), right=ssd_spec(W, r, eps), factors=(fl, fr), normed=False))
    mixer, plain = bound_part(MIXERS, spec, dtype, rt, seed=7)
    widths = (l["heads"] * l["vdim"], r["heads"] * r["vdim"])
    assert mixer.joined == (dtype == "float32" or not any(w % 8 for w in widths))
    x = _x(n, W, dtype, 8)
    m = dict(left=l, right=r, left_scale=fl, right_scale=fr)
    want = pf.side_by_side(x.double().numpy(), m, plain, "m.", eps)
    for cuts in CUTS:
        got = run_mixer(mixer, rt, x, cuts, page_size=16)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts
    if mixer.joined and dtype == "float32":
        for member in (mixer.left, mixer.right):
            member.joinable = False
        apart, _ = bound_part(MIXERS, spec, dtype, rt, seed=7)
        for member in (apart.left, apart.right):
            member.joinable = False
        g = torch.Generator().manual_seed(7)                                # (the same weights once more, each member with products of its own)
        w = {}
        for k, ts in apart.tensors().items():
            v = torch.randn(tuple(ts.shape), generator=g) * 0.3
            w[k] = rt.to_device(1 + v if ts.role == "vector32" and k.endswith("norm.weight") else v, ts.role)
        apart.bind(w, rt)
        assert not apart.joined
        assert np.abs(run_mixer(apart, rt, x, CUTS[1], page_size=16) - want).max() < TOL[dtype] * np.abs(want).max()


# ---------------------------------------------------------------- the feed-forward
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,W,F,limit", [(1, 40, 24, 0.8), (5, 64, 100, 0.3), (16, 128, 64, 2.0), (33, 96, 50, 1.0), (64, 64, 8, 0.5), (150, 40, 36, 0.7), (300, 256, 520, 1.5), (20, 36, 50, 9.0)])
def test_a_dense_feed_forward_with_a_clamped_gate(dtype, n, W, F, limit):
    """Rows for every product kernel; limits that bite often and seldom."""
    from flambeau_amd.parts import FEED_FORWARDS, PartSpec
    rt = make_rt(dtype, max_tokens=512)
    part, plain = bound_part(FEED_FORWARDS, PartSpec("clamped_mlp", dict(hidden_size=W, intermediate_size=F, limit=limit)), dtype, rt, seed=n)
    x = _x(n, W, dtype, 3)
    h = x.double().numpy()
    want = pf.clamped_ff(h, {"limit": limit}, plain, "m.")
    g, u = h @ plain["m.gate"].T, h @ plain["m.up"].T
    assert limit > 5 or ((g > limit).any() and (u > limit).any() and (u < -limit).any() and (g < -limit).any())       # the limit bites, and not below the gate
    got = part.forward(dev(x), None).compute(rt).double().cpu().numpy()
    assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max()
    with pytest.raises(ValueError):
        FEED_FORWARDS.create(PartSpec("clamped_mlp", dict(hidden_size=8, intermediate_size=8, limit=0.0)))


# ---------------------------------------------------------------- layer by layer
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_the_stream_after_every_layer(dirs, name, dtype):
    from flambeau_amd.engine import StepEntry
    d = dirs[(name, dtype)]
    runner = runner_for(d, dtype, n_pages=16, page_size=CONFIGS[name]["page_size"], step_programs=False, decode_graphs=False)
    seen = []
    for b in runner.model.blocks:
        def wrapped(stream, step, cache, fwd=b.forward):
            fwd(stream, step, cache)
            seen.append(stream.flush().double().cpu().numpy())
        b.forward = wrapped
    toks = rh.make_requests(CONFIGS[name]["config"]["vocab"], [37], seed=1)["r0"]
    assert runner.begin("a")
    runner.step([StepEntry("a", toks, [0])])
    cfg, t = read_model(d)
    want = []
    pf.forward(cfg, t, toks, layer_outputs=want)
    assert len(seen) == len(want)
    for i, (g, w) in enumerate(zip(seen, want)):
        err = np.abs(g - w).max(axis=1) / np.abs(w).max()
        assert err.max() < (3e-5 if dtype == "float32" else 1.5e-1) and np.median(err) < (3e-5 if dtype == "float32" else 3e-2), (f"layer {i}", err.max(), np.median(err))


# ---------------------------------------------------------------- whole models in every cutting
LENGTHS = {"A": [40, 70, 97, 1, 33, 64, 2, 90, 340, 128, 21], "B": [97, 1, 150, 64, 31, 2, 120, 17, 65],
           "C": [150, 64, 3, 65, 1, 200, 31, 90], "D": [40, 100, 7, 64, 130, 2, 55]}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", list(CONFIGS))
def test_every_cutting(dirs, name, dtype):
    d = dirs[(name, dtype)]
    ps = CONFIGS[name]["page_size"]
    reqs = rh.make_requests(CONFIGS[name]["config"]["vocab"], LENGTHS[name], seed=5)
    ref = reference(d, reqs)
    for mode, steps in [("whole", rh.trace_whole(reqs)), ("tail", rh.trace_tail(reqs)), ("portions", rh.trace_portions(reqs)),
                        ("mixed", rh.trace_mixed(reqs, seed=13))]:
        peak = rh.peak_tokens(steps)
        runner = runner_for(d, dtype, n_pages=peak // ps, page_size=ps, max_tokens=max(peak, 256), slots=4)
        for entry in runner.storage.entries:                                # (records are zeroed when a slot is claimed)
            if entry.state is not None:
                entry.state.fill_(float("nan"))
        got = rh.run_in_process(runner, steps)
        pools = runner.manager.pools
        assert sum(p.n_acquired for p in pools) > sum(p.n_pages for p in pools), mode       # pages were used again
        assert not runner.manager.live and runner.manager.n_free_slots == 4
        close(got, ref, dtype, f"{name} {mode}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_recorded_steps_of_single_tokens(dirs, name, dtype):
    """A batch of three decodes side by side: its steps are recorded, replayed and turned into graphs; one request sits a step
    out now and then, and one that ends makes room for another."""
    from flambeau_amd.engine import StepEntry
    d = dirs[(name, dtype)]
    reqs = rh.make_requests(CONFIGS[name]["config"]["vocab"], [20, 33, 40, 30], seed=12)
    ref = reference(d, reqs)
    runner = runner_for(d, dtype, n_pages=24, page_size=CONFIGS[name]["page_size"], max_tokens=256, slots=3)
    assert not runner.decode_graphs and runner.step_programs
    got, at = {}, {rid: 0 for rid in reqs}
    waiting, live = list(reqs), []
    turn = 0
    while waiting or live:
        while waiting and len(live) < 3:
            rid = waiting.pop(0)
            assert runner.begin(rid)
            runner.step([StepEntry(rid, reqs[rid][:3], [])])
            at[rid] = 3
            live.append(rid)
        turn += 1
        now = [rid for k, rid in enumerate(live) if not (turn % 5 == 0 and k == 1 and len(live) > 1)]
        rows = runner.step([StepEntry(rid, [reqs[rid][at[rid]]], [0]) for rid in now]).cpu().double().numpy()
        for rid, row in zip(now, rows):
            got[(rid, at[rid])] = row
            at[rid] += 1
            if at[rid] == len(reqs[rid]):
                runner.end(rid)
                live.remove(rid)
    assert runner.n_replayed > 10 and any(p.graphs for p in runner._programs.values()) and len(got) == sum(len(t) - 3 for t in reqs.values())
    close(got, ref, dtype, f"{name} recorded")


def test_a_batch_equals_each_request_alone(dirs):
    """Unequal requests in one step against each alone: in 32-bit not a bit differs, whatever the neighbours, pages
    and slots are."""
    from flambeau_amd.engine import StepEntry
    d = dirs[("A", "float32")]
    reqs = rh.make_requests(83, [50, 3, 1, 77], seed=9)
    alone = {}
    for rid, toks in reqs.items():
        r = runner_for(d, "float32", n_pages=32, page_size=8)
        assert r.begin(rid)
        alone[rid] = r.step([StepEntry(rid, toks, list(range(len(toks))))]).cpu().numpy().copy()
    r = runner_for(d, "float32", n_pages=32, page_size=8)
    for rid in ("x", "y"):                  # two requests come and go first: other slots, other pages, records that are not zero
        assert r.begin(rid)
        r.step([StepEntry(rid, [1, 2, 3, 4, 5, 6, 7, 8, 9], [])])
    r.end("x"); r.end("y")
    for rid in reversed(list(reqs)):
        assert r.begin(rid)
    both = r.step([StepEntry(rid, toks, list(range(len(toks)))) for rid, toks in reqs.items()]).cpu().numpy()
    at = 0
    for rid, toks in reqs.items():
        assert np.array_equal(both[at:at + len(toks)], alone[rid]), rid
        at += len(toks)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["sharp", "memory"])
def test_far_keys_and_long_memories(dirs, dtype, kind):
    """Score scales six times as large, so that single keys hundreds of tokens back or next to a page's edge carry the
    output; recurrences that forget little beside sinks of some weight: a key or a state that is lost shows."""
    d = dirs[(kind, dtype)]
    reqs = rh.make_requests(83, [380, 131], seed=2)
    ref = reference(d, reqs)
    blunt = reference(dirs[("A", dtype)], reqs)
    assert np.abs(ref["r0"] - blunt["r0"]).max() > 0.05 * np.abs(ref["r0"]).max()
    for mode, steps in [("whole", rh.trace_whole(reqs)), ("tail", rh.trace_tail(reqs, tail=90)),
                        ("portions", rh.trace_portions(reqs, sizes=(7, 2, 8, 9, 16, 1, 15, 33, 3)))]:
        runner = runner_for(d, dtype, n_pages=64, page_size=8)
        close(rh.run_in_process(runner, steps), ref, dtype, f"{kind} {mode}", bf16=8e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dirs, dtype):
    """340 single-token steps behind 57 tokens: every page of the request is kept, and every state goes on."""
    d = dirs[("A", dtype)]
    toks = rh.make_requests(83, [397], seed=4)["r0"]
    reqs = {"r0": toks}
    ref = reference(d, reqs)
    runner = runner_for(d, dtype, n_pages=56, page_size=8)
    got = rh.run_in_process(runner, [dict(s, end=[]) for s in rh.trace_tail(reqs, tail=340)])
    for g in range(len(runner.manager.groups)):
        assert sum(p >= 0 for p in runner.manager.table_row("r0", g)) == -(-397 // 8)
    runner.end("r0")
    close(got, ref, dtype, "long decoding")


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(dirs, dtype):
    """Requests of one and two tokens, alone, side by side, and continued one token at a time: the first token sees itself and
    the sinks alone, its convolution zeros before it, and a state that starts from nothing."""
    d = dirs[("A", dtype)]
    reqs = rh.make_requests(83, [1, 2, 1, 3], seed=7)
    ref = reference(d, reqs)
    steps = [dict(entries=[dict(id=rid, tokens=toks[:1], want=[0]) for rid, toks in reqs.items()], end=["r0", "r2"]),
             dict(entries=[dict(id="r1", tokens=reqs["r1"][1:], want=[0]), dict(id="r3", tokens=reqs["r3"][1:2], want=[0])], end=["r1"]),
             dict(entries=[dict(id="r3", tokens=reqs["r3"][2:], want=[0])], end=["r3"])]
    close(rh.run_in_process(runner_for(d, dtype, n_pages=8, page_size=8), steps), ref, dtype, "first tokens")


@pytest.mark.parametrize("name", ["A", "D"])
def test_a_slot_that_is_used_again_starts_from_nothing(dirs, name):
    """One state slot: every request inherits the slot of the one before, whose states and kept inputs are not zero, and
    still gives the plain logits."""
    d = dirs[(name, "float32")]
    reqs = rh.make_requests(CONFIGS[name]["config"]["vocab"], [30, 9, 1, 44], seed=8)
    ref = reference(d, reqs)
    runner = runner_for(d, "float32", n_pages=8, page_size=16, slots=1)
    close(rh.run_in_process(runner, rh.trace_portions(reqs, sizes=(5, 2, 11))), ref, "float32", "one slot")


# ---------------------------------------------------------------- through the entry points
@pytest.mark.parametrize("dtype", DTYPES)
def test_greedy_generation_through_the_engine(dirs, dtype):
    """``generate``: scheduler, portions, batching, device sampler.  Every token is the plain implementation's argmax
    (or within rounding of it)."""
    from flambeau_amd import generate
    d = dirs[("A", dtype)]
    cfg, t = read_model(d)
    prompts = [p for p in rh.make_requests(83, [7, 19, 1, 30, 12], seed=3).values()]
    outs = generate(str(d), prompts, max_new_tokens=10, dtype=dtype, page_size=8, inflight_slots=3, prefill_chunk_tokens=16)
    turned = 0
    for prompt, out in zip(prompts, outs):
        assert len(out) == 10
        toks = list(prompt)
        for tok in out:
            logits = pf.forward(cfg, t, toks)[-1]
            best = int(np.argmax(logits))
            if not (tok == best or logits[best] - logits[tok] < (1e-4 if dtype == "float32" else 3e-2) * np.abs(logits).max()):
                turned += 1
            toks.append(tok)
    assert turned <= (0 if dtype == "float32" else 2), turned


@pytest.mark.parametrize("dtype", DTYPES)
def test_trace_replay_as_a_program(dirs, tmp_path, dtype):
    d = dirs[("C", dtype)]
    reqs = rh.make_requests(150, [40, 70, 97, 33, 64, 12, 90, 55], seed=6)
    ref = reference(d, reqs)
    steps = rh.trace_mixed(reqs, seed=3)
    stats = {}
    got = rh.run_program(d, dtype, steps, tmp_path / "o", rh.peak_tokens(steps), 150, extra=("--poison-cache",), stats=stats)
    assert stats["handed_out"] > stats["pool"]
    close(got, ref, dtype, "trace_run")


def test_the_command_line_serves_it(tmp_path):
    """``random-weights`` -> ``inspect`` -> ``infer --json`` on a Fipitar configuration, greedy in 32-bit with so few
    slots and pages that requests wait and are pre-empted (a pre-empted request starts again with nothing kept): exactly
    the plain implementation's tokens."""
    import subprocess
    import sys
    cfg = CONFIGS["A"]["config"]
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    d = tmp_path / "model"

    def cli(*args):
        r = subprocess.run([sys.executable, "-m", "flambeau_amd", *map(str, args)], capture_output=True, text=True, timeout=600, cwd=str(rh.ROOT))
        assert r.returncode == 0, f"{args}\n{r.stdout[-2000:]}\n{r.stderr[-4000:]}"
        return r
    cli("random-weights", "--config", tmp_path / "config.json", "--out", d, "--seed", 5, "--std", 0.3, "--gain-std", 0.1, "--dtype", "float32")
    seen = cli("inspect", d).stdout
    assert "architecture: Fipitar" in seen and "tensors fit the model" in seen and "l2.mix.right.conv.b" in seen
    prompts = list(rh.make_requests(83, [3, 30, 17], seed=6).values())
    flags = []
    for p in prompts:
        flags += ["--prompt", ",".join(map(str, p))]
    out = json.loads(cli("infer", "--model", d, *flags, "--max-tokens", 18, "--dtype", "float32", "--json", "--inflight-slots", 2,
                         "--paged-kv", 5, "--page-size", 16, "--prefill-chunk-tokens", 16, "--max-queue-depth", 4).stdout)
    conf, t = read_model(d)
    for p, o in zip(prompts, out["outputs"]):
        toks = list(p)
        for tok in o:
            logits = pf.forward(conf, t, toks)[-1]
            best = int(np.argmax(logits))
            assert tok == best or logits[best] - logits[tok] < 1e-4 * np.abs(logits).max()
            toks.append(tok)
        assert len(o) == 18
