"""Lufivik on the GPU against the plain implementation: every mechanism alone, the layers one by one, and whole
models in every cutting (whole prompts, single tokens, portions down to two tokens, mixed batches over a small
poisoned pool whose pages and slots are used again), in 32-bit and in bfloat16, at sizes of the tests' own."""
import json

import numpy as np
import pytest
import torch

import plain_lufivik as pl
import replay_helpers as rh
from lufivik_configs import CONFIGS, read_model, write_model
from test_bugidra_gpu import TOL, _x, run_mixer, runner_for
from test_bugidra_gpu import bound_part as _bound_part
from test_kuvidra_gpu import close, make_rt, make_step

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = ["float32", "bfloat16"]
TORCH = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def far_sighted(tensors):
    """A convolution whose kept inputs matter: taps as large as the token's own."""
    for n in tensors:
        if n.endswith("canon1"):
            tensors[n] = (tensors[n].float() * 2).to(tensors[n].dtype)


@pytest.fixture(scope="module")
def dirs(tmp_path_factory):
    base = tmp_path_factory.mktemp("lufivik")
    out = {}
    for name in CONFIGS:
        for store in DTYPES:
            out[(name, store)] = write_model(name, base / f"{name}-{store}", store)
    for store in DTYPES:          # (weights are stored in the dtype they are run in: the plain side reads the same numbers)
        out[("sharp", store)] = write_model("A", base / f"A-sharp-{store}", store, sharpen=8.0 if store == "float32" else 2.5, edit=far_sighted)
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
            _refs[key] = pl.forward(cfg, t, toks)
        out[rid] = _refs[key]
    return out


dev = lambda v: v.to(DEV).contiguous() if v is not None else None


def bound_part(*args, **kw):
    part, plain = _bound_part(*args, **kw)
    return part, {k.replace("_norm", ".norm") if k.endswith("_norm") else k: v for k, v in plain.items()}


# ---------------------------------------------------------------- each mechanism alone
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("W", [37, 40, 256, 516, 1000, 2048, 4096, 5000, 6002, 16384, 20000])
def test_a_sublayer_s_way_into_the_stream_alone(dtype, W):
    """Gate, norm, scale and sum in one kernel, with and without each, with the norm of the new stream, over rows that
    are held in registers and rows that are not; layer norms and root-mean-square norms; the rows of a token's experts
    added on the way."""
    from flambeau_amd.kernels import ops
    g = torch.Generator().manual_seed(W)
    n, eps, top = 7, 3e-4, 3
    rnd = lambda *s, c=0.0: c + torch.randn(*s, generator=g)
    y, x, gate, gb = rnd(n, W, c=0.3), rnd(n, W) * 2, rnd(n, W), rnd(W)
    w, b, ls, nw, nb = rnd(W, c=1.0), rnd(W), rnd(W), rnd(W, c=1.0), rnd(W)
    rows, place = rnd(n * top, W), torch.randperm(n * top, generator=g).int()
    d = lambda t: t.double().numpy() if t is not None else None

    def norm(v, w, b, centred):
        return pl.layer_norm(v, d(w), d(b) if b is not None else 0.0, eps) if centred else pl.rms_norm(v, d(w), eps) + (d(b) if b is not None else 0.0)
    for opt in range(8):
        gated, biased, scaled, centred, by_rows, next_centred = opt != 1, opt % 2 == 0, opt != 2, opt < 6, opt in (3, 7), opt != 5
        resid = dev(x)
        h = torch.full((n, W), float("nan"), dtype=TORCH[dtype], device=DEV) if opt != 4 else None
        ops.sublayer_step(dev(rows if by_rows else y), resid, dev(w), dev(b) if biased else None, eps, centred, scale=dev(ls) if scaled else None,
                          gate=dev(gate) if gated else None, gate_bias=dev(gb) if gated and biased else None,
                          place=dev(place) if by_rows else None, top=top if by_rows else 0,
                          next_norm=(dev(nw), dev(nb) if biased else None, eps, next_centred) if h is not None else None, out=h)
        v = d(rows)[place.long().numpy()].reshape(n, top, W).sum(axis=1) if by_rows else d(y)
        if gated:
            v = v * pl.sigmoid(d(gate) + (d(gb) if biased else 0.0))
        want = d(x) + (d(ls) if scaled else 1.0) * norm(v, w, b if biased else None, centred)
        assert np.abs(d(resid.cpu()) - want).max() < 1e-5 * np.abs(want).max(), opt
        if h is not None:
            want_h = norm(want, nw, nb if biased else None, next_centred)
            assert np.abs(h.double().cpu().numpy() - want_h).max() < (2e-5 if dtype == "float32" else 1e-2) * np.abs(want_h).max(), opt


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,taps", [(40, 3), (37, 1), (64, 5), (300, 2), (2052, 4), (36, 7)])
def test_the_input_convolution_alone(dtype, C, taps):
    """Two requests side by side, cut into portions shorter and longer than the convolution reaches, in slots whose
    neighbours hold NaN; rows without a slot write nothing; in both types not a bit depends on the cutting; a step of
    one token leaves the same record however often it runs."""
    from flambeau_amd.kernels import ops
    g = torch.Generator().manual_seed(C + taps)
    n = 40
    hs = [torch.randn(n, C, generator=g).to(TORCH[dtype]) for _ in range(2)]
    w = torch.randn(C, taps, generator=g)
    wt = dev(w.t())
    want = [h.double().numpy() + pl.causal_convolution(h.double().numpy(), w.double().numpy()) for h in hs]
    results = []
    for cuts in ([40], [1] * 40, [2, 1, 3, 7, 2, 1, 1, 8, 2, 13], [5, 35], [33, 1, 6]):
        ring = torch.full((5, taps, C), float("nan"), device=DEV)
        ring[3], ring[1] = 0.0, 0.0
        got = [[], []]
        at = 0
        for k in cuts:
            step = make_step([(at, k), (at, k)], 8, 20, slots=[3, 1])
            h = dev(torch.cat([x[at:at + k] for x in hs]))
            for _ in range(2 if k == 1 else 1):
                out = ops.input_conv(h, wt, ring, step, torch.full_like(h, float("nan")))
            got[0].append(out[:k].double().cpu().numpy()); got[1].append(out[k:].double().cpu().numpy())
            at += k
        assert torch.isnan(ring[[0, 2, 4]]).all()
        results.append([np.concatenate(x) for x in got])
        for a, b in zip(results[-1], want):
            assert np.abs(a - b).max() < (1e-6 if dtype == "float32" else 6e-3) * np.abs(b).max(), cuts
        assert all(np.array_equal(a, b) for a, b in zip(results[-1], results[0])), cuts
    # rows that pad a batch: no slot, nothing is read or written
    ring = torch.full((2, taps, C), 3.0, device=DEV)
    step = make_step([(9, 1), (0, 1)], 8, 20, slots=[-1, -1])
    h = dev(hs[0][:2])
    out = ops.input_conv(h, wt, ring, step, torch.empty_like(h))
    assert (ring == 3.0).all() and torch.isfinite(out.float()).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("buckets,mul_prev,mul_cur", [(31, 7, 3), (1, 5, 0), (5000, 100003, 99991), (64, 0, 9), (97, 2147483629, 2147483587)])
def test_the_embedding_with_a_row_per_pair_alone(dtype, buckets, mul_prev, mul_cur):
    """Rows of token pairs across the steps' edges, the extra row for first tokens, products beyond 32 bits; requests of
    unequal lengths side by side in reused slots; a step of one token that runs twice changes nothing."""
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.parts import EMBEDDINGS, PartSpec
    rt = make_rt(dtype)
    V, W, eps = 211, 44, 1e-5
    spec = PartSpec("bigram_token_embedding", dict(vocab_size=V, hidden_size=W, buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur,
                                                   norm=PartSpec("layernorm", dict(hidden_size=W, eps=eps))))
    part, plain = bound_part(EMBEDDINGS, spec, dtype, rt, seed=7, prefix="")
    t = {"embed": plain["weight"], "bigram": plain["pairs"], "embed.norm": plain["norm"], "embed.norm.b": plain.get("norm.b", plain.get("norm.bias"))}
    cfg = {"embedding": {"bigram": dict(buckets=buckets, mul_prev=mul_prev, mul_cur=mul_cur)}, "norm": {"eps": eps}}
    rng = np.random.default_rng(3)
    toks = [[int(x) for x in rng.integers(0, V, 30)] for _ in range(2)]
    toks[0][3], toks[0][4] = 0, V - 1
    want = [pl.embed(x, cfg, t) for x in toks]
    cache = CacheStorage([part.cache_spec()], [None], rt.device, rt.dtype, n_pages=4, page_size=8, max_slots=3).entries[0]
    for cuts in ([30], [1] * 30, [2, 1, 5, 4, 2, 16], [29, 1]):
        cache.state.fill_(77)                                  # (what other requests left; a first token never reads it)
        at = 0
        for k in cuts:
            step = make_step([(at, k), (at, k)], 8, 20, slots=[2, 0])
            ids = torch.tensor(toks[0][at:at + k] + toks[1][at:at + k], dtype=torch.int32, device=DEV)
            for _ in range(2 if k == 1 else 1):
                got = part.forward(ids, torch.empty(2 * k, W, device=DEV), step=step, cache=cache).double().cpu().numpy()
            for r in range(2):
                assert np.abs(got[r * k:(r + 1) * k] - want[r][at:at + k]).max() < 2e-5 * np.abs(want[r]).max(), (cuts, at, r)
            at += k
        assert (cache.state[1] == 77).all()
    pad = make_step([(4, 1)], 8, 20, slots=[-1])               # a row that pads a batch
    cache.state.fill_(9)
    part.forward(torch.tensor([3], dtype=torch.int32, device=DEV), torch.empty(1, W, device=DEV), step=pad, cache=cache)
    assert (cache.state == 9).all()


def mixer_spec(W, H, D, Dr, Dv, Rq, R, scale, eps, window, base, dims=None):
    from flambeau_amd.parts import PartSpec
    return PartSpec("latent_attention", dict(hidden_size=W, n_heads=H, head_dim=D, value_dim=Dv, q_rank=Rq, kv_rank=R, scale=scale, eps=eps,
                                             window=window, rot_dim=Dr, position=PartSpec("rope_neox", dict(
                                                 head_dim=Dr, theta=base, rotated_dims=Dr if dims is None else dims))))


def mixer_dict(H, D, Dr, Dv, R, scale, window, base, dims=None):
    return dict(heads=H, dim=D, rot_dim=Dr, vdim=Dv, kv_rank=R, scale=scale, rot={"base": base, "dims": Dr if dims is None else dims},
                mask={"size": window} if window else None)


SHAPES = [
    # H, D, Dr, Dv, Rq, R, window, base, rotated dims
    (3, 10, 6, 12, 14, 24, 13, 100.0, None), (1, 7, 2, 5, 9, 150, 1, 30.0, None), (6, 4, 8, 4, 4, 64, 70, 1000.0, 4), (2, 16, 10, 16, 8, 33, 0, 50.0, None),
    # sizes that the matrix-core kernels take, all three or some of them
    (20, 32, 32, 48, 24, 96, 64, 100.0, None), (4, 64, 16, 16, 40, 160, 33, 5000.0, None), (16, 8, 64, 32, 8, 32, 100, 70.0, None),
    (2, 96, 24, 16, 16, 512, 40, 10000.0, None), (40, 40, 34, 16, 24, 256, 90, 10000.0, 18),
    (40, 64, 32, 32, 24, 128, 70, 300.0, None), (36, 32, 64, 16, 24, 512, 100, 2000.0, None),
    (3, 24, 70, 16, 16, 64, 50, 300.0, None),          # a rotated part wider than they take beside the latent
]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,D,Dr,Dv,Rq,R,window,base,dims", SHAPES)
def test_latent_attention_with_a_rotated_part_alone(dtype, H, D, Dr, Dv, Rq, R, window, base, dims):
    """Both latents and their norms, the folded keys, the rotated part of queries and keys, the window and the gate
    against the plain function, whole and in portions that cross the window's edge, page borders and the kernels' chunks."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype)
    W, n, eps, scale = 40, 150, 2e-5, 0.4 / max(1, R / 64)
    mixer, plain = bound_part(MIXERS, mixer_spec(W, H, D, Dr, Dv, Rq, R, scale, eps, window, base, dims), dtype, rt, seed=H + D)
    assert mixer.cache_spec().window == window and mixer.graph_safe and mixer.replayable
    x = _x(n, W, dtype, 5)
    m = mixer_dict(H, D, Dr, Dv, R, scale, window, base, dims)
    want = pl.latent_attention(x.double().numpy(), m, plain, "m.", eps)
    if window != 1:                                                         # the rotation matters
        other = pl.latent_attention(x.double().numpy(), dict(m, rot={"base": base * 3, "dims": m["rot"]["dims"]}), plain, "m.", eps)
        assert Dr == 2 or np.abs(other - want).max() > 1e-3 * np.abs(want).max()
    for cuts in ([n], [60, 5, 1, 1, 2, 30, 2, 6, 1, 42], [1] * 90 + [60]):
        got = run_mixer(mixer, rt, x, cuts, page_size=16 if H > 3 else 8)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts


@pytest.mark.parametrize("H,R,rot,ps", [(20, 128, 32, 16), (5, 128, 64, 32), (32, 256, 64, 16), (64, 256, 0, 32), (70, 512, 64, 16), (16, 512, 32, 64), (33, 512, 0, 16),
                                        (20, 96, 64, 16), (17, 192, 32, 16)])
@pytest.mark.parametrize("window", [0, 1, 40, 64, 131])
def test_the_prompt_kernels_of_latent_attention(H, R, rot, ps, window):
    """The matrix-core kernels whose blocks share their keys against the float kernel: unequal requests, one of a single
    token, some that start mid-context, one that ends at a page's border; every row that no query sees, in pages beyond
    the newest token and behind the window alike, holds NaN; one (query, key) score per request stands out."""
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.kernels import latent_attention as la
    from flambeau_amd.kernels import ops
    from flambeau_amd.parts import PagedRowSpec
    n_pages, K = -(-1600 // ps), R + rot
    store = CacheStorage([PagedRowSpec(K, window, R)], [None], torch.device(DEV), torch.bfloat16, n_pages=n_pages, page_size=ps, max_slots=4)
    pool = store.pools[0][0]                                                # [pages, ps * (K + R)]
    g = torch.Generator().manual_seed(H + R)
    seqs = [(0, 150), (300, 7), (63, 1), (122, 70)]
    step = make_step(seqs, ps, n_pages)
    pool.fill_(float("nan"))
    for s, (st, q) in enumerate(seqs):
        for j in range(max(0, st - window + 1) if window else 0, st + q):
            page, r = int(step.block_tables[0][s, j // ps]), j % ps
            v = torch.randn(K, generator=g).to(torch.bfloat16).to(DEV) * 0.7
            pool[page, r * K:(r + 1) * K] = v
            pool[page, ps * K:].view(R, ps)[:, r] = v[:R]
    n = step.n_tokens
    qa = (torch.randn(n, H, K, generator=g) * 0.4).to(torch.bfloat16).to(DEV)
    at = 0
    for s, (st, q) in enumerate(seqs):                                      # the request's last query points at the oldest key it sees
        key = max(0, st + q - 1 - (window or 10 ** 6) + 1)
        page, r = int(step.block_tables[0][s, key // ps]), key % ps
        qa[at + q - 1] = pool[page, r * K:(r + 1) * K]
        at += q
    qa = qa.view(n, H * K).contiguous()
    cache = store.entries[0].kv
    args = (cache, step.positions, step.tok_seq, step.block_tables[0], H, 0.25, window)
    want = ops.latent_attention(qa.float(), torch.empty(n, H * R, device=DEV), *args)
    tiles = torch.tensor(la.shared_tiles(step.host, -(-H // 16)), dtype=torch.int32, device=DEV)
    got = la.latent_attention_shared(qa, torch.full((n, H * R), float("nan"), device=DEV), *args, tiles)
    assert torch.isfinite(want).all() and torch.isfinite(got).all()
    assert (got - want).abs().max().item() < 1e-2 * want.abs().max().item()
    dealt = la.latent_attention_mfma(qa, torch.full((n, H * R), float("nan"), device=DEV), *args, dealt=True)
    assert (dealt - want).abs().max().item() < 1e-2 * want.abs().max().item()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("R,window", [(64, 700), (512, 0), (96, 1025)])
def test_long_contexts(dtype, R, window):
    """1,400 tokens: keys in many chunks and, for single tokens behind them, in many parts."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype, max_tokens=1536)
    W, n, eps, H, D, Dr, Dv, Rq, base = 24, 1400, 1e-5, 4, 32, 16, 16, 16, 1000.0
    scale = 2.4 / R ** 0.5
    mixer, plain = bound_part(MIXERS, mixer_spec(W, H, D, Dr, Dv, Rq, R, scale, eps, window, base), dtype, rt, seed=R)
    x = _x(n, W, dtype, 4)
    want = pl.latent_attention(x.double().numpy(), mixer_dict(H, D, Dr, Dv, R, scale, window, base), plain, "m.", eps)
    for cuts in ([n], [1300, 60, 17] + [1] * 23, [900, 400, 100]):
        assert sum(cuts) == n
        got = run_mixer(mixer, rt, x, cuts, page_size=16, n_pages=100)
        assert np.abs(got - want).max() < TOL[dtype] * np.abs(want).max(), cuts[:4]


def pointing(kind, H, D, Dr, R, base, back):
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
    if kind == "latent":
        for h in range(H):
            for d in range(D):
                uq[h * (D + Dr) + d, (d + h) % R] = 1.0
                uk[h * D + d, (d + h) % R] = 1.0
    else:
        half = Dr // 2
        dq.zero_()
        dq[:, 2 * R] = 1.0                                                  # (the query latent is a vector of ones)
        for i in range(half):
            a = back * base ** (-2.0 * i / Dr)
            dkv[R + i, 2 * R] = 1.0                                         # key part (1, .., 0, ..)
            for h in range(H):
                # (cos, -sin) turned by p is (cos, ..) turned by p - back
                uq[h * (D + Dr) + D + i, 0] = np.cos(a)
                uq[h * (D + Dr) + D + half + i, 0] = -np.sin(a)
    return W, {"dq.weight": lambda v: dq, "dkv.weight": lambda v: dkv, "uq.weight": lambda v: uq, "uk.weight": lambda v: uk,
               "dq_norm.weight": lambda v: torch.ones_like(v), "dkv_norm.weight": lambda v: torch.ones_like(v)}


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["latent", "rotated"])
@pytest.mark.parametrize("window,page", [(13, 8), (64, 16), (300, 16), (1, 8), (129, 32)])
def test_one_key_stands_out_at_the_window_s_edges(dtype, kind, window, page):
    """Every query points at the key ``back`` tokens behind it, by its latent or by its position alone, and gives it nearly
    all the weight if it is seen: the window's last key inside and the first outside, the query's own and its
    neighbour, in a whole prompt, in portions and token by token, over pages of several sizes."""
    from flambeau_amd.parts import MIXERS
    rt = make_rt(dtype, max_tokens=512)
    H, R, Dr, Dv, eps, base = 4, 32, 32, 16, 1e-6, 4.0
    D = R
    n = max(2 * window + 40, 120) if window < 200 else 420
    gen = torch.Generator().manual_seed(window)
    u = torch.randn(n, R, generator=gen)
    for back in sorted({b for b in (0, 1, window - 1, window, window + 1, window // 2) if b >= 0}):
        W, fix = pointing(kind, H, D, Dr, R, base, back)
        a = torch.roll(u, back, 0)
        a[:back] = torch.randn(back, R, generator=gen)                       # (no such key yet)
        x = torch.cat([a, u, torch.ones(n, 1)], dim=1).to(TORCH[dtype])
        scale = 1.0 if kind == "latent" else 4.0
        mixer, plain = bound_part(MIXERS, mixer_spec(W, H, D, Dr, Dv, R, R, scale, eps, window, base), dtype, rt, seed=5, fix=fix)
        m = mixer_dict(H, D, Dr, Dv, R, scale, window, base)
        h = x.double().numpy()
        want = pl.latent_attention(h, m, plain, "m.", eps)
        # the plain side itself turns round when the edge moves by one key
        if back in (window - 1, window) and window > 1:
            moved = pl.latent_attention(h, dict(m, mask={"size": window - 1 if back == window - 1 else window + 1}), plain, "m.", eps)
            assert np.abs(moved[-1] - want[-1]).max() > 0.1 * np.abs(want).max(), back
        tail = min(n - 1, window + 20)
        for cuts in ([n], [n - tail] + [1] * tail, [7, 2, 9, 16, 1, 15, 33, 3] + [n - 86 - 30] + [1] * 30):
            assert sum(cuts) == n
            got = run_mixer(mixer, rt, x, cuts, page_size=page, n_pages=n // page + 6)
            err = np.abs(got - want).max(axis=1)
            worst = int(err.argmax())
            assert err[worst] < (2e-4 if dtype == "float32" else 0.1) * np.abs(want).max(), (back, cuts[:3], worst)


def experts_spec(W, f):
    from flambeau_amd.parts import PartSpec
    return PartSpec("routed_experts", dict(hidden_size=W, n_experts=f["router"]["experts"], top=f["router"]["top"], expert_size=f["expert"]["ff"],
                                           scoring="softmax", renormalise=False, weight_on="output", gate_limit=f["expert"]["limit"],
                                           gate_alpha=1.702, up_shift=1.0))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,W,E,top,F,limit", [(37, 40, 5, 2, 16, 0.8), (150, 64, 8, 3, 32, 1.5), (5, 36, 1, 1, 20, 0.2), (64, 48, 4, 4, 24, 5.0), (9, 64, 70, 16, 7, 1.0),
                                               (300, 64, 3, 2, 64, 0.5), (2, 96, 6, 3, 48, 0.6)])
def test_experts_with_a_clamped_gate_alone(dtype, n, W, E, top, F, limit):
    """The softmax router's scores as they are, the clamped gate with limits that bite often and seldom, the sum over a
    token's experts by its own kernel and left to whoever takes it."""
    from flambeau_amd.parts import FEED_FORWARDS
    from flambeau_amd.parts.base import ExpertRows
    rt = make_rt(dtype, max_tokens=512)
    f = {"router": {"experts": E, "top": top}, "expert": {"ff": F, "limit": limit}}
    part, plain = bound_part(FEED_FORWARDS, experts_spec(W, f), dtype, rt, seed=n, prefix="f.")
    x = _x(n, W, dtype, 3)
    h = x.double().numpy()
    want = pl.experts_ff(h, f, plain, "f.")
    pre = h @ plain["f.e0.up"].T
    assert (np.abs(pre) > limit).any()                                       # the limit bites
    got = part.forward(dev(x), None).double().cpu().numpy()
    part.leave_rows = True
    rows = part.forward(dev(x), None)
    assert isinstance(rows, ExpertRows)
    assert np.array_equal(rows.compute(rt).double().cpu().numpy(), got)
    # rows whose last chosen and first left-out scores are a rounding apart may turn either way: leave them out
    z = np.sort(h @ plain["f.router"].T, axis=1)[:, ::-1]
    sure = np.ones(n, dtype=bool) if top >= E else (z[:, top - 1] - z[:, top]) > (1e-5 if dtype == "float32" else 1e-2)
    assert sure.sum() > 0.6 * n
    assert np.abs(got - want)[sure].max() < (3e-5 if dtype == "float32" else 4e-2) * np.abs(want).max()


def test_a_gate_that_cannot_be_is_refused():
    from flambeau_amd.parts import FEED_FORWARDS, PartSpec
    base = dict(hidden_size=8, n_experts=2, top=1, expert_size=8)
    for bad in (dict(gate_limit=0.0), dict(gate_limit=-1.0), dict(gate_limit=1.0, gated=False), dict(gate_alpha=2.0), dict(up_shift=1.0)):
        with pytest.raises(ValueError):
            FEED_FORWARDS.create(PartSpec("routed_experts", dict(base, **bad)))


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_layer_without_its_options(dtype):
    """The arrangement without gate, scale and convolution, with root-mean-square norms and a dense feed-forward: norms
    on both sides and plain sums."""
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.parts import BLOCKS, PartSpec, ResidualStream
    rt = make_rt(dtype)
    W, n, eps, H, D, Dr, Dv, Rq, R = 40, 60, 1e-5, 3, 8, 6, 8, 12, 20
    spec = PartSpec("sandwich", dict(mixer=mixer_spec(W, H, D, Dr, Dv, Rq, R, 0.4, eps, 17, 60.0), hidden_size=W,
                                     feed_forward=PartSpec("swiglu", dict(hidden_size=W, intermediate_size=24)),
                                     norm=PartSpec("rmsnorm", dict(hidden_size=W, eps=eps))))
    block, p = bound_part(BLOCKS, spec, dtype, rt, seed=2, prefix="")
    assert not any("gate.bias" in k or "scale" in k or "conv" in k for k in block.tensors())
    store = CacheStorage([block.cache_spec()], [None], rt.device, rt.dtype, n_pages=20, page_size=8, max_slots=2)
    x = torch.randn(n, W, generator=torch.Generator().manual_seed(1))
    step = make_step([(0, n)], 8, 20)
    step.extra.update({k: torch.tensor(a, dtype=torch.int32, device=DEV) for k, a in type(block.mixer).step_metadata_for(step.host, [block.mixer]).items()})
    resid = dev(x)
    stream = ResidualStream(resid, rt)
    block.forward(stream, step, store.entries[0])
    got = stream.flush().double().cpu().numpy()
    t = {k[len("mixer."):]: v for k, v in p.items() if k.startswith("mixer.") and k != "mixer.norm"}
    weight = lambda name: p[name.replace("_norm", ".norm")]
    v = x.double().numpy()
    h = pl.rms_norm(v, weight("mixer_norm"), eps)
    v = v + pl.rms_norm(pl.latent_attention(h, mixer_dict(H, D, Dr, Dv, R, 0.4, 17, 60.0), t, "", eps), weight("mixer_out_norm"), eps)
    h = pl.rms_norm(v, weight("ffn_norm"), eps)
    g = h @ p["ffn.gate"].T
    v = v + pl.rms_norm((g * pl.sigmoid(g) * (h @ p["ffn.up"].T)) @ p["ffn.down"].T, weight("ffn_out_norm"), eps)
    assert np.abs(got - v).max() < (3e-5 if dtype == "float32" else 4e-2) * np.abs(v).max()


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
    pl.forward(cfg, t, toks, layer_outputs=want)
    assert len(seen) == len(want)
    for i, (g, w) in enumerate(zip(seen, want)):
        err = np.abs(g - w).max(axis=1) / np.abs(w).max()
        if dtype == "float32":
            assert err.max() < 2e-5, f"layer {i}"
        else:               # (a token whose choice of experts is a close call may turn the other way in bfloat16, and is then far off)
            assert np.median(err) < 5e-2 and (err > 1e-1).mean() <= 0.2, f"layer {i}"


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
        got = rh.run_in_process(runner, steps)
        pools = runner.manager.pools
        assert sum(p.n_acquired for p in pools) > sum(p.n_pages for p in pools), mode       # pages were used again
        assert not runner.manager.live and runner.manager.n_free_slots == 4
        close(got, ref, dtype, f"{name} {mode}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("name", ["A", "C"])
def test_single_tokens_replay_captured_graphs(dirs, name, dtype):
    """Kept inputs and last tokens are written where a step of one token does not read, so steps of single tokens are
    captured and replayed; batches of three are padded to four, and the padding leaves slot 0, which belongs to a
    request, alone.  A request that sits steps out, and one that ends and whose slot is taken, ride along."""
    from flambeau_amd.engine import StepEntry
    d = dirs[(name, dtype)]
    reqs = rh.make_requests(CONFIGS[name]["config"]["vocab"], [20, 33, 40, 30], seed=12)
    ref = reference(d, reqs)
    runner = runner_for(d, dtype, n_pages=24, page_size=CONFIGS[name]["page_size"], max_tokens=256, slots=3)
    assert runner.decode_graphs
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
    assert runner._graphs and len(got) == sum(len(t) - 3 for t in reqs.values())
    close(got, ref, dtype, f"{name} graphs")


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
def test_peaked_attention_over_far_keys_and_page_borders(dirs, dtype):
    """Score scales eight times as large (in bfloat16, whose rounding eight layer runs would blow up, two and a half times) and convolutions that reach back as strongly as they see the token itself: single
    keys, hundreds of tokens back or next to a page's or a window's edge, carry the output, so one key lost, one too
    many or one kept input lost shows in the logits."""
    d = dirs[("sharp", dtype)]
    reqs = rh.make_requests(83, [380, 131], seed=2)
    ref = reference(d, reqs)
    blunt = reference(dirs[("A", dtype)], reqs)
    assert np.abs(ref["r0"] - blunt["r0"]).max() > 0.05 * np.abs(ref["r0"]).max()
    for mode, steps in [("whole", rh.trace_whole(reqs)), ("tail", rh.trace_tail(reqs, tail=90)),
                        ("portions", rh.trace_portions(reqs, sizes=(7, 2, 8, 9, 16, 1, 15, 33, 3)))]:
        runner = runner_for(d, dtype, n_pages=64, page_size=8)
        close(rh.run_in_process(runner, steps), ref, dtype, f"sharp {mode}", bf16=8e-2)


@pytest.mark.parametrize("dtype", DTYPES)
def test_long_decoding(dirs, dtype):
    """340 single-token steps, during which windows of 1, 13, 70 and 300 keys pass over decoded tokens; the pages behind
    a window are given back (every pass of the loop has its own), and what is left is what the window still needs."""
    d = dirs[("A", dtype)]
    toks = rh.make_requests(83, [397], seed=4)["r0"]
    reqs = {"r0": toks}
    ref = reference(d, reqs)
    runner = runner_for(d, dtype, n_pages=56, page_size=8)
    got = rh.run_in_process(runner, [dict(s, end=[]) for s in rh.trace_tail(reqs, tail=340)])
    for g, spec in enumerate(runner.manager.groups):
        held = [b for b, p in enumerate(runner.manager.table_row("r0", g)) if p >= 0]
        assert held[0] == (397 - spec.window + 1) // 8, (g, spec.window, held[:3])
    runner.end("r0")
    close(got, ref, dtype, "long decoding")


@pytest.mark.parametrize("dtype", DTYPES)
def test_first_tokens(dirs, dtype):
    """Requests of one and two tokens, alone, side by side, and continued one token at a time: the first token takes the
    extra row of the table of pairs, its convolution sees zeros before it, and it sees itself alone."""
    d = dirs[("A", dtype)]
    reqs = rh.make_requests(83, [1, 2, 1, 3], seed=7)
    ref = reference(d, reqs)
    steps = [dict(entries=[dict(id=rid, tokens=toks[:1], want=[0]) for rid, toks in reqs.items()], end=["r0", "r2"]),
             dict(entries=[dict(id="r1", tokens=reqs["r1"][1:], want=[0]), dict(id="r3", tokens=reqs["r3"][1:2], want=[0])], end=["r1"]),
             dict(entries=[dict(id="r3", tokens=reqs["r3"][2:], want=[0])], end=["r3"])]
    close(rh.run_in_process(runner_for(d, dtype, n_pages=8, page_size=8), steps), ref, dtype, "first tokens")
    # the extra row is another than any pair's: without it the first token's logits differ
    cfg, t = read_model(d)
    t = dict(t, bigram=np.concatenate([t["bigram"][:-1], t["bigram"][:1]]))
    assert np.abs(pl.forward(cfg, t, reqs["r1"])[0] - ref["r1"][0]).max() > 1e-2 * np.abs(ref["r1"]).max()


@pytest.mark.parametrize("name", ["A", "D"])
def test_a_slot_that_is_used_again_starts_from_nothing(dirs, name):
    """One state slot: every request inherits the slot of the one before, whose kept inputs and last tokens are not zero,
    and still gives the plain logits."""
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
            logits = pl.forward(cfg, t, toks)[-1]
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
    """``random-weights`` -> ``inspect`` -> ``infer --json`` on a Lufivik configuration, greedy in 32-bit with so few
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
    assert "architecture: Lufivik" in seen and "tensors fit the model" in seen and "l1.rg2.b" in seen and "bigram" in seen
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
            logits = pl.forward(conf, t, toks)[-1]
            best = int(np.argmax(logits))
            assert tok == best or logits[best] - logits[tok] < 1e-4 * np.abs(logits).max()
            toks.append(tok)
        assert len(o) == 18
