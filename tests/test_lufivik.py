"""Lufivik without a GPU: its configuration, its description as parts, what its layers and its embedding keep per
request, its tensor names, random weights as a folder, and the plain implementation's own invariants."""
import json

import numpy as np
import pytest
import torch

import plain_lufivik as pl
from lufivik_configs import CONFIGS, read_model, write_model


def _spec(name):
    from flambeau_amd.registry import config_from_dict
    arch, cfg = config_from_dict(CONFIGS[name]["config"], "test")
    return arch, cfg, arch.build_spec(cfg)


def test_the_architecture_is_found_by_its_name():
    from flambeau_amd.registry import known_architectures
    assert {"Lufivik", "Lenedra", "Fitevik", "Bugidra", "Kuvidra", "MistralForCausalLM"} <= set(known_architectures())
    arch, cfg, spec = _spec("A")
    assert arch.name == "Lufivik" and cfg.width == 40 and cfg.vocab_size == 83 and not spec.tied_head
    assert spec.embedding.kind == "bigram_token_embedding"
    assert {k: spec.embedding.params[k] for k in ("buckets", "mul_prev", "mul_cur")} == dict(buckets=31, mul_prev=7, mul_cur=3)
    assert all(l.block.kind == "sandwich" and l.block.params["gated"] and l.block.params["layer_scale"] and l.block.params["conv_taps"] == 3
               for l in spec.layers)
    assert spec.layers[2].block.params["feed_forward"] is None
    assert [e.layer for e in spec.run_order] == [0, 1, 2, 1, 2, 1, 2, 3] and all(e.cache_of is None for e in spec.run_order)
    _, _, d = _spec("D")                                                    # no table of pairs; a loop of one pass
    assert d.embedding.kind == "normed_token_embedding" and [e.layer for e in d.run_order] == [0, 1]
    _, _, b = _spec("B")
    assert [e.layer for e in b.run_order] == [0, 1]


def test_every_size_comes_from_the_file():
    _, cfg, _ = _spec("A")
    l0, l1, l2, l3 = cfg.layers
    m = l0.mixer
    assert (m.heads, m.dim, m.rot_dim, m.vdim, m.q_rank, m.kv_rank, m.scale, m.window, m.rot_base, m.rot_dims) == (3, 10, 6, 12, 14, 24, 0.5, 13, 100.0, 6)
    assert (l0.mlp.experts, l0.mlp.top, l0.mlp.ff, l0.mlp.limit) == (5, 2, 16, 0.8)
    assert l1.mixer.rot_base == 1000.0 and l2.mlp is None and l2.mixer.window == 1 and l3.mixer.window == 300
    assert (cfg.loop.start, cfg.loop.stop, cfg.loop.times) == (1, 3, 3) and cfg.taps == 3 and cfg.eps == 1e-5
    _, b, _ = _spec("B")
    assert b.loop is None and b.layers[1].mixer.rot_dims == 4 and b.layers[1].mixer.rot_dim == 8
    _, d, _ = _spec("D")
    assert d.layers[0].mixer.window == 0 and d.bigram is None                          # no mask


@pytest.mark.parametrize("damage,text", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c.pop("canon"), "canon"),
    (lambda c: c["canon"].update(taps=0), "taps"),
    (lambda c: c["embedding"]["bigram"].pop("buckets"), "buckets"),
    (lambda c: c["embedding"]["bigram"].update(mul_prev=1.5), "mul_prev"),
    (lambda c: c["embedding"]["bigram"].pop("mul_cur"), "mul_cur"),
    (lambda c: c["layers"][0].update(type="conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].pop("dim"), "dim"),
    (lambda c: c["layers"][0]["mixer"].pop("rot_dim"), "rot_dim"),
    (lambda c: c["layers"][0]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][0]["mixer"].pop("kv_rank"), "kv_rank"),
    (lambda c: c["layers"][0]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][0]["mixer"]["rot"].pop("base"), "base"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=8), "dims"),                 # more than the part has
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=5), "dims"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "size"),
    (lambda c: c["layers"][0]["mlp"].update(kind="dense"), "dense"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=6), "top"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"]["expert"].update(limit=-1.0), "limit"),
    (lambda c: c["loop"].update(stop=5), "loop"),
    (lambda c: c["loop"].update(times=0), "times"),
    (lambda c: c.update(layers=[]), "layers"),
])
def test_a_configuration_that_cannot_be_is_refused_by_name(damage, text):
    from flambeau_amd.config.base import ConfigError
    from flambeau_amd.registry import config_from_dict
    raw = json.loads(json.dumps(CONFIGS["A"]["config"]))
    damage(raw)
    with pytest.raises(ConfigError) as e:
        config_from_dict(raw, "cfg")
    assert text in str(e.value)


def test_what_layers_and_embedding_keep_per_request():
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.models.decoder import DecoderModel
    from flambeau_amd.parts import PagedRowSpec
    from flambeau_amd.parts.base import RecordedCacheSpec
    _, cfg, spec = _spec("A")
    model = DecoderModel(spec, rt=None)
    specs, shares = model.cache_entries()
    assert len(specs) == 9 and shares == [None] * 9                         # eight layer runs and the embedding
    assert all(isinstance(s, RecordedCacheSpec) for s in specs[:8])
    assert specs[0].inner == PagedRowSpec(64, 13, 32)                       # a latent of 24 and a part of 6, in steps of 32
    assert specs[1].inner == PagedRowSpec(96, 70, 64) and specs[7].inner == PagedRowSpec(128, 300, 96)
    store = CacheStorage(specs, shares, torch.device("cpu"), torch.float32, n_pages=5, page_size=8, max_slots=3)
    # every pass of the loop has pages and kept inputs of its own; layers of equal rows and windows share tables
    assert len(store.pools) == 4 and [e.group for e in store.entries] == [0, 1, 2, 1, 2, 1, 2, 3, -1]
    rings = [e.records["input_conv"] for e in store.entries[:8]]
    assert all(tuple(r.shape) == (3, 3, 40) and r.dtype == torch.float32 for r in rings) and len({r.data_ptr() for r in rings}) == 8
    last = store.entries[8]
    assert tuple(last.state.shape) == (3, 2) and last.state.dtype == torch.int32 and last.kv is None
    kv = store.entries[1].kv
    assert (kv.width, kv.value_width, kv.page_size, kv.n_pages) == (96, 64, 8, 5)
    for r in rings:
        r.fill_(7.0)
    last.state.fill_(5)
    store.zero_slots([1])                                                   # a slot that is claimed again starts from zero, the others stay
    assert all((r[1] == 0).all() and (r[[0, 2]] == 7).all() for r in rings) and last.state.tolist() == [[5, 5], [0, 0], [5, 5]]
    assert store.bytes_per_token() == 4 * (96 + 3 * 160 + 3 * 96 + 224)
    # nothing keeps a decode step from being captured: single tokens write places they do not read
    assert model.capturable() and all(getattr(p, "graph_safe", True) for p in model.all_parts())
    assert all(c.graph_safe for c in model.mixer_classes())


def test_rows_that_are_values_in_part():
    """Rows of which only a part is summed have pages of their own kind; rows that are summed whole stay as they were."""
    from flambeau_amd.kernels.library import KernelError
    from flambeau_amd.kernels.ops import LatentLayerCache
    from flambeau_amd.parts import PagedRowSpec
    whole, part = PagedRowSpec(64, 9), PagedRowSpec(96, 9, 64)
    assert whole.page_group() != part.page_group() != PagedRowSpec(96, 9).page_group() and part.page_group().window == 9
    pool = part.allocate_pool(2, 4, 16, torch.float32, "cpu")
    assert tuple(pool.shape) == (2, 4, 16 * 160)
    view = part.layer_view(pool, 1)
    assert (view.width, view.value_width, view.page_size, view.n_pages) == (96, 64, 16, 4) and view.pool.data_ptr() == pool[1].data_ptr()
    v = whole.layer_view(whole.allocate_pool(1, 4, 16, torch.float32, "cpu"), 0)
    assert (v.width, v.value_width, v.page_size) == (64, 64, 16)
    assert (whole.bytes_per_token(2), part.bytes_per_token(2)) == (256, 320)
    with pytest.raises(KernelError):
        LatentLayerCache(pool[0], 16, 96, 96)


def test_tensor_names_and_random_weights(tmp_path):
    from flambeau_amd.models.decoder import DecoderModel
    d = write_model("A", tmp_path / "m")
    cfg, t = read_model(d)
    names = set(t)
    assert {"embed", "bigram", "embed.norm", "embed.norm.b", "final.norm", "final.norm.b", "head", "l0.norm1", "l0.norm1.b", "l0.norm1b",
            "l0.norm1b.b", "l0.norm2b", "l0.ls1", "l0.ls2", "l0.rg1", "l0.rg1.b", "l0.rg2", "l0.canon1", "l0.mix.dq", "l0.mix.dq.norm",
            "l0.mix.dkv", "l0.mix.uk", "l0.mix.g", "l0.mlp.router", "l0.mlp.e4.down"} <= names
    assert not any(n.startswith("l2.mlp") or n in ("l2.norm2", "l2.ls2", "l2.rg2", "l2.norm2b") for n in names)
    assert t["bigram"].shape == (32, 40) and t["l0.mix.uq"].shape == (3 * 16, 14) and t["l0.mix.dkv"].shape == (30, 40) and t["l0.canon1"].shape == (40, 3)
    _, _, spec = _spec("A")
    assert set(DecoderModel(spec, rt=None).manifest()) == names
    again = read_model(write_model("A", tmp_path / "m2"))[1]
    assert all(np.array_equal(t[n], again[n]) for n in names)
    assert "bigram" not in read_model(write_model("D", tmp_path / "d"))[1]


# ---------------------------------------------------------------- the plain implementation's own invariants
@pytest.mark.parametrize("name", list(CONFIGS))
def test_plain_logits_do_not_look_ahead(tmp_path, name):
    cfg, t = read_model(write_model(name, tmp_path / "m"))
    rng = np.random.default_rng(1)
    toks = [int(x) for x in rng.integers(0, cfg["vocab"], 30)]
    full = pl.forward(cfg, t, toks)
    assert full.shape == (30, cfg["vocab"]) and np.isfinite(full).all()
    assert np.allclose(pl.forward(cfg, t, toks[:11]), full[:11], atol=1e-10)
    changed = pl.forward(cfg, t, toks[:20] + [(toks[20] + 1) % cfg["vocab"]] + toks[21:])
    assert np.allclose(changed[:20], full[:20], atol=1e-10) and np.abs(changed[20] - full[20]).max() > 1e-3


def test_plain_mechanisms():
    rng = np.random.default_rng(0)
    assert pl.bigram_rows([5, 2, 0, 9], 7, 3, 2) == [7, (15 + 4) % 7, (6 + 0) % 7, (0 + 18) % 7]
    h = rng.normal(size=(9, 4))
    w = rng.normal(size=(4, 3))
    c = pl.causal_convolution(h, w)
    assert np.allclose(c[0], h[0] * w[:, 2]) and np.allclose(c[1], h[1] * w[:, 2] + h[0] * w[:, 1])
    assert np.allclose(c[5], h[5] * w[:, 2] + h[4] * w[:, 1] + h[3] * w[:, 0])
    m = pl.window_mask(6, 3)
    assert m[4].tolist() == [False, False, True, True, True, False] and m[0].tolist() == [True] + [False] * 5
    # rotation keeps lengths, and products depend on the distance alone
    a, b = rng.normal(size=(1, 6)), rng.normal(size=(1, 6))
    at = lambda v, p: pl.rotate(v, [p], 50.0, 6)[0]
    assert np.isclose(at(a, 7) @ at(b, 3), at(a, 104) @ at(b, 100)) and np.isclose(np.linalg.norm(at(a, 9)), np.linalg.norm(a))
    assert not np.isclose(at(a, 7) @ at(b, 3), at(a, 7) @ at(b, 4)) and np.allclose(at(a, 0), a[0])
    part = pl.rotate(rng.normal(size=(5, 2, 6)), np.arange(5), 50.0, 4)
    assert part.shape == (5, 2, 6)
    chosen, s = pl.route(np.log(np.array([[0.1, 0.4, 0.2, 0.3]])), 2)
    assert chosen.tolist() == [[1, 3]] and np.allclose(s, [[0.4, 0.3]])      # the scores as they are, not over their sum
    t = {"e.gate": np.eye(2), "e.up": np.eye(2), "e.down": np.eye(2)}
    y = pl.expert(np.array([[3.0, -2.0]]), t, "e.", 1.5)
    assert np.allclose(y, [[1.5 * pl.sigmoid(1.702 * 1.5) * 2.5, -2.0 * pl.sigmoid(1.702 * -2.0) * -0.5]])      # the gate is clamped above only
    assert pl.run_order({"layers": [0] * 4, "loop": {"start": 1, "stop": 3, "times": 2}}) == [0, 1, 2, 1, 2, 3]


def test_key_parts_follow_the_window():
    from flambeau_amd.kernels.latent_attention import key_splits
    from flambeau_amd.parts import HostBatch
    one = HostBatch([0], [1], [4000], [0], 1, 0)
    assert key_splits(one, 32) == 32 and key_splits(one, 32, 1024) == 16 and key_splits(one, 32, 40) == 1 and key_splits(one, 32, 1 << 20) == 32
