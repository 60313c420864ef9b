"""Fipitar without a GPU: its configuration, its description as parts, what its layers keep per request, its tensor names,
random weights as a folder, and the plain implementation's own invariants."""
import json

import numpy as np
import pytest
import torch

import plain_fipitar as pf
from fipitar_configs import CONFIGS, read_model, rot, write_model


def _spec(name):
    from flambeau_amd.registry import config_from_dict
    arch, cfg = config_from_dict(CONFIGS[name]["config"], "test")
    return arch, cfg, arch.build_spec(cfg)


def test_the_architecture_is_found_by_its_name():
    from flambeau_amd.registry import known_architectures
    assert {"Fipitar", "Lufivik", "Lenedra", "Fitevik", "Bugidra", "Kuvidra", "MistralForCausalLM"} <= set(known_architectures())
    arch, cfg, spec = _spec("A")
    assert arch.name == "Fipitar" and cfg.width == 40 and cfg.vocab_size == 83 and not spec.tied_head and spec.embedding is None
    assert all(l.block.kind == "outnorm" and l.block.params["norm"].kind == "layernorm" for l in spec.layers)
    kinds = [l.block.params["mixer"].kind for l in spec.layers]
    assert kinds == ["gated_linear_attention", "latent_attention", "side_by_side", "gated_linear_attention", "side_by_side"]
    assert [l.block.params["feed_forward"] is None for l in spec.layers] == [False, False, True, False, False]
    assert spec.layers[0].block.params["feed_forward"].params["alpha"] == 1.702
    p = spec.layers[2].block.params["mixer"].params
    assert p["factors"] == (0.7, 1.3) and p["normed"] is False and p["left"].params["sink"] == 0.0 and p["left"].params["gate_per"] == "head"
    assert spec.layers[1].block.params["mixer"].params["position"].kind == "rope_blended"
    assert spec.layers[1].block.params["mixer"].params["position"].params["layout"] == "interleaved"
    _, _, b = _spec("B")
    assert b.layers[0].block.params["mixer"].params["left"].params["position"].kind == "none"
    assert b.layers[1].block.params["mixer"].params["position"].kind == "rope_interleaved"


def test_every_size_comes_from_the_file():
    _, cfg, _ = _spec("A")
    g, l, p = (cfg.layers[i].mixer for i in range(3))
    assert (g.heads, g.dim, g.vdim, g.tau, g.decay_rank) == (3, 10, 7, 4.0, 5)
    assert (l.heads, l.dim, l.rot_dim, l.vdim, l.q_rank, l.kv_rank, l.scale, l.rot.base, l.rot.dims) == (3, 10, 6, 12, 14, 24, 0.5, 1000.0, 6)
    assert (l.rot.scaling.factor, l.rot.scaling.original, l.rot.scaling.fast, l.rot.scaling.slow) == (4.0, 30, 8.0, 1.0)
    assert (p.left.heads, p.left.kv_heads, p.left.dim, p.left.vdim, p.left.scale, p.left.softcap, p.left.rot.dims) == (6, 2, 12, 9, 0.4, 5.0, 8)
    assert (p.right.heads, p.right.vdim, p.right.state, p.right.groups, p.right.conv, p.right.norm_groups) == (4, 6, 10, 2, 4, 3)
    assert (p.left_scale, p.right_scale) == (0.7, 1.3) and cfg.layers[2].mlp is None and cfg.eps == 1e-5
    assert (cfg.layers[0].mlp.ff, cfg.layers[0].mlp.limit) == (28, 0.8)


def test_the_rank_of_the_decay_comes_from_its_tensor(tmp_path):
    from flambeau_amd.config.base import ConfigError
    from flambeau_amd.registry import config_from_dict, config_from_dir
    d = write_model("A", tmp_path / "m")
    raw = json.loads((d / "config.json").read_text())
    assert not any("decay_rank" in l["mixer"] for l in raw["layers"])
    _, cfg = config_from_dir(d)
    assert cfg.layers[0].mixer.decay_rank == 5 and cfg.layers[3].mixer.decay_rank == 1
    with pytest.raises(ConfigError, match="decay_rank"):
        config_from_dict(raw, "cfg")


@pytest.mark.parametrize("damage,text", [
    (lambda c: c.pop("width"), "width"),
    (lambda c: c.pop("vocab"), "vocab"),
    (lambda c: c["norm"].pop("eps"), "eps"),
    (lambda c: c["layers"][0].update(type="conv"), "conv"),
    (lambda c: c["layers"][0]["mixer"].pop("tau"), "tau"),
    (lambda c: c["layers"][0]["mixer"].update(tau=0.0), "tau"),
    (lambda c: c["layers"][0]["mixer"].pop("vdim"), "vdim"),
    (lambda c: c["layers"][0]["mlp"].update(kind="moe"), "moe"),
    (lambda c: c["layers"][0]["mlp"].pop("limit"), "limit"),
    (lambda c: c["layers"][0]["mlp"].update(limit=-1.0), "limit"),
    (lambda c: c["layers"][1]["mixer"].pop("rot_dim"), "rot_dim"),
    (lambda c: c["layers"][1]["mixer"].pop("q_rank"), "q_rank"),
    (lambda c: c["layers"][1]["mixer"].pop("scale"), "scale"),
    (lambda c: c["layers"][1]["mixer"].pop("rot"), "rot"),
    (lambda c: c["layers"][1]["mixer"]["rot"].update(dims=8), "dims"),                  # more than the part has
    (lambda c: c["layers"][1]["mixer"]["rot"]["scaling"].pop("slow"), "slow"),
    (lambda c: c["layers"][2]["mixer"]["left"].update(kv_heads=4), "key/value heads"),
    (lambda c: c["layers"][2]["mixer"]["left"]["rot"].update(dims=5), "dims"),
    (lambda c: c["layers"][2]["mixer"]["left"].update(softcap=0.0), "softcap"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(groups=3), "groups"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(norm_groups=5), "norm_groups"),
    (lambda c: c["layers"][2]["mixer"]["right"].update(conv=0), "conv"),
    (lambda c: c["layers"][2]["mixer"].pop("right_scale"), "right_scale"),
    (lambda c: c["layers"][2]["mixer"].pop("right"), "right"),
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


@pytest.mark.parametrize("change,text", [
    (lambda m: m[0].update(dim=513), "dim"), (lambda m: m[1].update(kv_rank=2000), "kv_rank"),
    (lambda m: m[2]["left"].update(dim=300), "head_dim"), (lambda m: m[2]["right"].update(state=513), "state"),
])
def test_sizes_beyond_the_kernels_are_refused_when_the_model_is_built(change, text):
    from flambeau_amd.config.base import ConfigError
    from flambeau_amd.models.decoder import DecoderModel
    from flambeau_amd.registry import config_from_dict
    raw = json.loads(json.dumps(CONFIGS["A"]["config"]))
    change([l["mixer"] for l in raw["layers"]])
    arch, cfg = config_from_dict(raw, "cfg")
    with pytest.raises(ConfigError, match=text):
        DecoderModel(arch.build_spec(cfg), rt=None)


def test_what_layers_keep_per_request():
    from flambeau_amd.cache.storage import CacheStorage
    from flambeau_amd.models.decoder import DecoderModel
    from flambeau_amd.parts import JoinedCacheSpec, PagedKVSpec, PagedRowSpec, StateSpec
    _, cfg, spec = _spec("A")
    model = DecoderModel(spec, rt=None)
    specs, shares = model.cache_entries()
    assert shares == [None] * 5
    assert specs[0] == StateSpec((3 * 10 * 7,)) and specs[1] == PagedRowSpec(64, 0, 32) and specs[3] == StateSpec((33 * 20,))
    assert isinstance(specs[2], JoinedCacheSpec) and specs[2].paged == PagedKVSpec(2, 16)
    # 4 heads x 10 x 6 floats of state, then 4 inputs of 24 + 2 x 20 channels
    assert specs[2].states[1] == StateSpec((240 + 4 * 64,)) and specs[4].paged == PagedKVSpec(3, 16)
    store = CacheStorage(specs, shares, torch.device("cpu"), torch.float32, n_pages=5, page_size=8, max_slots=3)
    assert len(store.pools) == 3 and [e.group for e in store.entries] == [-1, 0, 1, -1, 2]
    states = [e.state for e in store.entries if e.state is not None]
    assert len(states) == 4 and all(s.dtype == torch.float32 and s.shape[0] == 3 for s in states)
    for s in states:
        s.fill_(7.0)
    store.zero_slots([1])                                                   # a slot that is claimed again starts from zero, the others stay
    assert all((s[1] == 0).all() and (s[[0, 2]] == 7).all() for s in states)
    # its steps are recorded and replayed; a step that advances a state is not run twice to be captured
    assert model.replayable() and model.capturable() and not all(getattr(c, "graph_safe", False) for c in model.mixer_classes())


def test_tensor_names_and_random_weights(tmp_path):
    from flambeau_amd.models.decoder import DecoderModel
    d = write_model("A", tmp_path / "m")
    cfg, t = read_model(d)
    names = set(t)
    assert {"embed", "final.norm", "final.norm.b", "head", "l0.norm1", "l0.norm1.b", "l0.norm2.b", "l0.mix.a1", "l0.mix.a2", "l0.mix.a2.b", "l0.mix.norm",
            "l0.mlp.gate", "l1.mix.dq.norm", "l1.mix.sink", "l2.mix.left.q.norm", "l2.mix.left.g", "l2.mix.right.in", "l2.mix.right.conv",
            "l2.mix.right.conv.b", "l2.mix.right.dt_bias", "l2.mix.right.A_log", "l2.mix.right.D", "l2.mix.right.norm", "l2.mix.right.o"} <= names
    assert not any(n.startswith(("l2.mlp", "l2.norm2")) for n in names) and "l1.mix.g" not in names
    assert t["l0.mix.a1"].shape == (5, 40) and t["l0.mix.a2"].shape == (30, 5) and t["l2.mix.left.g"].shape == (6, 40)
    assert t["l2.mix.right.in"].shape == (24 + 64 + 4, 40) and t["l2.mix.right.conv"].shape == (64, 4) and t["l1.mix.dkv"].shape == (30, 40)
    _, _, spec = _spec("A")
    assert set(DecoderModel(spec, rt=None).manifest()) == names
    again = read_model(write_model("A", tmp_path / "m2"))[1]
    assert all(np.array_equal(t[n], again[n]) for n in names)


# ---------------------------------------------------------------- the plain implementation's own invariants
@pytest.mark.parametrize("name", list(CONFIGS))
def test_plain_logits_do_not_look_ahead(tmp_path, name):
    cfg, t = read_model(write_model(name, tmp_path / "m"))
    rng = np.random.default_rng(1)
    toks = [int(x) for x in rng.integers(0, cfg["vocab"], 30)]
    full = pf.forward(cfg, t, toks)
    assert full.shape == (30, cfg["vocab"]) and np.isfinite(full).all()
    assert np.allclose(pf.forward(cfg, t, toks[:11]), full[:11], atol=1e-10)
    changed = pf.forward(cfg, t, toks[:20] + [(toks[20] + 1) % cfg["vocab"]] + toks[21:])
    assert np.allclose(changed[:20], full[:20], atol=1e-10) and np.abs(changed[20] - full[20]).max() > 1e-3


def test_plain_mechanisms():
    rng = np.random.default_rng(0)
    # a sink takes its share of the weights and nothing else changes
    s = rng.normal(size=(5, 5))
    w, ws = pf.causal_softmax(s, None), pf.causal_softmax(s, 0.7)
    assert np.allclose(w.sum(axis=1), 1.0) and np.allclose(ws / ws.sum(axis=1, keepdims=True), w)
    assert np.isclose(ws[0, 0], np.exp(s[0, 0]) / (np.exp(s[0, 0]) + np.exp(0.7))) and (np.triu(w, 1) == 0).all()
    assert np.isclose(pf.causal_softmax(s, 0.0)[0, 0], np.exp(s[0, 0]) / (1 + np.exp(s[0, 0])))
    # rotation keeps lengths, products depend on the distance alone, the two layouts pair other dims
    a, b = rng.normal(size=6), rng.normal(size=6)
    for inter in (False, True):
        turned = lambda v: pf.rotate(np.tile(v, (110, 1)), rot(6, 50.0), inter)
        assert np.isclose(turned(a)[7] @ turned(b)[3], turned(a)[104] @ turned(b)[100]) and np.allclose(turned(a)[0], a)
        assert np.isclose(np.linalg.norm(turned(a)[9]), np.linalg.norm(a)) and not np.isclose(turned(a)[7] @ turned(b)[3], turned(a)[7] @ turned(b)[4])
    v = np.tile(a, (3, 1))
    assert np.allclose(np.hypot(*pf.rotate(v, rot(6), True)[2][[2, 3]]), np.hypot(a[2], a[3]))
    assert np.allclose(np.hypot(*pf.rotate(v, rot(6), False)[2][[1, 4]]), np.hypot(a[1], a[4]))
    assert np.allclose(pf.rotate(v, rot(4), True)[:, 4:], a[4:])
    # a stretched ladder: fast dims keep their frequency, slow ones are divided, and the magnitude follows the factor
    f, m = pf.frequencies(rot(16, 10000.0, (8.0, 4096, 32.0, 1.0)))
    f0, one = pf.frequencies(rot(16, 10000.0))
    assert one == 1.0 and np.isclose(m, 0.1 * np.log(8.0) + 1) and np.isclose(f[0], f0[0]) and np.isclose(f[-1], f0[-1] / 8.0)
    assert all(y / 8 - 1e-15 <= x <= y for x, y in zip(f, f0))
    # convolution
    h, w = rng.normal(size=(9, 4)), rng.normal(size=(4, 3))
    c = pf.causal_convolution(h, w, np.arange(4.0))
    assert np.allclose(c[0], h[0] * w[:, 2] + np.arange(4)) and np.allclose(c[5], h[5] * w[:, 2] + h[4] * w[:, 1] + h[3] * w[:, 0] + np.arange(4))
    # the gate is clamped above only, the other half on both sides
    t = {"e.gate": np.eye(2), "e.up": np.eye(2), "e.down": np.eye(2)}
    y = pf.clamped_ff(np.array([[3.0, -2.0]]), {"limit": 1.5}, t, "e.")
    assert np.allclose(y, [[1.5 * pf.sigmoid(1.702 * 1.5) * 2.5, -2.0 * pf.sigmoid(1.702 * -2.0) * -0.5]])


def test_the_framework_s_ladder_is_the_plain_one():
    from flambeau_amd.parts.rope import blended_frequencies
    for dims, base, sc in ((6, 1000.0, (4.0, 30, 8.0, 1.0)), (64, 5e5, (8.0, 8192, 4.0, 1.0)), (2, 30.0, (2.0, 16, 32.0, 1.0)), (128, 1e4, (1.0, 4096, 32.0, 1.0))):
        f, m = blended_frequencies(dims, base, *sc)
        want, mag = pf.frequencies(rot(dims, base, sc))
        assert np.allclose(f, want, rtol=1e-14) and np.isclose(m, mag)
