"""Small Fipitar configurations for the tests, and their random weights.

They differ from one another in every size and option, layer by layer: head counts from one to more than a tile of the
matrix cores holds, key and value sizes that differ either way and are multiples of nothing, of 8 or of 32, low ranks of
one and more, powers of the forget gate of one and more, latents narrower and wider than a wave, rotated parts of two
dims, of 32 and of more than 32, ladders of frequencies stretched, cut inside the ladder, and plain, heads that share keys
and heads that do not, scores with and without a cap, with and without a rotation, convolutions of one to six taps, groups
and norm parts of one and more, limits that bite always and almost never, layers without a feed-forward, factors that are
equal, negative and 1, widths and vocabularies that are no multiples of 8."""
import json

import torch

from flambeau_amd.weights import SafetensorsFile, write_random_model, write_safetensors


def rot(dims, base=100.0, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def gla(heads, dim, vdim, tau, decay_rank):
    return {"type": "gla", "mixer": dict(heads=heads, dim=dim, vdim=vdim, tau=tau, decay_rank=decay_rank)}


def latent(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, base=100.0, scaling=None):
    return {"type": "latent_attention", "mixer": dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank,
                                                      scale=scale, rot=rot(rot_dim, base, scaling))}


def left(heads, kv_heads, dim, vdim, scale, softcap=None, r=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale)
    if softcap:
        m["softcap"] = softcap
    if r:
        m["rot"] = r
    return m


def right(heads, vdim, state, groups, conv, norm_groups):
    return dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


def pair(l, r, left_scale, right_scale):
    return {"type": "parallel", "mixer": dict(left=l, right=r, left_scale=left_scale, right_scale=right_scale)}


def dense(ff, limit):
    return {"kind": "dense", "ff": ff, "limit": limit}


def model(vocab, width, eps, layers):
    return {"architecture": "Fipitar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": [dict(l, mlp=m) for l, m in layers]}


CONFIGS = {
    # every kind of layer, sizes that are multiples of nothing, a layer without a feed-forward
    "A": dict(config=model(83, 40, 1e-5, [
        (gla(3, 10, 7, 4.0, 5), dense(28, 0.8)),
        (latent(3, 10, 6, 12, 14, 24, 0.5, 1000.0, (4.0, 30, 8.0, 1.0)), dense(20, 2.0)),
        (pair(left(6, 2, 12, 9, 0.4, 5.0, rot(8)), right(4, 6, 10, 2, 4, 3), 0.7, 1.3), None),
        (gla(1, 33, 20, 1.0, 1), dense(36, 0.3)),
        (pair(left(3, 3, 7, 15, 0.5, 2.0, rot(2, 30.0)), right(2, 9, 5, 1, 1, 1), -0.5, 1.0), dense(24, 1.0)),
    ]), seed=3, std=0.15, page_size=8),
    # an odd width, no cap and no rotation on the left, a plain ladder, one head of everything, odd widths that cannot be joined
    "B": dict(config=model(61, 37, 3e-4, [
        (pair(left(1, 1, 5, 5, 0.9), right(3, 5, 7, 3, 2, 5), 1.0, 1.0), dense(11, 0.5)),
        (latent(2, 6, 2, 5, 9, 12, 0.8), None),
        (gla(2, 3, 3, 9.0, 2), dense(10, 1.5)),
    ]), seed=11, std=0.3, page_size=16),
    # sizes that run on the matrix cores in bfloat16: more heads than a tile of 16, pages of 16
    "C": dict(config=model(150, 64, 1e-5, [
        (latent(20, 32, 32, 48, 48, 64, 0.2, 5000.0, (8.0, 64, 16.0, 2.0)), dense(96, 1.5)),
        (gla(4, 32, 48, 16.0, 16), dense(64, 0.6)),
        (pair(left(8, 2, 64, 40, 0.15, 10.0, rot(32, 2500.0)), right(4, 16, 32, 2, 4, 2), 0.8, 1.1), dense(64, 3.0)),
        (pair(left(34, 2, 32, 32, 0.2, 4.0, rot(32, 700.0)), right(8, 8, 64, 8, 3, 4), 1.5, 0.25), None),
    ]), seed=21, std=0.12, page_size=16),
    # latents as wide as the kernels deal out, rotated parts wider than 32, six taps, values wider than keys
    "D": dict(config=model(90, 48, 1e-6, [
        (pair(left(4, 4, 24, 56, 0.2, 30.0, rot(24, 400.0)), right(1, 40, 16, 1, 6, 8), 1.1, 0.6), dense(40, 0.7)),
        (latent(3, 16, 40, 24, 16, 160, 0.2, 9000.0, (32.0, 4096, 32.0, 1.0)), dense(32, 4.0)),
        (latent(6, 24, 16, 16, 24, 512, 0.1), None),
        (gla(5, 64, 24, 2.5, 9), None),
    ]), seed=41, std=0.2, page_size=16),
}

STORE = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def write_model(name, out_dir, store="float32", sharpen=1.0, edit=None):
    """The folder of a configuration.  ``sharpen`` multiplies every score scale: softmax becomes peaked and single keys
    carry the output; ``edit(tensors)`` changes tensors before they are written."""
    c = CONFIGS[name]
    config = json.loads(json.dumps(c["config"]))
    for layer in config["layers"]:
        for m in (layer["mixer"], layer["mixer"].get("left", {})):
            if "scale" in m:
                m["scale"] *= sharpen
    d = write_random_model(config, out_dir, seed=c["seed"], std=c["std"], gain_std=0.1, store_dtype=STORE[store])
    for layer in config["layers"]:                                           # (a file's ranks are its tensors')
        layer["mixer"].pop("decay_rank", None)
    (d / "config.json").write_text(json.dumps(config, indent=1))             # exactly the keys the design has
    if edit:
        f = SafetensorsFile(d / "model.safetensors")
        tensors = {n: f.read(n) for n in f.names()}
        f.close()
        edit(tensors)
        write_safetensors(d / "model.safetensors", tensors)
    return d


def long_memory(tensors):
    """Recurrences that forget little, sinks that weigh as much as a few keys."""
    for n, v in tensors.items():
        if n.endswith("a2.b"):
            tensors[n] = (v.float() + 6.0).to(v.dtype)
        elif n.endswith("A_log"):
            tensors[n] = (v.float() * 0 - 4.0).to(v.dtype)
        elif n.endswith("sink"):
            tensors[n] = (v.float() + 1.5).to(v.dtype)


def read_model(model_dir):
    """``(config dictionary, {name: float64 array})`` as the plain implementation takes them."""
    cfg = json.loads((model_dir / "config.json").read_text())
    f = SafetensorsFile(model_dir / "model.safetensors")
    tensors = {n: f.read(n).to(torch.float64).numpy() for n in f.names()}
    f.close()
    return cfg, tensors
