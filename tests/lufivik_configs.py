"""Small Lufivik configurations for the tests, and their random weights.

They differ from one another in every size and option, layer by layer: head counts from one to more than a tile of the
matrix cores holds, unrotated, rotated and value sizes that differ and are no multiples of 8 (or of anything), latents
narrower and wider than a wave and no multiples of 32, rotated parts of two dims, of 32 and of more than 32, rotated as
a whole or in part, windows of one key, of a few, across pages and beyond 256 keys, and none, convolutions of one to
six taps, one, some and all experts per token, limits that bite always and almost never, layers without a
feed-forward, loops over a stretch in the middle, over everything, one pass, three passes and no loop, tables of token
pairs with few and many buckets and none, widths and vocabularies that are no multiples of 8."""
import json

import torch

from flambeau_amd.weights import SafetensorsFile, write_random_model, write_safetensors


def att(heads, dim, rot_dim, vdim, q_rank, kv_rank, scale, window, base=100.0, dims=None):
    m = dict(heads=heads, dim=dim, rot_dim=rot_dim, vdim=vdim, q_rank=q_rank, kv_rank=kv_rank, scale=scale,
             rot={"base": base, "dims": rot_dim if dims is None else dims})
    if window is not None:                  # (None: no mask, every earlier key is seen)
        m["mask"] = {"size": window}
    return {"type": "latent_attention", "mixer": m}


def moe(experts, top, ff, limit):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff, "limit": limit}}


def model(vocab, width, eps, layers, taps, loop=None, bigram=None):
    cfg = {"architecture": "Lufivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps},
           "layers": [dict(l, mlp=m) for l, m in layers]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    if bigram:
        cfg["embedding"] = {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}
    return cfg


CONFIGS = {
    # a loop over a stretch in the middle, three passes; windows that differ from layer to layer; a layer without a
    # feed-forward inside the loop; sizes that are multiples of nothing
    "A": dict(config=model(83, 40, 1e-5, [
        (att(3, 10, 6, 12, 14, 24, 0.5, 13), moe(5, 2, 16, 0.8)),
        (att(2, 9, 4, 7, 11, 40, 0.6, 70, base=1000.0), moe(3, 3, 12, 2.0)),
        (att(5, 8, 2, 5, 9, 18, 0.7, 1), None),
        (att(1, 20, 10, 33, 21, 70, 0.4, 300, base=30.0), moe(4, 1, 20, 0.3)),
    ], taps=3, loop=(1, 3, 3), bigram=(31, 7, 3)), seed=3, std=0.12, page_size=8),
    # no loop, a convolution of one tap, one expert alone, a table of two buckets, an odd width
    "B": dict(config=model(61, 37, 3e-4, [
        (att(2, 6, 4, 6, 5, 9, 0.9, 20), moe(1, 1, 10, 1.0)),
        (att(4, 5, 8, 3, 7, 12, 0.8, 5, dims=4), None),
    ], taps=1, bigram=(2, 1, 1)), seed=11, std=0.3, page_size=16),
    # sizes that run on the matrix cores in bfloat16: more heads than a tile of 16, pages of 16; the whole model is the loop
    "C": dict(config=model(150, 64, 1e-5, [
        (att(20, 32, 32, 48, 48, 64, 0.2, 64), moe(4, 4, 32, 1.5)),
        (att(4, 40, 64, 16, 32, 96, 0.15, 33, base=5000.0), moe(6, 2, 32, 0.5)),
    ], taps=5, loop=(0, 2, 2), bigram=(97, 13, 29)), seed=21, std=0.12, page_size=16),
    # no table of pairs, no masks, six taps, a loop of one pass, a latent as wide as the kernels of single tokens deal out
    "D": dict(config=model(90, 48, 1e-6, [
        (att(3, 16, 40, 24, 16, 160, 0.2, None), moe(3, 1, 24, 0.7)),
        (att(6, 24, 16, 16, 24, 512, 0.1, 50), moe(2, 2, 16, 4.0)),
    ], taps=6, loop=(1, 2, 1)), seed=41, std=0.2, page_size=16),
}

STORE = {"float32": torch.float32, "bfloat16": torch.bfloat16}


def write_model(name, out_dir, store="float32", sharpen=1.0, edit=None):
    """The folder of a configuration.  ``sharpen`` multiplies every score scale: softmax becomes peaked and single keys
    carry the output; ``edit(tensors)`` changes tensors before they are written."""
    c = CONFIGS[name]
    config = json.loads(json.dumps(c["config"]))
    for layer in config["layers"]:
        layer["mixer"]["scale"] *= sharpen
    d = write_random_model(config, out_dir, seed=c["seed"], std=c["std"], gain_std=0.1, store_dtype=STORE[store])
    (d / "config.json").write_text(json.dumps(config, indent=1))             # exactly the keys the design has
    if edit:
        f = SafetensorsFile(d / "model.safetensors")
        tensors = {n: f.read(n) for n in f.names()}
        f.close()
        edit(tensors)
        write_safetensors(d / "model.safetensors", tensors)
    return d


def read_model(model_dir):
    """``(config dictionary, {name: float64 array})`` as the plain implementation takes them."""
    cfg = json.loads((model_dir / "config.json").read_text())
    f = SafetensorsFile(model_dir / "model.safetensors")
    tensors = {n: f.read(n).to(torch.float64).numpy() for n in f.names()}
    f.close()
    return cfg, tensors
