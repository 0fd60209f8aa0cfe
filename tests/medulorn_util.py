"""Small Medulorn configurations for the tests, and folders of random weights for them in which the numbers
that plain random weights would leave without effect (norm weights, sinks, biases, the token shift, the router's bias)
are large enough to show, and in which scores differ enough for single keys to stand out."""
import json
import os

import numpy as np
import torch


def rotation(dims, base=10000.0, scaling=None):
    out = {"base": base, "dims": dims}
    if scaling:
        out["scaling"] = dict(zip(("factor", "low", "high", "original"), scaling))
    return out


def attention(heads, kv_heads, dim, vdim, scale, chunk=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot:
        m["rot"] = rot
    return {"type": "attention", "mixer": m}


def window(heads, kv_heads, dim, vdim, scale, size=None, keep=0, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        m["mask"] = {"size": size}
        if keep:
            m["mask"]["keep_first"] = keep
    if rot:
        m["rot"] = rot
    return m


def lightning(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def pair(left, right, left_scale=1.0, right_scale=1.0):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": left_scale, "right_scale": right_scale}}


def dense(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff})


def moe(layer, ff, limit, experts, top, shared=None):
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": {"experts": experts, "top": top}}
    if shared:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    return dict(layer, mlp=mlp)


def bare(layer):
    return dict(layer, mlp=None)


def config(vocab, width, eps, alpha, layers, scale=1.0, softcap=None):
    out = {"architecture": "Medulorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
           "postln_alpha": alpha, "layers": layers}
    if softcap:
        out["logit_softcap"] = softcap
    return out


def every_expert(config_json):
    """The same model with every expert for every token (nothing is chosen: no near tie of a router)."""
    out = json.loads(json.dumps(config_json))
    for layer in out["layers"]:
        if layer["mlp"] is not None and layer["mlp"]["kind"] == "moe":
            layer["mlp"]["router"]["top"] = layer["mlp"]["router"]["experts"]
    return out


# both mixers twice, every kind of feed-forward and a layer without one; chunks, windows and kept tokens that are no
# multiples of a page; sizes that the matrix-core kernels take
M_A = config(131, 64, 1e-6, 1.7, [
    moe(attention(4, 2, 32, 16, 0.25, chunk=37, rot=rotation(32)), 32, 0.8, 6, 2, shared=(64, 1.2)),
    dense(pair(window(4, 2, 32, 16, 0.2, size=19, keep=3, rot=rotation(16, 500.0, (4.0, 1.0, 4.0, 64))),
               lightning(2, 16, 32, (0.9, 0.97)), 0.7, 1.3), 96),
    bare(attention(6, 3, 32, 16, 0.2, chunk=21, rot=rotation(16))),
    moe(pair(window(6, 2, 48, 32, 0.15, size=40, keep=18, rot=rotation(48)), lightning(3, 8, 16, (0.5, 1.0, 0.99))), 32, 1.5, 5, 3),
], scale=8.0, softcap=9.0)
# sizes that are multiples of nothing, as many key heads as heads and one key head for all, a chunk and a window of
# one, nothing rotated, no cap, alpha of one, more kept tokens than the window holds, every expert for every token
M_B = config(97, 74, 1e-5, 1.0, [
    dense(pair(window(3, 3, 10, 12, 0.3, size=7, keep=1, rot=rotation(6, 300.0)), lightning(3, 12, 20, (0.8, 0.99, 0.95)), 1.0, 0.5), 33),
    moe(attention(5, 1, 14, 6, 0.25, chunk=11), 10, 0.5, 4, 4, shared=(13, 0.7)),
    bare(pair(window(4, 1, 20, 6, 0.2, size=1, keep=9, rot=rotation(20)), lightning(1, 5, 7, (0.999,)))),
    dense(attention(2, 2, 6, 10, 0.4, chunk=1, rot=rotation(4)), 21),
    moe(attention(3, 3, 10, 10, 0.3), 7, 1.0, 3, 1),
])
# a larger one for prompts of hundreds of tokens: chunks and windows over several pages and tiles, kept tokens over
# more than a tile, experts of sizes that the grouped kernels take
M_C = config(500, 128, 1e-6, 2.0, [
    moe(attention(8, 2, 48, 32, 0.2, chunk=150, rot=rotation(48, 5000.0)), 64, 1.0, 8, 2, shared=(128, 1.5)),
    moe(pair(window(8, 2, 32, 16, 0.2, size=70, keep=5, rot=rotation(32, 10000.0, (8.0, 1.0, 4.0, 256))),
             lightning(4, 32, 32, (0.95, 0.98, 0.99, 0.999)), 0.6, 0.8), 96, 1.2, 8, 2, shared=(64, 2.0)),
    dense(attention(4, 4, 80, 64, 0.1, chunk=64, rot=rotation(32)), 160),
    moe(pair(window(6, 2, 96, 64, 0.1, size=33, keep=40, rot=rotation(96)), lightning(2, 64, 48, (0.9, 0.9995))), 64, 0.9, 8, 3),
], scale=11.0, softcap=20.0)
CONFIGS = {"A": M_A, "B": M_B, "C": M_C, "A every expert": every_expert(M_A), "C every expert": every_expert(M_C)}

# one mechanism each
SINGLE = {
    "chunk": config(50, 48, 1e-6, 1.5, [bare(attention(3, 3, 16, 12, 0.3, chunk=6, rot=rotation(8)))]),
    "no chunk": config(50, 48, 1e-6, 1.5, [bare(attention(4, 2, 32, 16, 0.3, rot=rotation(32)))]),
    "window": config(50, 48, 1e-6, 0.5, [bare(pair(window(4, 2, 32, 16, 0.3, size=6, keep=2, rot=rotation(32)),
                                                   lightning(1, 1, 1, (0.0,)), 1.0, 0.0))]),
    "lightning": config(50, 48, 1e-6, 1.0, [bare(pair(window(1, 1, 16, 16, 0.3, size=1), lightning(3, 8, 12, (0.9, 0.6, 1.0)), 0.0, 1.0))]),
    "dense": config(50, 48, 1e-6, 2.0, [dense(attention(1, 1, 4, 4, 0.5, chunk=2), 40)], scale=3.0),
    "experts": config(50, 48, 1e-6, 0.8, [moe(attention(1, 1, 4, 4, 0.5, chunk=2), 20, 0.6, 7, 3)]),
    "shared": config(50, 64, 1e-6, 0.8, [moe(attention(1, 1, 4, 4, 0.5, chunk=2), 32, 0.6, 4, 1, shared=(64, 0.3))], softcap=2.0),
    "two bare layers": config(61, 58, 1e-6, 1.2, [bare(attention(2, 1, 14, 10, 0.3, chunk=9, rot=rotation(14))),
                                                   bare(attention(2, 2, 6, 6, 0.3, chunk=4))]),
}


def make_tensors(config_json, seed, std=0.1):
    """name -> float32 tensor."""
    import hfee_amd  # noqa: F401
    from hfee_amd.config import config_from_dict
    from hfee_amd.engine.model import declared_tensors
    from hfee_amd.weights.random_init import random_tensors
    cfg = config_from_dict(config_json)
    tensors = random_tensors(declared_tensors(cfg), seed, std, torch.float32, "cpu")
    g = torch.Generator().manual_seed(seed + 1)
    for name in list(tensors):
        t = tensors[name]
        rand = lambda: torch.randn(t.shape, generator=g)                     # noqa: E731
        if name.endswith("q.norm") or name.endswith("k.norm"):
            t = 1.5 + rand() * 0.5
        elif name.endswith("norm1") or name.endswith("norm2") or name.endswith("norm"):
            t = 1.0 + rand() * 0.2
        elif name.endswith(".sink"):
            t = rand() * 1.5
        elif name.endswith(".shift"):
            t = torch.rand(t.shape, generator=g)
        elif name.endswith(".b"):
            t = rand() * 0.4
        elif name.endswith(".router") or ".mlp." in name:
            t = rand() * 0.25
        tensors[name] = t
    return tensors


def make_folder(path, config_json, seed, dtype="float32", std=0.1, tensors=None):
    """config.json + model.safetensors with seeded weights; returns the folder."""
    from hfee_amd.weights.safetensors_io import write_safetensors
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype]
    tensors = make_tensors(config_json, seed, std) if tensors is None else tensors
    tensors = {n: t.to(dt) for n, t in tensors.items()}
    os.makedirs(path, exist_ok=True)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(config_json, f)
    write_safetensors(os.path.join(str(path), "model.safetensors"), tensors, metadata={"format": "pt"})
    return str(path)


def load_plain(folder):
    """(config.json's keys, name -> tensor) of a folder, for the plain implementation."""
    from safetensors.torch import load_file
    with open(os.path.join(folder, "config.json")) as f:
        cj = json.load(f)
    return cj, load_file(os.path.join(folder, "model.safetensors"))


def rel(a, b):
    a, b = np.asarray(a, dtype=np.float64), np.asarray(b, dtype=np.float64)
    return float(np.abs(a - b).max() / np.abs(b).max())
