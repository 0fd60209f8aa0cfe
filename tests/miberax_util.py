"""Small Miberax configurations for the tests, and folders of random weights for them in which the numbers that plain
random weights would leave without effect (norm weights, decays, convolution taps, the router's correction, the four
numbers of the activation) are large enough to show, and in which scores differ enough for single keys to stand out."""
import json
import os

import numpy as np
import torch


def rotation(dims, base=10000.0, factor=None):
    out = {"base": base, "dims": dims}
    if factor:
        out["scaling"] = {"factor": factor}
    return out


def attention(heads, kv_heads, dim, vdim, scale, chunk=None, rot=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if chunk:
        m["mask"] = {"size": chunk}
    if rot:
        m["rot"] = rot
    return m


def delta(heads, kv_heads, dim, vdim, conv):
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "conv": conv}


def pair(left, right):
    return {"type": "parallel", "mixer": {"left": left, "right": right}}


def dense(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff})


def moe(layer, ff, limit, experts, top, identity=0, groups=None, scale=1.0, shared=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if identity:
        router["identity"] = identity
    if groups:
        router["groups"] = dict(zip(("count", "keep"), groups))
    mlp = {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": router}
    if shared:
        mlp["shared"] = {"ff": shared[0], "limit": shared[1]}
    return dict(layer, mlp=mlp)


def bare(layer):
    return dict(layer, mlp=None)


def config(vocab, width, eps, groups, layers):
    return {"architecture": "Miberax", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "layers": layers}


def every_expert(config_json):
    """The same model with every expert for every token (nothing is chosen: no near tie of a router)."""
    out = json.loads(json.dumps(config_json))
    for layer in out["layers"]:
        if layer["mlp"] is not None and layer["mlp"]["kind"] == "moe":
            r = layer["mlp"]["router"]
            r["top"] = r["experts"] + r.get("identity", 0)
            if "groups" in r:
                r["groups"]["keep"] = r["groups"]["count"]
    return out


# every kind of feed-forward and a layer without one; chunks that are no multiples of a page and a layer that sees every
# earlier position; part and whole rotations; groups of experts, experts that hand on their input, with and without a
# shared one; sizes that the matrix-core kernels take
B_A = config(131, 64, 1e-6, 2, [
    moe(pair(attention(4, 2, 32, 16, 0.25, chunk=37, rot=rotation(32, factor=3.0)), delta(4, 2, 16, 32, 4)), 32, 0.8, 6, 3,
        identity=2, groups=(4, 3), scale=1.5, shared=(64, 1.2)),
    dense(pair(attention(6, 3, 32, 16, 0.2, chunk=21, rot=rotation(16, 500.0)), delta(2, 2, 32, 48, 3)), 96),
    bare(pair(attention(4, 4, 48, 32, 0.2, chunk=64, rot=rotation(48)), delta(6, 3, 8, 16, 2))),
    moe(pair(attention(6, 2, 64, 32, 0.15, rot=rotation(64, 900.0, 2.0)), delta(3, 1, 16, 16, 1)), 64, 1.5, 5, 2),
])
# sizes that are multiples of nothing, groups that are no fours, as many key heads as heads and one key head for all, a
# chunk of one, nothing rotated, more taps than the one launch takes, key sizes that are no powers of two, one expert a
# token, more experts that hand on their input than others
B_B = config(97, 78, 1e-5, 3, [
    dense(pair(attention(3, 3, 10, 12, 0.3, chunk=7, rot=rotation(6, 300.0, 1.5)), delta(3, 3, 12, 20, 5)), 33),
    moe(pair(attention(5, 1, 14, 6, 0.25, chunk=11), delta(2, 1, 6, 7, 4)), 10, 0.5, 4, 1, identity=5, groups=(3, 1), scale=0.7,
        shared=(13, 0.7)),
    bare(pair(attention(2, 2, 6, 10, 0.4, chunk=1, rot=rotation(4)), delta(4, 1, 20, 5, 7))),
    moe(pair(attention(3, 3, 10, 10, 0.3, rot=rotation(10)), delta(1, 1, 36, 3, 2)), 7, 1.0, 3, 4, identity=1, scale=2.5),
])
# a larger one for prompts of hundreds of tokens: chunks over several pages and tiles, portions over several chunks of the
# recurrence, experts of sizes that the grouped kernels take, more than 64 router outputs, one group
B_C = config(500, 128, 1e-6, 1, [
    moe(pair(attention(8, 2, 48, 32, 0.2, chunk=150, rot=rotation(48, 5000.0, 2.0)), delta(4, 2, 32, 64, 4)), 64, 1.0, 8, 2,
        identity=2, groups=(5, 2), scale=2.0, shared=(128, 1.5)),
    dense(pair(attention(8, 2, 32, 16, 0.2, chunk=70, rot=rotation(32)), delta(2, 1, 64, 48, 4)), 160),
    moe(pair(attention(4, 4, 80, 64, 0.1, chunk=64, rot=rotation(32)), delta(2, 2, 128, 32, 3)), 32, 0.9, 60, 3, identity=12,
        groups=(6, 4), scale=1.3, shared=(96, 2.0)),
])
CONFIGS = {"A": B_A, "B": B_B, "C": B_C, "A every expert": every_expert(B_A), "C every expert": every_expert(B_C)}

_TINY_LEFT, _TINY_RIGHT = attention(1, 1, 4, 4, 0.5, chunk=2), delta(1, 1, 4, 4, 2)
# one mechanism each (SILENT: the mixer of the pair whose result counts zero times)
SINGLE = {
    "chunk": config(50, 48, 1e-6, 1, [bare(pair(attention(3, 3, 16, 12, 0.3, chunk=6, rot=rotation(8)), _TINY_RIGHT))]),
    "no chunk": config(50, 48, 1e-6, 4, [bare(pair(attention(4, 2, 32, 16, 0.3, rot=rotation(32, 100.0, 4.0)), _TINY_RIGHT))]),
    "delta": config(50, 48, 1e-6, 2, [bare(pair(_TINY_LEFT, delta(4, 2, 16, 12, 4)))]),
    "delta of odd sizes": config(50, 48, 1e-6, 2, [bare(pair(_TINY_LEFT, delta(3, 3, 10, 7, 6)))]),
    "both": config(50, 48, 1e-2, 3, [bare(pair(attention(2, 1, 16, 16, 0.3, chunk=8), delta(2, 2, 8, 8, 3)))]),
    "dense": config(50, 48, 1e-2, 1, [dense(pair(_TINY_LEFT, _TINY_RIGHT), 40)]),
    "experts": config(50, 48, 1e-6, 1, [moe(pair(_TINY_LEFT, _TINY_RIGHT), 20, 0.6, 7, 3, scale=3.0)]),
    "grouped experts": config(50, 48, 1e-6, 1, [moe(pair(_TINY_LEFT, _TINY_RIGHT), 20, 0.6, 9, 2, identity=3, groups=(4, 2))]),
    "shared": config(50, 64, 1e-6, 2, [moe(pair(_TINY_LEFT, _TINY_RIGHT), 32, 0.6, 4, 1, shared=(64, 0.3))]),
    "hands on": config(50, 64, 1e-6, 2, [moe(pair(_TINY_LEFT, _TINY_RIGHT), 32, 0.6, 2, 1, identity=4)]),
}
SILENT = {"chunk": "right", "no chunk": "right", "delta": "left", "delta of odd sizes": "left"}


def make_tensors(config_json, seed, std=0.1, silent=None):
    """name -> float32 tensor."""
    import hfee_amd  # noqa: F401
    from hfee_amd.config import config_from_dict
    from hfee_amd.engine.model import declared_tensors
    from hfee_amd.weights.random_init import random_tensors
    specs = [s for s in declared_tensors(config_from_dict(config_json)) if not s.optional]
    tensors = random_tensors(specs, seed, std, torch.float32, "cpu")
    g = torch.Generator().manual_seed(seed + 1)
    for name in list(tensors):
        t = tensors[name]
        rand = lambda: torch.randn(t.shape, generator=g)                     # noqa: E731
        if name == "embed":
            t = rand()
        elif name.endswith("norm1") or name.endswith("norm2") or name.endswith("norm"):
            t = 1.0 + rand() * 0.2
        elif name.endswith(".out"):
            t = (1.0 + rand() * 0.3) * (0.0 if silent and f".{silent}." in name else 1.0)
        elif name.endswith(".A_log"):            # (heads that hardly decay beside heads that do)
            t = -3.5 + 2.5 * torch.linspace(-1.0, 1.0, t.numel()) if t.numel() > 1 else torch.tensor([-4.0])
        elif name.endswith(".dt_bias"):
            t = rand() * 0.5
        elif name.endswith(".conv"):
            t = rand() * 0.6
        elif name.endswith(".act"):
            t = torch.tensor([0.8, -0.6, 0.5, 0.3]) + rand() * 0.1
        elif name.endswith(".correction"):       # (negative choice scores too)
            t = rand() * 0.15 - 0.1
        elif ".mlp." in name or name.endswith("right.b") or name.endswith("right.a"):
            t = rand() * 0.25
        elif ".mix." in name:
            t = rand() * t.shape[-1] ** -0.5 * 1.3
        tensors[name] = t.contiguous()
    return tensors


def make_folder(path, config_json, seed, dtype="float32", tensors=None, silent=None):
    """config.json + model.safetensors with seeded weights; returns the folder."""
    from hfee_amd.weights.safetensors_io import write_safetensors
    dt = {"float32": torch.float32, "bfloat16": torch.bfloat16}[dtype]
    tensors = make_tensors(config_json, seed, silent=silent) if tensors is None else tensors
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
