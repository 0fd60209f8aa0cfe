"""A plain, slow Medulorn decoder in float64 torch on the CPU, one function per mechanism, written from
the design's equations.  It shares no code with hfee_amd: the tests compare the engine with it.

Notation.  x: the residual stream [T, width] of one sequence whose first token sits at position 0.
`w`: a dict from tensor names to tensors (linear weights [out, in], applied as W x).  `m`: the "mixer"
dict of a layer's entry in config.json (or one of the two of a pair).  Every function takes the whole
sequence at once; the recurrence walks over it token by token, so cutting a sequence can change nothing here.
"""
from __future__ import annotations

import math

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def scalar_norm(x, gain, eps):
    """One number for all coordinates."""
    return rms(x, eps) * gain


def silu(z):
    return z * torch.sigmoid(z)


def token_shift(h, mu):
    """h_t + (h_(t-1) - h_t) * mu, the token before the first one being zeros."""
    before = torch.cat([torch.zeros_like(h[:1]), h[:-1]], dim=0)
    return h + (before - h) * mu


def rotation_frequencies(rot):
    out = []
    for i in range(rot["dims"] // 2):
        f = rot["base"] ** (-2.0 * i / rot["dims"])
        sc = rot.get("scaling")
        if sc is not None:
            length = 2.0 * math.pi / f
            if length > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            elif length >= sc["original"] / sc["high"]:
                s = (sc["original"] / length - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def rotate(x, rot):
    """x [T, heads, dim]: pairs (i, i + dims/2) of the first `dims` dims of each head, by the position."""
    if rot is None:
        return x
    half = rot["dims"] // 2
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * rotation_frequencies(rot)[None, :]
    cos, sin = torch.cos(a).to(x.dtype)[:, None, :], torch.sin(a).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:2 * half]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., 2 * half:]], dim=-1)


def chunk_sight(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def window_sight(T, size, keep_first):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & ((i - j < size) | (j < keep_first))


def weigh(scores, sight, extra):
    """scores [H, T, T]: exp of a visible score over the sum of all of them and exp(extra[h])."""
    s = scores.masked_fill(~sight[None], float("-inf"))
    top = torch.maximum(s.max(-1, keepdim=True).values, extra[:, None, None])
    e = torch.exp(s - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(extra[:, None, None] - top))


def mix_values(q, k, v, scale, sight, extra):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H * V]."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    kk, vv = k.repeat_interleave(per, 1), v.repeat_interleave(per, 1)
    s = torch.einsum("ihd,jhd->hij", q, kk) * scale
    return torch.einsum("hij,jhv->ihv", weigh(s, sight, extra), vv).reshape(T, -1)


def chunk_attention(h, w, pre, m, eps):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (h @ w[pre + "q"].T + w[pre + "q.b"]).view(T, H, D)
    k = (h @ w[pre + "k"].T + w[pre + "k.b"]).view(T, G, D)
    v = (h @ w[pre + "v"].T + w[pre + "v.b"]).view(T, G, V)
    q, k = rms(q, eps) * w[pre + "q.norm"], rms(k, eps) * w[pre + "k.norm"]
    q, k = rotate(q, m.get("rot")), rotate(k, m.get("rot"))
    sight = chunk_sight(T, m["mask"]["size"] if m.get("mask") else T)
    return mix_values(q, k, v, m["scale"], sight, torch.zeros(H, dtype=h.dtype)) @ w[pre + "o"].T


def kept_window_attention(h, w, pre, m, eps):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = (rms(h @ w[pre + "q"].T, eps) * w[pre + "q.norm"]).view(T, H, D)
    k = (rms(h @ w[pre + "k"].T, eps) * w[pre + "k.norm"]).view(T, G, D)
    v = (h @ w[pre + "v"].T).view(T, G, V)
    q, k = rotate(q, m.get("rot")), rotate(k, m.get("rot"))
    mask = m.get("mask") or {"size": T}
    sight = window_sight(T, mask["size"], mask.get("keep_first", 0))
    return mix_values(q, k, v, m["scale"], sight, w[pre + "sink"]) @ w[pre + "o"].T


def lightning(h, w, pre, m, eps):
    T, H, D, V = h.shape[0], m["heads"], m["dim"], m["vdim"]
    q, k = silu(h @ w[pre + "q"].T).view(T, H, D), silu(h @ w[pre + "k"].T).view(T, H, D)
    v = silu(h @ w[pre + "v"].T).view(T, H, V)
    decay = torch.tensor(m["decay"], dtype=h.dtype)
    S = torch.zeros(H, D, V, dtype=h.dtype)
    out = []
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]).reshape(H * V))
    o = rms(torch.stack(out), eps) * w[pre + "norm"]
    return (o * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T


def side_by_side(h, w, pre, m, eps):
    return (m["left_scale"] * kept_window_attention(h, w, pre + "left.", m["left"], eps)
            + m["right_scale"] * lightning(h, w, pre + "right.", m["right"], eps))


def dense(h, w, pre):
    return (torch.relu(h @ w[pre + "gate"].T) * (h @ w[pre + "up"].T)) @ w[pre + "down"].T


def clipped_expert(h, w, pre, limit):
    g = torch.clamp(h @ w[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ w[pre + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def route(h, w, pre, top):
    """(chosen experts [T, top], their weights, the margin by which the last chosen one was chosen)."""
    z = h @ w[pre + "router"].T + w[pre + "router.b"]
    order = torch.sort(z, dim=-1, descending=True, stable=True)
    chosen = order.indices[:, :top]
    margin = order.values[:, top - 1] - order.values[:, top] if top < z.shape[1] else torch.full((h.shape[0],), float("inf"))
    return chosen, torch.softmax(order.values[:, :top], dim=-1), margin


def experts(h, w, pre, mlp, margins=None):
    chosen, weights, margin = route(h, w, pre, mlp["router"]["top"])
    if margins is not None:
        margins.append(margin)
    out = torch.zeros_like(h)
    for e in range(mlp["router"]["experts"]):
        at, place = (chosen == e).nonzero(as_tuple=True)
        if len(at):
            out[at] += weights[at, place][:, None] * clipped_expert(h[at], w, f"{pre}e{e}.", mlp["expert"]["limit"])
    if mlp.get("shared"):
        out = out + clipped_expert(h, w, pre + "shared.", mlp["shared"]["limit"])
    return out


MIXERS = {"attention": chunk_attention, "parallel": side_by_side}


def layer(x, w, i, cfg, margins=None):
    entry, eps, alpha = cfg["layers"][i], cfg["norm"]["eps"], cfg["postln_alpha"]
    pre = f"l{i}."
    h = token_shift(x, w[pre + "shift"])
    x = scalar_norm(alpha * x + MIXERS[entry["type"]](h, w, pre + "mix.", entry["mixer"], eps), w[pre + "norm1"], eps)
    mlp = entry.get("mlp")
    if mlp is None:
        return x
    y = dense(x, w, pre + "mlp.") if mlp["kind"] == "dense" else experts(x, w, pre + "mlp.", mlp, margins)
    return scalar_norm(alpha * x + y, w[pre + "norm2"], eps)


def forward(tokens, w, cfg, dtype=torch.float64, streams=None, margins=None):
    """Logits [T, vocab] of one sequence; `streams` (a list) gets the residual stream after every layer,
    `margins` every router's margins."""
    w = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in w.items()}
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * cfg["embedding"]["scale"]
    for i in range(len(cfg["layers"])):
        x = layer(x, w, i, cfg, margins)
        if streams is not None:
            streams.append(x)
    logits = scalar_norm(x, w["final.norm"], cfg["norm"]["eps"]) @ w["head"].T
    cap = cfg.get("logit_softcap")
    return cap * torch.tanh(logits / cap) if cap else logits


def greedy(tokens, w, cfg, count):
    tokens = list(tokens)
    out = []
    for _ in range(count):
        nxt = int(forward(tokens, w, cfg)[-1].argmax())
        out.append(nxt)
        tokens.append(nxt)
    return out
