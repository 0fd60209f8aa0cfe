"""A plain, slow Miberax decoder in float64 torch on the CPU, one function per mechanism, written from
the design's equations.  It shares no code with hfee_amd: the tests compare the engine with it.

Notation.  x: the residual stream [T, width] of one sequence whose first token sits at position 0.
`w`: a dict from tensor names to tensors (linear weights [out, in], applied as W x).  `m`: the dict of one
mixer of a pair in config.json.  Every function takes the whole sequence at once; the recurrence walks over
it token by token, so cutting a sequence can change nothing here.
"""
from __future__ import annotations

import torch


def rms(x, eps):
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def group_norm(x, weight, groups, eps):
    """Each of `groups` equal parts of a row by its own root mean square, the whole times the weight."""
    parts = x.view(*x.shape[:-1], groups, x.shape[-1] // groups)
    return rms(parts, eps).reshape(x.shape) * weight


def silu(z):
    return z * torch.sigmoid(z)


def rotation_frequencies(rot):
    stretch = (rot.get("scaling") or {}).get("factor", 1.0)
    return torch.tensor([rot["base"] ** (-2.0 * i / rot["dims"]) / stretch for i in range(rot["dims"] // 2)], dtype=torch.float64)


def rotate(x, rot):
    """x [T, heads, dim]: pairs (2i, 2i + 1) of the first `dims` dims of each head, by the position."""
    if rot is None:
        return x
    n = rot["dims"]
    a = torch.arange(x.shape[0], dtype=torch.float64)[:, None] * rotation_frequencies(rot)[None, :]
    cos, sin = torch.cos(a).to(x.dtype)[:, None, :], torch.sin(a).to(x.dtype)[:, None, :]
    out = x.clone()
    u, v = x[..., 0:n:2], x[..., 1:n:2]
    out[..., 0:n:2] = u * cos - v * sin
    out[..., 1:n:2] = v * cos + u * sin
    return out


def chunk_sight(T, size):
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size)


def mix_values(q, k, v, scale, sight):
    """q [T, H, D], k [T, G, D], v [T, G, V] -> [T, H * V]: softmax over the visible keys."""
    T, H, _ = q.shape
    per = H // k.shape[1]
    kk, vv = k.repeat_interleave(per, 1), v.repeat_interleave(per, 1)
    s = torch.einsum("ihd,jhd->hij", q, kk) * scale
    a = torch.softmax(s.masked_fill(~sight[None], float("-inf")), dim=-1)
    return torch.einsum("hij,jhv->ihv", a, vv).reshape(T, -1)


def chunk_attention(h, w, pre, m):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate((h @ w[pre + "q"].T).view(T, H, D), m.get("rot"))
    k = rotate((h @ w[pre + "k"].T).view(T, G, D), m.get("rot"))
    v = (h @ w[pre + "v"].T).view(T, G, V)
    sight = chunk_sight(T, m["mask"]["size"] if m.get("mask") else T)
    return mix_values(q, k, v, m["scale"], sight) @ w[pre + "o"].T


def short_conv(x, taps):
    """x [T, C], taps [C, K]: sum_j taps[:, K - 1 - j] x_(t - j), zeros before the sequence."""
    K = taps.shape[1]
    padded = torch.cat([torch.zeros(K - 1, x.shape[1], dtype=x.dtype), x], dim=0)
    return sum(padded[i:i + x.shape[0]] * taps[:, i] for i in range(K))


def unit(x, eps=1e-6):
    return x / torch.sqrt((x * x).sum(-1, keepdim=True) + eps)


def delta_rule(q, k, v, beta, g, S=None):
    """q, k [T, H, D], v [T, H, V], beta, g [T, H]; returns the reads [T, H, V] and the last state."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[2], dtype=q.dtype) if S is None else S.clone()
    out = []
    for t in range(T):
        S = g[t][:, None, None] * S
        u = beta[t][:, None] * (v[t] - torch.einsum("hdv,hd->hv", S, k[t]))
        S = S + k[t][:, :, None] * u[:, None, :]
        out.append(torch.einsum("hdv,hd->hv", S, q[t]))
    return torch.stack(out), S


def gated_delta(h, w, pre, m, eps):
    T, H, G, D, V = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    through = lambda r: silu(short_conv(h @ w[pre + r].T, w[pre + r + ".conv"]))      # noqa: E731
    q = unit(through("q").view(T, G, D)) * D ** -0.5
    k = unit(through("k").view(T, G, D))
    v = through("v").view(T, H, V)
    beta = torch.sigmoid(h @ w[pre + "b"].T)
    g = torch.exp(-torch.exp(w[pre + "A_log"]) * torch.nn.functional.softplus(h @ w[pre + "a"].T + w[pre + "dt_bias"], threshold=60.0))
    o, _ = delta_rule(q.repeat_interleave(H // G, 1), k.repeat_interleave(H // G, 1), v, beta, g)
    o = rms(o, eps) * w[pre + "norm"] * silu(h @ w[pre + "g"].T).view(T, H, V)
    return o.reshape(T, H * V) @ w[pre + "o"].T


def pair(h, w, pre, m, eps):
    left = rms(chunk_attention(h, w, pre + "left.", m["left"]), eps) * w[pre + "left.out"]
    right = rms(gated_delta(h, w, pre + "right.", m["right"], eps), eps) * w[pre + "right.out"]
    return 0.5 * (left + right)


def poly_norm(z, numbers, eps):
    a, b, c, e = numbers
    return a * rms(z, eps) + b * rms(z * z, eps) + c * rms(z * z * z, eps) + e


def dense(h, w, pre, eps):
    return poly_norm(h @ w[pre + "up"].T, w[pre + "act"], eps) @ w[pre + "down"].T


def clipped_expert(h, w, pre, limit):
    g = torch.clamp(h @ w[pre + "gate"].T, max=limit)
    u = torch.clamp(h @ w[pre + "up"].T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ w[pre + "down"].T


def choose(scores, choice, r):
    """(chosen [T, top], weights [T, top], margin [T]): the margin is the least difference of two choice scores by
    which the choice (of groups or of experts) would have been another."""
    T, N = choice.shape
    margin = torch.full((T,), float("inf"), dtype=choice.dtype)
    groups = r.get("groups")
    if groups and groups["keep"] < groups["count"]:
        best = choice.view(T, groups["count"], -1).max(-1).values
        order = torch.sort(best, dim=-1, descending=True, stable=True)
        margin = order.values[:, groups["keep"] - 1] - order.values[:, groups["keep"]]
        kept = torch.zeros(T, groups["count"], dtype=torch.bool)
        kept.scatter_(1, order.indices[:, :groups["keep"]], True)
        choice = choice.masked_fill(~kept.repeat_interleave(N // groups["count"], dim=1), float("-inf"))
    order = torch.sort(choice, dim=-1, descending=True, stable=True)
    chosen = order.indices[:, :r["top"]]
    if r["top"] < N:
        margin = torch.minimum(margin, order.values[:, r["top"] - 1] - order.values[:, r["top"]])
    s = scores.gather(1, chosen)
    return chosen, s / (s.sum(-1, keepdim=True) + 1e-20) * r["scale"], margin


def experts(h, w, pre, mlp, margins=None):
    r = mlp["router"]
    scores = torch.softmax(h @ w[pre + "router"].T, dim=-1)
    chosen, weights, margin = choose(scores, scores + w[pre + "correction"], r)
    if margins is not None:
        margins.append(margin)
    out = torch.zeros_like(h)
    for e in range(r["experts"] + r.get("identity", 0)):
        at, place = (chosen == e).nonzero(as_tuple=True)
        if len(at):
            y = clipped_expert(h[at], w, f"{pre}e{e}.", mlp["expert"]["limit"]) if e < r["experts"] else h[at]
            out[at] += weights[at, place][:, None] * y
    if mlp.get("shared"):
        out = out + torch.sigmoid(h @ w[pre + "shared.sg"].T) * clipped_expert(h, w, pre + "shared.", mlp["shared"]["limit"])
    return out


def layer(x, w, i, cfg, margins=None):
    entry, eps, groups = cfg["layers"][i], cfg["norm"]["eps"], cfg["norm"]["groups"]
    pre = f"l{i}."
    x = x + pair(group_norm(x, w[pre + "norm1"], groups, eps), w, pre + "mix.", entry["mixer"], eps)
    mlp = entry.get("mlp")
    if mlp is None:
        return x
    h = group_norm(x, w[pre + "norm2"], groups, eps)
    return x + (dense(h, w, pre + "mlp.", eps) if mlp["kind"] == "dense" else experts(h, w, pre + "mlp.", mlp, margins))


def forward(tokens, w, cfg, dtype=torch.float64, streams=None, margins=None):
    """Logits [T, vocab] of one sequence; `streams` (a list) gets the residual stream after every layer,
    `margins` every router's margins."""
    w = {n: (t.to(dtype) if t.is_floating_point() else t) for n, t in w.items()}
    x = w["embed"][torch.as_tensor(tokens, dtype=torch.long)]
    for i in range(len(cfg["layers"])):
        x = layer(x, w, i, cfg, margins)
        if streams is not None:
            streams.append(x)
    return group_norm(x, w["final.norm"], cfg["norm"]["groups"], cfg["norm"]["eps"]) @ w["embed"].T


def greedy(tokens, w, cfg, count):
    tokens = list(tokens)
    out = []
    for _ in range(count):
        nxt = int(forward(tokens, w, cfg)[-1].argmax())
        out.append(nxt)
        tokens.append(nxt)
    return out
