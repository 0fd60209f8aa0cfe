"""The Medulorn decoder on the GPU against the plain implementation: the new kernels alone (attention over chunks and
behind a window that keeps the first tokens, with sinks, with keys that stand out just inside and just outside every
edge, among the first tokens, far back and at page borders, in prompts and token by token; biases, norms and rotation
on the way into the cache; the norm behind the sum with what the next sub-layer reads; the token shift; the recurrence
in portions over slots; the router; the clipped gate in the products and in the experts; the cap on the logits), each
mechanism as a model of one layer, the whole model under four ways of cutting the same requests into steps (whole,
bulk then single tokens, portions down to two tokens, mixed batches on a small page pool with four state slots, pages
and slots used again), in 32-bit and in bfloat16, on configurations with even and with odd sizes; long decoding
through graph replays; greedy generation through the entry point and its scheduler; the trace runner and the command
line as subprocesses."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import medulorn_util as mu
import plain_medulorn as pm
import trace_util as tu
from conftest import ROOT

pytestmark = pytest.mark.gpu

TOL = {"float32": 3e-5, "bfloat16": 8e-2}
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
LENGTHS = {"A": [5, 17, 64, 1, 100, 38, 129, 49, 2], "B": [40, 3, 100, 65, 2, 31], "C": [420, 47, 311, 1, 161]}


def i32(a):
    return torch.as_tensor(np.asarray(a, dtype=np.int32)).cuda()


def _paged(lengths, page_size=16, seed=0):
    """Block tables for sequences of these lengths over shuffled pages (page 0 is never handed out, so that a
    table's unused entries, which hold 0, would show if they were read)."""
    rng = np.random.default_rng(seed)
    need = [-(-n // page_size) for n in lengths]
    pages = rng.permutation(np.arange(1, sum(need) + 1))
    tables, at = np.zeros((len(lengths), max(need)), dtype=np.int32), 0
    for s, k in enumerate(need):
        tables[s, :k] = pages[at:at + k]
        at += k
    return tables, sum(need) + 1


# ------------------------------------------------------------------ kernels alone

def sight_of(n, window, chunk, keep):
    i, j = torch.arange(n)[:, None], torch.arange(n)[None, :]
    near = torch.ones(n, n, dtype=torch.bool)
    if window:
        near &= i - j < window
    if chunk:
        near &= i // chunk == j // chunk
    return (j <= i) & (near | (j < keep))


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,dk,dv,window,chunk,keep,sink", [
    (4, 2, 32, 16, 19, 0, 3, "learned"), (3, 3, 10, 12, 7, 0, 1, "zero"), (8, 2, 48, 32, 70, 0, 40, "learned"),
    (4, 1, 96, 64, 33, 0, 33, None), (8, 2, 32, 16, 0, 37, 0, "zero"), (6, 2, 80, 64, 0, 64, 0, "zero"),
    (5, 1, 14, 6, 0, 11, 0, "zero"), (4, 4, 32, 32, 0, 150, 0, None), (16, 1, 48, 32, 1, 0, 9, "learned"),
    (8, 2, 32, 16, 0, 1, 0, "zero"), (6, 3, 32, 16, 21, 50, 5, "learned"), (4, 2, 32, 16, 0, 0, 0, "zero"),
    (8, 2, 64, 64, 45, 0, 100, "learned")])
def test_attention_over_chunks_and_kept_windows(dtype, H, G, dk, dv, window, chunk, keep, sink):
    """Two sequences side by side, written in portions whose edges fall inside pages, windows and chunks, read by
    portions and by single tokens (plain, and where the sizes allow on the matrix cores, the single tokens' keys
    whole and split).  Keys are made to stand out for queries at the end: the first key of the window or chunk and
    the one before it, the last kept token and the one behind it, the first token, a key far back, the keys on both
    sides of a page border; every position is compared with the definition, so an edge that is one token off
    shows there."""
    from hfee_amd.kernels import ops
    dt = DT[dtype]
    g = torch.Generator().manual_seed(dk + H + window + chunk)
    lengths, scale = [333, 37], 0.25
    qs = [torch.randn(n, H, dk, generator=g) for n in lengths]
    ks = [torch.randn(n, G, dk, generator=g) for n in lengths]
    vs = [torch.randn(n, G, dv, generator=g) for n in lengths]
    last, kv1 = lengths[0] - 1, min(1, H - 1) // (H // G)
    standouts = [0, 3, 15, 16, 200]
    if window:
        standouts += [last - window + 1, last - window]
    if chunk:
        standouts += [last - last % chunk, last - last % chunk - 1]
    if keep:
        standouts += [keep - 1, keep]
    for back, j in enumerate(standouts):        # each is what some query near the end looks at hardest
        if 0 <= j < lengths[0]:
            ks[0][j, kv1] = qs[0][last - back % 3, min(1, H - 1)] * 3.0
    qs, ks, vs = ([t.to(dt).float() for t in x] for x in (qs, ks, vs))
    sinks = {"zero": torch.zeros(H), "learned": torch.randn(H, generator=g) * 2.0, None: None}[sink]
    extra = torch.full((H,), -1e30, dtype=torch.float64) if sinks is None else sinks.double()
    want = [pm.mix_values(q.double(), k.double(), v.double(), scale, sight_of(n, window, chunk, keep), extra)
            for q, k, v, n in zip(qs, ks, vs, lengths)]
    tables, pages = _paged(lengths)
    cache = torch.zeros(pages, G, 16 * (dk + dv), dtype=dt, device="cuda")
    cache[0].fill_(float("nan"))
    bt = i32(tables)
    matrix = dtype == "bfloat16" and ops.attention_kv_sizes_fit(dk, dv)
    sight = dict(window=window, chunk=chunk, keep_first=keep)
    on_gpu = None if sinks is None else sinks.cuda()
    fed = [0, 0]
    for sizes in ([7, 2], [9, 0], [150, 17], [140, 16], [1, 1], [5, 1], [1, 0], [20, 0]):
        segs = [(s, n) for s, n in enumerate(sizes) if n]
        n_all = sum(n for _, n in segs)
        cat = lambda xs: torch.cat([xs[s][fed[s]:fed[s] + n].reshape(n, -1) for s, n in segs]).to(dt).cuda()      # noqa: E731
        positions = i32(np.concatenate([np.arange(fed[s], fed[s] + n) for s, n in segs]))
        token_segment = i32(np.concatenate([np.full(n, i) for i, (_, n) in enumerate(segs)]))
        tab = bt[[s for s, _ in segs]].contiguous()
        q = torch.zeros(n_all, H * dk, dtype=dt, device="cuda")
        ops.qkv_write(q, cat(qs), cat(ks), cat(vs), positions, token_segment, tab, None, None, cache, H, G, dk, dv, 16,
                      int(positions.max()))
        out = torch.zeros(n_all, H * dv, dtype=dt, device="cuda")
        ops.attention_kv_plain(out, q, cache, positions, token_segment, tab, H, G, dk, dv, 16, scale, on_gpu, **sight)
        outs = [out]
        if matrix:
            rows_most = ops.attention_kv_rows(dk, dv, H // G, "softmax")
            portions, singles, row = [], [], 0
            for i, (s, n) in enumerate(segs):
                if n > 1:
                    portions += [(row + o, min(rows_most, n - o), fed[s] + o, i) for o in range(0, n, rows_most)]
                else:
                    singles.append((row, 1, fed[s], i))
                row += n
            out2 = torch.zeros(n_all, H * dv, dtype=dt, device="cuda")
            if portions:
                ops.attention_kv_bf16(out2, q, cache, i32(portions).reshape(-1, 4), 0, tab, H, G, dk, dv, 16, scale, on_gpu, **sight)
            if singles:
                for splits in (1, 3):
                    partial = torch.zeros(ops.attention_kv_partial_words(len(singles), H, dv, splits) + 1, device="cuda")
                    ops.attention_kv_bf16(out2, q, cache, i32(singles).reshape(-1, 4), 1, tab, H, G, dk, dv, 16, scale, on_gpu,
                                          partial=partial if splits > 1 else None, splits=splits, **sight)
                    if splits == 1:
                        first = out2.clone()
                    else:
                        rows_single = [r for r, _, _, _ in singles]
                        assert mu.rel(out2[rows_single].float().cpu(), first[rows_single].float().cpu()) < 2e-2
            outs.append(out2)
        row = 0
        for s, n in segs:
            for o in outs:
                w = want[s][fed[s]:fed[s] + n]
                err = (o[row:row + n].double().cpu() - w).abs().max() / w.abs().max()
                assert err < (2e-5 if dtype == "float32" else 3e-2), (sizes, s, float(err))
            fed[s] += n
            row += n
    assert fed == lengths and torch.isnan(cache[0].float()).all()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,dk,dv,rot,norm,biased,n,start", [
    (4, 2, 12, 10, 8, "head", True, 21, 5), (3, 1, 32, 16, 32, "row", False, 40, 0), (8, 2, 64, 32, 64, "head", True, 300, 16),
    (8, 8, 16, 16, 16, "row", True, 70, 3), (6, 2, 96, 48, 64, "row", False, 65, 32), (32, 8, 128, 128, 128, "head", True, 48, 64),
    (5, 5, 40, 24, 16, None, True, 33, 0), (2, 1, 8, 8, 0, "head", False, 1, 100), (40, 4, 128, 64, 128, "row", True, 5, 1),
    (16, 4, 80, 80, 80, "head", False, 2, 30)])
def test_biases_norms_and_rotation_on_the_way_into_the_cache(dtype, H, G, dk, dv, rot, norm, biased, n, start):
    from hfee_amd.kernels import ops
    dt = DT[dtype]
    g = torch.Generator().manual_seed(dk + n)
    widths = (H * dk, G * dk, G * dv)
    total = sum(widths)
    proj = torch.randn(n, (total + 7) // 8 * 8, generator=g).to(dt)[:, :total]
    biases = [torch.randn(w, generator=g) for w in widths] if biased else [None] * 3
    sizes = (H * dk, G * dk) if norm == "row" else (dk, dk)
    weights = [1.0 + torch.randn(s, generator=g) for s in sizes] if norm else [None] * 2
    eps = 1e-3
    q, k, v = (x.double() + (0 if b is None else b.double()) for x, b in zip(proj.split(widths, dim=1), biases))
    if norm == "head":
        q = (pm.rms(q.view(n, H, dk), eps) * weights[0].double()).view(n, -1)
        k = (pm.rms(k.view(n, G, dk), eps) * weights[1].double()).view(n, -1)
    elif norm == "row":
        q, k = pm.rms(q, eps) * weights[0].double(), pm.rms(k, eps) * weights[1].double()
    pos = torch.arange(start, start + n)
    cos = sin = None
    q, k = q.view(n, H, dk), k.view(n, G, dk)
    if rot:
        a = torch.arange(start + n, dtype=torch.float64)[:, None] * pm.rotation_frequencies(mu.rotation(rot, 300.0))[None, :]
        cos, sin = torch.cos(a).float().cuda(), torch.sin(a).float().cuda()
        turn = lambda x: pm.rotate(torch.cat([torch.zeros(start, *x.shape[1:], dtype=x.dtype), x]), mu.rotation(rot, 300.0))[start:]      # noqa: E731
        q, k = turn(q), turn(k)
    tables, pages = _paged([start + n])
    cache = torch.zeros(pages, G, 16 * (dk + dv), dtype=dt, device="cuda")
    q_out = torch.zeros(n, H * dk, dtype=dt, device="cuda")
    gp = proj.cuda()
    up = lambda t: None if t is None else t.cuda()      # noqa: E731
    ops.qkv_write(q_out, gp[:, :widths[0]], gp[:, widths[0]:widths[0] + widths[1]], gp[:, widths[0] + widths[1]:], i32(pos),
                  i32(np.zeros(n)), i32(tables), cos, sin, cache, H, G, dk, dv, 16, start + n - 1,
                  biases=tuple(up(b) for b in biases), norm=norm, q_weight=up(weights[0]), k_weight=up(weights[1]), eps=eps)
    tol = 2e-6 if dtype == "float32" else 1e-2
    assert mu.rel(q_out.double().cpu(), q.reshape(n, -1)) < tol
    held = cache.double().cpu()
    keys = torch.stack([held[tables[0, p // 16], :, :16 * dk].view(G, 16, dk)[:, p % 16] for p in pos.tolist()])
    values = torch.stack([held[tables[0, p // 16], :, 16 * dk:].view(G, dv, 16)[:, :, p % 16] for p in pos.tolist()])
    assert mu.rel(keys, k) < tol and mu.rel(values, v.view(n, G, dv)) < tol
    untouched = sum(int(held[p].abs().sum() > 0) for p in range(pages) if p not in tables[0, start // 16:].tolist())
    assert untouched == 0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width", [(8, 4096), (70, 72), (3, 5000), (40, 1024), (1, 58), (5, 20000)])
def test_the_norm_behind_the_sum_and_the_next_input(dtype, n, width):
    """With and without second rows; the new rows alone, in the engine's dtype, and shifted by the slots' rows."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + width)
    x, y, y2 = (torch.randn(n, width, generator=g) for _ in range(3))
    w, shift, before = torch.rand(width, generator=g) + 0.5, torch.rand(width, generator=g), torch.randn(n + 2, width, generator=g)
    slots = torch.randperm(n + 2, generator=g)[:n]
    tol = 2e-6 if dtype == "float32" else 1e-2
    for second in (None, y2):
        want = pm.rms(1.7 * x.double() + 0.6 * y.double() + (0 if second is None else 0.9 * y2.double()), 1e-5) * w.double()
        more = {} if second is None else dict(y2=y2.cuda(), scale2=0.9)
        got = x.clone().cuda()
        ops.post_norm(got, y.cuda(), 1.7, w.cuda(), 1e-5, scale=0.6, **more)
        assert mu.rel(got.double().cpu(), want) < 2e-6
        got, nxt = x.clone().cuda(), torch.zeros(n, width, dtype=DT[dtype], device="cuda")
        ops.post_norm(got, y.cuda(), 1.7, w.cuda(), 1e-5, scale=0.6, next_out=nxt, **more)
        assert mu.rel(got.double().cpu(), want) < 2e-6 and mu.rel(nxt.double().cpu(), want) < tol
        got, state = x.clone().cuda(), before.clone().cuda()
        ops.post_norm(got, y.cuda(), 1.7, w.cuda(), 1e-5, scale=0.6, next_out=nxt, shift=shift.cuda(), state=state,
                      segment_slots=i32(slots), **more)
        assert mu.rel(got.double().cpu(), want) < 2e-6
        assert mu.rel(nxt.double().cpu(), want + (before[slots].double() - want) * shift.double()) < tol
        assert torch.equal(state[slots.cuda()], got)
        rest = [s for s in range(n + 2) if s not in slots.tolist()]
        assert torch.equal(state[rest].cpu(), before[rest])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("width", [64, 58, 4100])
def test_the_token_shift_across_portions(dtype, width):
    """Two requests in other slots, in portions down to one token: the row before a portion comes from the slot; a
    slot of NaNs beside them stays untouched."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    lengths, slots = [30, 11], [2, 0]
    xs, shift = [torch.randn(n, width, generator=g) for n in lengths], torch.rand(width, generator=g)
    want = [pm.token_shift(x.double(), shift.double()) for x in xs]
    state = torch.zeros(4, width, device="cuda")
    state[1].fill_(float("nan"))
    fed = [0, 0]
    for sizes in ([5, 2], [1, 1], [0, 3], [2, 0], [22, 5]):
        segs = [(s, n) for s, n in enumerate(sizes) if n]
        x = torch.cat([xs[s][fed[s]:fed[s] + n] for s, n in segs]).cuda()
        rows = np.cumsum([0] + [n for _, n in segs])[:-1]
        out = torch.zeros(x.shape, dtype=DT[dtype], device="cuda")
        ops.token_shift(out, x, state, shift.cuda(), i32(np.concatenate([np.full(n, i) for i, (_, n) in enumerate(segs)])), i32(rows),
                        i32([n for _, n in segs]), i32([slots[s] for s, _ in segs]))
        row = 0
        for s, n in segs:
            assert mu.rel(out[row:row + n].double().cpu(), want[s][fed[s]:fed[s] + n]) < (2e-6 if dtype == "float32" else 1e-2)
            fed[s] += n
            row += n
            assert torch.equal(state[slots[s]].cpu(), xs[s][fed[s] - 1])
    assert fed == lengths and torch.isnan(state[1]).all()


@pytest.mark.parametrize("chunks", [False, True])
@pytest.mark.parametrize("H,D,V", [(2, 16, 32), (3, 12, 20), (4, 64, 64), (1, 4, 4), (2, 128, 256), (3, 100, 17), (2, 256, 48)])
def test_the_recurrence_in_portions(H, D, V, chunks):
    """Two requests in other slots, in portions of unequal size, token by token and with the long portions in
    chunks, against the closed form o_t = sum_j decay^(t - j) (q_t . k_j) v_j; a slot of NaNs beside them stays
    untouched."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(H + D)
    lengths, slots = [290, 90], [2, 0]
    decay = torch.tensor([1.0, 0.9, 0.0, 0.99][:H])
    qs, ks = ([torch.randn(n, H, D, generator=g) * D ** -0.25 for n in lengths] for _ in range(2))
    vs = [torch.randn(n, H, V, generator=g) for n in lengths]
    want = []
    for q, k, v in zip(qs, ks, vs):
        t = torch.arange(q.shape[0])
        power = (t[:, None] - t[None, :]).clamp(min=0).double()
        w = torch.einsum("ihd,jhd->hij", q.double(), k.double()) * decay.double()[:, None, None] ** power[None]
        want.append(torch.einsum("hij,jhv->ihv", w * (t[None, :] <= t[:, None]), v.double()).reshape(q.shape[0], -1))
    state = torch.zeros(4, H, *ops.scan_state_shape(D, V), device="cuda")
    state[1].fill_(float("nan"))
    fed = [0, 0]
    for sizes in ([5, 2], [1, 1], [40, 0], [2, 17], [150, 3], [64, 65], [28, 2]):
        segs = [(s, n) for s, n in enumerate(sizes) if n]
        cat = lambda xs: torch.cat([xs[s][fed[s]:fed[s] + n].reshape(n, -1) for s, n in segs]).cuda()      # noqa: E731
        q, k, v = cat(qs), cat(ks), cat(vs)
        rows = np.cumsum([0] + [n for _, n in segs])[:-1]
        out = torch.zeros(q.shape[0], H * V, device="cuda")
        more = {}
        words = ops.linear_chunks_scratch(max(n for _, n in segs), q.shape[0], H, D)
        if chunks and words:
            more = dict(scratch=torch.full((words,), float("nan"), device="cuda"), longest=max(n for _, n in segs),
                        shortest=min(n for _, n in segs))
        ops.linear_scan(out, state, q, k, v, decay.cuda(), None, i32(rows), i32([n for _, n in segs]), i32([slots[s] for s, _ in segs]),
                        H, H, D, V, "decay_add", decay_per_head=True, **more)
        row = 0
        for s, n in segs:
            assert mu.rel(out[row:row + n].double().cpu(), want[s][fed[s]:fed[s] + n]) < 2e-5, (sizes, s)
            fed[s] += n
            row += n
    assert fed == lengths and torch.isnan(state[1]).all() and torch.isfinite(state[[0, 2, 3]]).all()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width", [(5, 96), (70, 4096), (3, 1500)])
def test_all_heads_normed_as_one_and_gated(dtype, n, width):
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(width)
    o, z, w = torch.randn(n, width, generator=g), torch.randn(n, width, generator=g).to(DT[dtype]), torch.rand(width, generator=g) + 0.5
    out = torch.zeros(n, width, dtype=DT[dtype], device="cuda")
    ops.head_norm_gate(out, o.cuda(), z.cuda(), w.cuda(), 1, width, 1e-4, "sigmoid")
    want = pm.rms(o.double(), 1e-4) * w.double() * torch.sigmoid(z.double())
    assert mu.rel(out.double().cpu(), want) < (2e-6 if dtype == "float32" else 1e-2)
    silu = torch.zeros(n, width, device="cuda")
    ops.scan_gate(silu, z.cuda(), "silu")
    assert mu.rel(silu.double().cpu(), torch.nn.functional.silu(z.double())) < 2e-6


@pytest.mark.parametrize("n,E,top", [(50, 5, 2), (7, 70, 3), (33, 4, 4), (9, 130, 1), (20, 16, 3)])
def test_the_router_weighs_the_chosen(n, E, top):
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + E)
    logits, bias = torch.randn(n, E, generator=g), torch.randn(E, generator=g)
    for b in (bias, None):
        chosen = torch.zeros(n, top, dtype=torch.int32, device="cuda")
        weights = torch.zeros(n, top, device="cuda")
        ops.router_topk(chosen, weights, logits.cuda(), top, score="softmax_chosen", bias=None if b is None else b.cuda())
        z = logits.double() + (0 if b is None else b.double())
        order = torch.sort((logits + (0 if b is None else b)), dim=-1, descending=True, stable=True).indices[:, :top]
        assert torch.equal(chosen.cpu().long(), order)
        assert mu.rel(weights.double().cpu(), torch.softmax(torch.gather(z, 1, order), -1)) < 1e-6


def clipped(g, u, limit, sharpness=1.702):
    g, u = torch.clamp(g, max=limit), torch.clamp(u, min=-limit, max=limit)
    return g * torch.sigmoid(sharpness * g) * (u + 1.0)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,E,top,ff,width", [(6, 5, 2, 20, 28), (90, 4, 2, 64, 96), (50, 8, 3, 32, 64), (3, 4, 4, 32, 32)])
def test_clipped_experts(dtype, n, E, top, ff, width):
    """Token by token, and where the sizes allow grouped on the matrix cores."""
    from hfee_amd.kernels import ops
    dt, limit = DT[dtype], 0.7
    g = torch.Generator().manual_seed(ff + n)
    h = torch.randn(n, width, generator=g).to(dt)
    wg, wu = (torch.randn(E, ff, width, generator=g).mul(width ** -0.5).to(dt) for _ in range(2))
    wd = torch.randn(E, width, ff, generator=g).mul(ff ** -0.5).to(dt)
    chosen = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(n)])
    weights = torch.softmax(torch.randn(n, top, generator=g), -1)
    x = torch.randn(n, width, generator=g)
    want = x.double().clone()
    for t in range(n):
        for j in range(top):
            e = int(chosen[t, j])
            a = clipped(wg[e].double() @ h[t].double(), wu[e].double() @ h[t].double(), limit)
            want[t] += weights[t, j].double() * (wd[e].double() @ a)
    numbers = (limit, 1.702)
    act = torch.zeros(n * top, ff, dtype=dt, device="cuda")
    got = x.clone().cuda()
    ops.moe_up(act, h.cuda(), wg.cuda(), wu.cuda(), top, chosen=i32(chosen), activation="clipped", numbers=numbers)
    ops.moe_down(got, act, wd.cuda(), top, pair_weights=weights.cuda(), chosen=i32(chosen))
    tol = 2e-5 if dtype == "float32" else 2e-2
    assert mu.rel(got.double().cpu(), want) < tol
    if ops.moe_grouped_fits(dt, width, ff):
        got = x.clone().cuda()
        order = torch.zeros(n * top, dtype=torch.int32, device="cuda")
        tiles = torch.zeros(3 * ops.moe_group_tiles(n, top, E) + 1, dtype=torch.int32, device="cuda")
        y = torch.zeros(n * top, width, device="cuda")
        ops.moe_grouped(got, h.cuda(), wg.cuda(), wu.cuda(), wd.cuda(), top, order, tiles, act, y, pair_weights=weights.cuda(),
                        chosen=i32(chosen), activation="clipped", numbers=numbers)
        assert mu.rel(got.double().cpu(), want) < tol


@pytest.mark.parametrize("M,ff,K", [(70, 48, 64), (300, 512, 256), (9, 40, 72), (2048, 1024, 512), (100, 36, 128)])
def test_the_clipped_gate_behind_a_product(M, ff, K):
    """As the epilogue of the tiled products (bfloat16) and as a launch of its own (both dtypes)."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(M + ff)
    x = torch.randn(M, K, generator=g).to(torch.bfloat16)
    w = torch.randn(2 * ff, K, generator=g).mul(K ** -0.5).to(torch.bfloat16)
    both = x.double() @ w.double().T
    want = clipped(both[:, 0::2], both[:, 1::2], 0.8)
    out = torch.zeros(M, ff, dtype=torch.bfloat16, device="cuda")
    ops.linear(out, x.cuda(), w.cuda(), gate=True, activation="clipped", numbers=(0.8, 1.702))
    assert mu.rel(out.double().cpu(), want) < 1e-2
    for dt in (torch.float32, torch.bfloat16):
        z = both.to(dt)
        out = torch.zeros(M, ff, dtype=dt, device="cuda")
        ops.swiglu(out, z.cuda()[:, 0::2], z.cuda()[:, 1::2], activation="clipped", numbers=(0.8, 1.702))
        assert mu.rel(out.double().cpu(), clipped(z[:, 0::2].double(), z[:, 1::2].double(), 0.8)) < (2e-6 if dt == torch.float32 else 1e-2)


def test_the_cap_on_the_logits():
    from hfee_amd.kernels import ops
    x = torch.linspace(-90.0, 90.0, 1001).view(7, 143)
    got = x.clone().cuda()
    ops.softcap(got, 12.5)
    assert mu.rel(got.double().cpu(), 12.5 * torch.tanh(x.double() / 12.5)) < 1e-6


# ------------------------------------------------------------------ the whole model

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("medulorn")
    return {(name, dtype): mu.make_folder(base / f"{name.replace(' ', '_')}_{dtype}", cj, seed=7 + ord(name[0]), dtype=dtype)
            for name, cj in list(mu.CONFIGS.items()) + list(mu.SINGLE.items()) for dtype in ("float32", "bfloat16")}


def plain_logits(folder, tokens, margins=None):
    """The plain implementation's logits; margins: a list that receives, a position, the smallest margin by
    which any of its routers chose."""
    cj, w = mu.load_plain(folder)
    each = []
    logits = pm.forward(tokens, w, cj, margins=each).numpy()
    if margins is not None:
        margins.extend(torch.stack(each).min(0).values.tolist() if each else [float("inf")] * len(tokens))
    return logits


# In bfloat16 a router reads rounded numbers: a token whose last chosen expert and the best one not chosen score
# almost alike may go to the other one, and the states and the cache carry the difference to every token behind
# it.  So in bfloat16 a request is compared up to the first position at which a router of the plain
# implementation chose by less than NEAR_TIE, and the configurations in which every token uses every expert
# ("... every expert": nothing is chosen) are compared at every position.
NEAR_TIE = 0.05


class Rows(dict):
    """(request, position) -> logits of the plain implementation; `.margins`: -> the routers' smallest margin."""
    margins: dict


@pytest.fixture(scope="module")
def plain_rows(folders):
    cache = {}

    def get(name, dtype, lengths=None):
        key = (name, dtype, tuple(lengths or LENGTHS[name[0]]))
        if key not in cache:
            cj = (mu.CONFIGS.get(name) or mu.SINGLE[name])
            reqs = tu.make_requests(cj["vocab"], list(key[2]), seed=ord(name[0]))
            rows = Rows()
            rows.margins = {}
            for rid, toks in reqs.items():
                margins = []
                logits = plain_logits(folders[(name, dtype)], toks, margins)
                rows.update({(rid, i): logits[i] for i in range(len(toks))})
                rows.margins.update({(rid, i): margins[i] for i in range(len(toks))})
            cache[key] = (reqs, rows)
        return cache[key]
    return get


def compare(got, want, dtype, what, margins=None):
    """32-bit: every position within the tolerance.  bfloat16: every position before its request's first near
    tie (see NEAR_TIE) within twice the tolerance and all but one in a hundred of them (or one) within it; over all
    positions the median is well within it."""
    assert set(got) == set(want), f"{what}: positions differ"
    tol = TOL[dtype]
    margins = margins if margins is not None else getattr(want, "margins", {})
    errors = {key: mu.rel(got[key], want[key]) for key in want}
    keys = sorted(want)
    if dtype != "float32":
        first_tie = {}
        for rid, at in keys:
            if margins.get((rid, at), float("inf")) < NEAR_TIE:
                first_tie[rid] = min(at, first_tie.get(rid, at))
        keys = [(rid, at) for rid, at in keys if at < first_tie.get(rid, at + 1)]
    over = sorted((errors[key], key) for key in keys if not errors[key] < tol)
    allowed = 0 if dtype == "float32" else max(1, len(keys) // 100)
    assert len(over) <= allowed and not any(e >= 2 * tol for e, _ in over), \
        f"{what}: {len(over)} of {len(keys)} positions beyond {tol}, the worst {over[-1]}, the first {min(k for _, k in over)}"
    assert np.median(list(errors.values())) < tol / 2, f"{what}: median relative error {np.median(list(errors.values())):.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(mu.SINGLE))
def test_each_mechanism_as_a_model_of_one_layer(folders, plain_rows, name, dtype):
    from hfee_amd.trace_replay import Replayer
    reqs, want = plain_rows(name, dtype, [37, 2, 11])
    for what, steps in (("whole", tu.whole(reqs)), ("bulk then single tokens", tu.bulk_then_tail(reqs, 9)),
                        ("portions", tu.portions(reqs, sizes=(2, 5, 3, 2, 7)))):
        rep = Replayer(folders[(name, dtype)], dtype, 64, max_requests=2)
        compare(tu.run(rep, steps), want, dtype, f"{name} {dtype} {what}")


@pytest.mark.parametrize("name,dtype", [(n, d) for n in ("A", "B", "C") for d in ("float32", "bfloat16")]
                         + [("A every expert", "bfloat16"), ("C every expert", "bfloat16")])
def test_every_way_of_cutting_gives_the_plain_logits(folders, plain_rows, name, dtype):
    from hfee_amd.trace_replay import Replayer
    reqs, want = plain_rows(name, dtype)
    longest = max(len(t) for t in reqs.values())
    one = (longest + 63) // 64 * 64
    for what, steps, room in (("whole", tu.whole(reqs), one), ("bulk then single tokens", tu.bulk_then_tail(reqs, 40), one),
                              ("portions", tu.portions(reqs), one), ("mixed", *tu.mixed(reqs, seed=len(name[0])))):
        rep = Replayer(folders[(name, dtype)], dtype, room, max_requests=4)
        got = tu.run(rep, steps)
        compare(got, want, dtype, f"{name} {dtype} {what}")
        rep.engine.cache.check()
        assert not rep.engine.cache.requests


def test_cuts_agree_closely_in_32_bit(folders, plain_rows):
    """Whole prompts against portions and single tokens: rounding apart, the same logits."""
    from hfee_amd.trace_replay import Replayer
    reqs, _ = plain_rows("A", "float32")
    runs = []
    for steps in (tu.whole(reqs), tu.portions(reqs, sizes=(2, 3, 16, 1, 15, 17, 2)), tu.bulk_then_tail(reqs, 20)):
        runs.append(tu.run(Replayer(folders[("A", "float32")], "float32", 192, max_requests=4), steps))
    for other in runs[1:]:
        for key in runs[0]:
            assert mu.rel(other[key], runs[0][key]) < 1e-5


@pytest.mark.parametrize("name", ["A", "B"])
def test_a_slot_that_is_used_again_starts_from_nothing(folders, plain_rows, name):
    """One state slot and a pool of one request's pages: every request inherits the slot and the pages of the
    one before, whose states, last rows and first tokens must be gone."""
    from hfee_amd.trace_replay import Replayer
    reqs, want = plain_rows(name, "float32")
    longest = max(len(t) for t in reqs.values())
    rep = Replayer(folders[(name, "float32")], "float32", (longest + 63) // 64 * 64, max_requests=1)
    got = tu.run(rep, tu.portions(reqs, sizes=(9, 2, 30)))
    compare(got, want, "float32", f"{name}: one slot for all")


def test_chunks_and_windows_give_back_the_pages_they_have_passed(folders, plain_rows):
    """A chunk's and a window's cache are window groups of the manager: a request of 150 tokens holds the pages of
    its reach, and of the first tokens that are kept, and no more, whether it came in portions or token by token, and
    its logits are the plain ones."""
    from hfee_amd.trace_replay import Replayer
    for name, reach, keep in (("chunk", 6, 0), ("window", 6, 2)):
        reqs, want = plain_rows(name, "float32", [150])
        toks = reqs["r0"]
        rep = Replayer(folders[(name, "float32")], "float32", 192, max_requests=2)
        groups = rep.engine.cache.groups
        assert [(g.kind, g.window, g.keep_first) for g in groups] == [("window", reach, keep)]
        got, fed = {}, 0
        for n in [40, 3, 2, 50] + [1] * 55:
            rows = rep.step([("r0", toks[fed:fed + n], list(range(n)))])
            got.update({("r0", fed + i): rows[i] for i in range(n)})
            fed += n
            table = rep.engine.cache.get("r0").tables[0]
            held = [b for b, p in enumerate(table) if p >= 0]
            assert len(held) <= (3 if keep else 2) and (0 in held) == bool(keep or fed < 22), (fed, held)
            rep.engine.cache.check()
        compare(got, want, "float32", f"{name}: a window group")
        rep.engine.release("r0")
        assert not rep.engine.cache.requests


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(folders, dtype):
    """300 single tokens after a short prompt: decode steps replayed from captured graphs, across page borders and
    chunks' edges, while the windows move on, the states and the last rows carried through every replay; a
    second request joins on the way, so that steps of two rows are replayed as well."""
    from hfee_amd.trace_replay import Replayer
    rng = np.random.default_rng(9)
    toks, other = rng.integers(0, 500, size=330).tolist(), rng.integers(0, 500, size=90).tolist()
    name = "C" if dtype == "float32" else "C every expert"      # (in bfloat16 no near tie of a router on the way)
    rep = Replayer(folders[(name, dtype)], dtype, 512, max_requests=4)
    steps = [{"entries": [("a", toks[:30], [29])], "end": []}]
    steps += [{"entries": [("a", toks[i:i + 1], [0])], "end": ["a"] if i == 329 else []} for i in range(30, 330)]
    steps[50]["entries"].append(("b", other[:10], [9]))
    for i in range(10, 90):
        steps[51 + i]["entries"].insert(0, ("b", other[i:i + 1], [0]))
        if i == 89:
            steps[51 + i]["end"].append("b")
    got = tu.run(rep, steps)
    assert rep.engine.graph_replays > 250
    want, margins = {}, {}
    for rid, t, first in (("a", toks, 29), ("b", other, 9)):
        m = []
        rows = plain_logits(folders[(name, dtype)], t, m)
        want.update({(rid, i): rows[i] for i in range(first, len(t))})
        margins.update({(rid, i): v for i, v in enumerate(m)})
    compare(got, want, dtype, f"long decoding {dtype}", margins)


@pytest.mark.parametrize("name", ["window", "lightning"])
def test_the_first_token_shows_100_tokens_later(folders, name):
    """Two sequences that differ in their first token only: 100 tokens later the engine's logits differ by what the
    plain implementation says, in a model whose only path back is a kept first token, or a head that does not decay."""
    from hfee_amd.trace_replay import Replayer
    folder = folders[(name, "float32")]
    toks = tu.make_requests(50, [101], seed=3)["r0"]
    other = [(toks[0] + 7) % 50] + toks[1:]
    rep = Replayer(folder, "float32", 256, max_requests=2)
    got = tu.run(rep, [{"entries": [("a", toks[:60], []), ("b", other[:60], [])], "end": []},
                       {"entries": [("b", other[60:], [40]), ("a", toks[60:], [40])], "end": ["a", "b"]}])
    want = plain_logits(folder, toks)[100] - plain_logits(folder, other)[100]
    assert np.abs(want).max() > 1e-6
    assert mu.rel(got[("a", 100)] - got[("b", 100)], want) < 1e-2


def test_the_shift_reaches_over_a_chunks_edge_and_a_steps(folders):
    """At a chunk's first position the token before it is out of sight of the attention and reaches it through the
    token shift alone; with every token a step of its own that row comes from the slot."""
    from hfee_amd.trace_replay import Replayer
    folder = folders[("chunk", "float32")]
    toks = tu.make_requests(50, [13], seed=4)["r0"]
    other = list(toks)
    other[11] = (other[11] + 5) % 50
    rep = Replayer(folder, "float32", 128, max_requests=2)
    steps = [{"entries": [("a", toks[i:i + 1], [0]), ("b", other[i:i + 1], [0])], "end": []} for i in range(13)]
    got = tu.run(rep, steps)
    want = plain_logits(folder, toks)[12] - plain_logits(folder, other)[12]
    assert np.abs(want).max() > 1e-4 and mu.rel(got[("a", 12)] - got[("b", 12)], want) < 1e-3


def greedy(folder, prompt, count):
    seq = list(prompt)
    for _ in range(count):
        seq.append(int(np.argmax(plain_logits(folder, seq)[-1])))
    return seq[len(prompt):]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_entry_point(folders, dtype):
    from hfee_amd import LLM, SamplingParams
    folder = folders[("A" if dtype == "float32" else "A every expert", dtype)]      # (no router's near tie in bfloat16)
    llm = LLM(folder, dtype=dtype, num_ctx=128, num_parallel=3, max_batch_tokens=24)
    g = np.random.default_rng(5)
    prompts = [g.integers(0, 131, size=n).tolist() for n in (5, 40, 1, 17, 33)]
    outs = llm.generate(prompts, SamplingParams.greedy(num_predict=8))
    for p, o in zip(prompts, outs):
        want = greedy(folder, p, 8)
        if dtype == "float32":
            assert o.token_ids == want
        else:
            logits = plain_logits(folder, p + want)
            margins = []
            for i in range(8):
                row = np.sort(logits[len(p) - 1 + i])
                margins.append(float((row[-1] - row[-2]) / np.abs(row).max()))
            tu.agree_until_a_near_tie(o.token_ids, want, margins, f"greedy {dtype}")


def test_trace_runner_as_a_subprocess(folders, tmp_path):
    folder = folders[("B", "float32")]
    toks = list(range(1, 40))
    lines = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:21], "want": [0, 20]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[21:22], "want": []}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[22:], "want": [16]}, {"id": "y", "tokens": toks[:2], "want": [1]}],
              "end": ["x", "y"]}]
    out = tmp_path / "out"
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32",
                        "--out", str(out), "--max-tokens", "128"], input="\n".join(json.dumps(l) for l in lines) + "\n",
                       capture_output=True, text=True, timeout=600)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [l for l in p.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = plain_logits(folder, toks)
    a = np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1)
    c = np.fromfile(out / "2.f32", dtype="<f4").reshape(2, -1)
    assert not (out / "1.f32").exists()
    assert mu.rel(a[0], want[0]) < 3e-5 and mu.rel(a[1], want[20]) < 3e-5
    assert mu.rel(c[0], want[38]) < 3e-5 and mu.rel(c[1], want[1]) < 3e-5


def test_the_command_line_runs_the_design(folders):
    """`hfee run <folder> --tokens ...`: the greedy continuation's ids."""
    folder = folders[("B", "float32")]
    prompt = tu.make_requests(97, [11], seed=8)["r0"]
    want = greedy(folder, prompt, 7)
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "hfee"), "run", folder, "--tokens",
                        ",".join(map(str, prompt)), "--dtype", "float32", "--temperature", "0", "--repeat-penalty", "1",
                        "--num-predict", "7", "--num-ctx", "128", "--verbose"],
                       capture_output=True, text=True, timeout=300, stdin=subprocess.DEVNULL)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [int(t) for t in p.stdout.strip().splitlines()[0].split()] == want
