"""The Miberax decoder on the GPU against the plain implementation: the new kernels alone (norms in groups, the pair's
norms with the addition and the next norm, the launch in which the experts' outputs join the stream, the polynomial of
normed powers, the router with groups and corrections, what enters the delta rule, the delta rule token by token and in
chunks, the heads' norm and gate), each mechanism as a model of one layer, the whole model under four ways of cutting
the same requests into steps (whole, bulk then single tokens, portions down to two tokens, mixed batches on a small page
pool with four state slots, pages and slots used again), in 32-bit and in bfloat16, on configurations with even and with
odd sizes; keys that stand out on both sides of a chunk's edge; long decoding through graph replays; greedy generation
through the entry point and its scheduler; the trace runner and the command line as subprocesses."""
import json
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

import miberax_util as bu
import plain_miberax as pb
import trace_util as tu
from conftest import ROOT

pytestmark = pytest.mark.gpu

TOL = {"float32": 3e-5, "bfloat16": 8e-2}
DT = {"float32": torch.float32, "bfloat16": torch.bfloat16}
LENGTHS = {"A": [5, 17, 64, 1, 100, 38, 129, 49, 2], "B": [40, 3, 100, 65, 2, 31], "C": [420, 47, 311, 1, 161]}
NAN = float("nan")


def i32(a):
    return torch.as_tensor(np.asarray(a, dtype=np.int32)).cuda()


# ------------------------------------------------------------------ kernels alone

ROWS = [(8, 4096, 4), (70, 72, 3), (3, 5000, 2), (40, 1024, 1), (1, 58, 2), (5, 20000, 5), (9, 78, 3), (300, 128, 1), (6, 256, 2),
        (4, 2048, 8), (2, 33000, 3), (7, 60, 60)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width,groups", ROWS)
def test_the_norm_in_groups(dtype, n, width, groups):
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + width)
    # (groups of very unequal size, so that a part normed with another's sum would show)
    x = torch.randn(n + 3, width, generator=g) * torch.logspace(-2, 1, groups).repeat_interleave(width // groups)
    w = torch.rand(width, generator=g) + 0.5
    out = torch.zeros(n, width, dtype=DT[dtype], device="cuda")
    tol = 2e-6 if dtype == "float32" else 1e-2
    for rows in (None, torch.randperm(n + 3, generator=g)[:n]):
        ops.group_norm(out, x.cuda(), w.cuda(), 1e-3, groups, rows=None if rows is None else i32(rows))
        want = pb.group_norm((x[:n] if rows is None else x[rows]).double(), w.double(), groups, 1e-3)
        assert bu.rel(out.double().cpu(), want) < tol
        each = (out.double().cpu() - want).view(n, groups, -1).abs().amax((0, 2)) / want.view(n, groups, -1).abs().amax((0, 2))
        assert each.max() < tol


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width,groups", ROWS)
def test_two_normed_results_join_the_stream(dtype, n, width, groups):
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + width)
    x, y, y2 = (torch.randn(n, width, generator=g) * s for s in (1.0, 5.0, 0.02))
    w1, w2, w3 = (torch.rand(width, generator=g) + 0.5 for _ in range(3))
    want = x.double() + 0.5 * pb.rms(y.double(), 1e-4) * w1.double() + 0.25 * pb.rms(y2.double(), 1e-4) * w2.double()
    got = x.clone().cuda()
    ops.pair_norm_add(got, y.cuda(), y2.cuda(), w1.cuda(), w2.cuda(), 1e-4, (0.5, 0.25))
    assert bu.rel(got.double().cpu(), want) < 2e-6
    got, nxt = x.clone().cuda(), torch.zeros(n, width, dtype=DT[dtype], device="cuda")
    ops.pair_norm_add(got, y.cuda(), y2.cuda(), w1.cuda(), w2.cuda(), 1e-4, (0.5, 0.25), next_out=nxt, next_weight=w3.cuda(), next_eps=1e-3,
                      next_groups=groups)
    assert bu.rel(got.double().cpu(), want) < 2e-6
    assert bu.rel(nxt.double().cpu(), pb.group_norm(want, w3.double(), groups, 1e-3)) < (3e-6 if dtype == "float32" else 1e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width,groups", ROWS)
@pytest.mark.parametrize("top,experts,outputs", [(3, 4, 7), (1, 2, 4), (2, 5, 5)])
def test_the_experts_join_the_stream(dtype, n, width, groups, top, experts, outputs):
    """The pairs' rows one by one and already summed, experts that hand on their input (whose rows hold NaNs), with and
    without the shared one and its gate, the next norm written where the input lies."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + width + top)
    x, shared, gates = torch.randn(n, width, generator=g), torch.randn(n, width, generator=g), torch.randn(n, 5, generator=g)
    h = torch.randn(n, width, generator=g).to(DT[dtype])
    y, w3 = torch.randn(n, top, width, generator=g), torch.rand(width, generator=g) + 0.5
    chosen = torch.stack([torch.randperm(outputs, generator=g)[:top] for _ in range(n)])
    weights = torch.rand(n, top, generator=g)
    real = (chosen < experts)[..., None]
    routed = (weights[..., None].double() * torch.where(real, y, torch.zeros(()))).sum(1)
    handed = (weights.double() * (chosen >= experts)).sum(1, keepdim=True) * h.double()
    pairs = torch.where(real, y, torch.full((), NAN)).reshape(n * top, width)
    for given, s, gate in ((pairs, shared, gates[:, 2]), (pairs, None, None), (routed.float(), shared, None)):
        want = x.double() + routed + handed
        if s is not None:
            want = want + s.double() * (1.0 if gate is None else torch.sigmoid(gate.double())[:, None])
        got, hn = x.clone().cuda(), h.clone().cuda()
        args = dict(summed=given is not pairs, shared=None if s is None else s.cuda(), gate=None if gate is None else gates.cuda()[:, 2])
        ops.experts_join(got, given.cuda(), i32(chosen), weights.cuda(), experts, hn, **args)
        assert bu.rel(got.double().cpu(), want) < 2e-6 and torch.equal(hn.cpu(), h)
        got = x.clone().cuda()
        ops.experts_join(got, given.cuda(), i32(chosen), weights.cuda(), experts, hn, next_out=hn, next_weight=w3.cuda(), next_eps=1e-3,
                         next_groups=groups, **args)
        assert bu.rel(got.double().cpu(), want) < 2e-6
        assert bu.rel(hn.double().cpu(), pb.group_norm(want, w3.double(), groups, 1e-3)) < (3e-6 if dtype == "float32" else 1e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,width", [(9, 40), (70, 33), (3, 5000), (300, 4096), (2, 21504), (4, 33000), (1, 10), (5, 16384)])
def test_the_polynomial_of_normed_powers(dtype, n, width):
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + width)
    wide = torch.randn(n, width + 8, generator=g).to(DT[dtype])
    z, numbers = wide[:, :width], torch.tensor([0.7, -1.3, 0.4, 0.2])
    want = pb.poly_norm(z.double(), numbers.double(), 1e-3)
    tol = 3e-6 if dtype == "float32" else 1e-2
    buffer = wide.cuda()
    out = torch.zeros(n, width, dtype=DT[dtype], device="cuda")
    ops.poly_norm(out, buffer[:, :width], numbers.cuda(), 1e-3)
    assert bu.rel(out.double().cpu(), want) < tol
    ops.poly_norm(buffer[:, :width], buffer[:, :width], numbers.cuda(), 1e-3)          # in place
    assert bu.rel(buffer[:, :width].double().cpu(), want) < tol and torch.equal(buffer[:, width:].cpu(), wide[:, width:])


@pytest.mark.parametrize("n,outputs,top,groups", [(50, 8, 3, (4, 3)), (7, 70, 3, (7, 2)), (33, 4, 4, (2, 2)), (9, 130, 5, (10, 3)),
                                                  (20, 16, 3, None), (41, 64, 8, (8, 4)), (12, 64, 64, None), (15, 96, 2, (96, 5)),
                                                  (15, 60, 2, (60, 5)), (6, 200, 40, (2, 1)), (30, 20, 4, (1, 1)), (8, 9, 3, (3, 1))])
def test_the_router_with_groups(n, outputs, top, groups):
    """Corrections that make choice scores negative and move the choice, weights without them, divided by their sum."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(n + outputs)
    wide = torch.randn(n, outputs + 3, generator=g) * 2.0
    logits = wide[:, :outputs]
    r = {"top": top, "scale": 1.7}
    if groups:
        r["groups"] = dict(zip(("count", "keep"), groups))
    for correction in (torch.randn(outputs, generator=g) * 0.2 - 0.3, torch.zeros(outputs)):
        scores = torch.softmax(logits.double(), -1)
        chosen, weights, margin = pb.choose(scores, scores + correction.double(), r)
        clear = margin > 1e-6                                     # (float32 scores may tie where these do not)
        assert clear.float().mean() > 0.9
        got_chosen = torch.zeros(n, top, dtype=torch.int32, device="cuda")
        got_weights = torch.zeros(n, top, device="cuda")
        ops.router_topk(got_chosen, got_weights, wide.cuda()[:, :outputs], top, score="softmax", correction=correction.cuda(), groups=groups,
                        renormalize=True, scale=1.7)
        same = (torch.sort(got_chosen.cpu().long(), -1).values == torch.sort(chosen, -1).values).all(-1)
        assert same[clear].all()
        by_number = lambda c, w: torch.gather(w, 1, torch.argsort(c, -1))      # noqa: E731
        assert bu.rel(by_number(got_chosen.cpu().long(), got_weights.double().cpu())[clear], by_number(chosen, weights)[clear]) < 2e-6
    # the other kinds of scores go through both kernels as well
    for score, of in (("sigmoid", torch.sigmoid), ("softmax_chosen", None)):
        ops.router_topk(got_chosen, got_weights, wide.cuda()[:, :outputs], top, score=score)
        order = torch.sort(logits, dim=-1, descending=True, stable=True).indices[:, :top]
        picked = torch.gather(logits.double(), 1, order)
        assert torch.equal(got_chosen.cpu().long(), order)
        assert bu.rel(got_weights.double().cpu(), of(picked) if of else torch.softmax(picked, -1)) < 1e-6


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("H,G,D,V,K", [(4, 2, 16, 32, 4), (2, 2, 32, 48, 3), (6, 3, 8, 16, 2), (3, 1, 16, 16, 1), (16, 8, 128, 256, 4),
                                       (1, 1, 4, 8, 4), (2, 1, 256, 20, 4), (3, 3, 64, 4, 3)])
def test_what_enters_the_delta_rule(dtype, H, G, D, V, K):
    """Two requests in other slots, in portions down to one token and in steps of single tokens: convolutions whose
    inputs before a portion come from the slot, unit vectors, decays and strengths; a slot of NaNs stays untouched."""
    from hfee_amd.kernels import ops
    dt = DT[dtype]
    g = torch.Generator().manual_seed(D + V + K)
    qk, C = G * D, 2 * G * D + H * V
    assert ops.delta_inputs_fit(C, D, K)
    lengths, slots = [90, 40], [2, 0]
    xs = [torch.randn(n, C, generator=g).to(dt) for n in lengths]
    ab = [torch.randn(n, 2 * H, generator=g).to(dt) for n in lengths]
    taps, bias, a_log = torch.randn(C, K, generator=g) * 0.6, torch.randn(H, generator=g), torch.randn(H, generator=g)
    want = []
    for x in xs:
        y = pb.silu(pb.short_conv(x.double(), taps.double()))
        heads = lambda t: pb.unit(t.view(-1, G, D)).reshape(-1, qk)      # noqa: E731
        want.append(torch.cat([heads(y[:, :qk]) * D ** -0.5, heads(y[:, qk:2 * qk]), y[:, 2 * qk:]], 1))
    state = torch.zeros(4, K - 1, C, dtype=dt, device="cuda")
    state[1].fill_(NAN)
    fed = [0, 0]
    for sizes in ([5, 2], [1, 1], [1, 1], [0, 3], [2, 0], [1, 1], [60, 9], [1, 0], [19, 23]):
        segs = [(s, n) for s, n in enumerate(sizes) if n]
        n_all = sum(n for _, n in segs)
        buffer = torch.cat([torch.cat([xs[s][fed[s]:fed[s] + n], ab[s][fed[s]:fed[s] + n]], 1) for s, n in segs])
        buffer = torch.nn.functional.pad(buffer, (0, -buffer.shape[1] % 8)).cuda()
        rows, lens, at = np.cumsum([0] + [n for _, n in segs])[:-1], [n for _, n in segs], i32([slots[s] for s, _ in segs])
        token_segment = i32(np.concatenate([np.full(n, i) for i, (_, n) in enumerate(segs)]))
        y = torch.zeros(n_all, C + 4, device="cuda")[:, :C]
        decay, beta = torch.zeros(n_all, H, device="cuda"), torch.zeros(n_all, H, device="cuda")
        singles = n_all == len(segs)
        ops.delta_inputs(y, decay, beta, buffer[:, :C], buffer[:, C:C + H], buffer[:, C + H:C + 2 * H], state, taps.cuda(), bias.cuda(),
                         a_log.cuda(), token_segment, i32(rows), at, qk, D, H, 1e-6, D ** -0.5, keep=singles)
        if not singles:
            ops.short_conv_keep(state, buffer[:, :C], i32(rows), i32(lens), at)
        row = 0
        for s, n in segs:
            part = slice(fed[s], fed[s] + n)
            for cols in (slice(0, qk), slice(qk, 2 * qk), slice(2 * qk, C)):
                assert bu.rel(y[row:row + n, cols].double().cpu(), want[s][part, cols]) < 5e-6, (sizes, s, cols)
            z = ab[s][part].double()
            g_want = torch.exp(-torch.exp(a_log.double()) * torch.nn.functional.softplus(z[:, :H] + bias.double()))
            assert bu.rel(decay[row:row + n].double().cpu(), g_want) < 5e-6
            assert bu.rel(beta[row:row + n].double().cpu(), torch.sigmoid(z[:, H:])) < 2e-6
            fed[s] += n
            row += n
            for k in range(K - 1):
                i = fed[s] - (K - 1) + k
                assert torch.equal(state[slots[s], k].cpu(), xs[s][i] if i >= 0 else torch.zeros(C, dtype=dt))
    assert fed == lengths and torch.isnan(state[1].float()).all()


@pytest.mark.parametrize("chunks", [False, True])
@pytest.mark.parametrize("H,G,D,V,kind", [
    (2, 2, 16, 32, "mixed"), (3, 1, 12, 20, "mixed"), (4, 2, 64, 64, "mixed"), (1, 1, 4, 4, "mixed"), (4, 2, 128, 256, "mixed"),
    (3, 3, 100, 17, "mixed"), (2, 1, 256, 48, "mixed"), (2, 2, 32, 32, "alike"), (2, 1, 128, 16, "alike"), (2, 2, 16, 16, "no decay"),
    (2, 2, 64, 16, "all forgotten"), (3, 3, 32, 64, "far")])
def test_the_delta_rule_in_portions(H, G, D, V, kind, chunks):
    """Two requests in other slots, in portions of unequal size, token by token and with the long portions in chunks,
    against the definition token by token in float64, the last states too; keys that are almost the same vector, no
    decay at all, decays of zero, and one key far back that a query much later reads alone; a slot of NaNs beside them
    stays untouched, the scratch is full of NaNs."""
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(H + D + V)
    lengths, slots = [290, 90], [2, 0]
    data = []
    for n in lengths:
        k = torch.randn(n, G, D, generator=g)
        if kind == "alike":
            k = torch.randn(1, G, D, generator=g) + 0.05 * k
        decay = torch.rand(n, H, generator=g) ** (3.0 * torch.rand(H, generator=g)) * 0.2 + 0.8
        decay[:, 0] = 1.0
        decay[::7] *= 0.02
        if kind in ("no decay", "far"):
            decay.fill_(1.0)
        if kind == "all forgotten":
            decay[::5] = 0.0
            decay[3::11] = 1e-30
        q, beta = torch.randn(n, G, D, generator=g), torch.rand(n, H, generator=g)
        if kind == "far":                       # (everything but the far key is at right angles to what reads it)
            k[..., 0] = q[..., 0] = 0.0
            k[2] = 0.0
            k[2, :, 0] = q[-1, :, 0] = 1.0
            q[-1, :, 1:] = 0.0
        q, k = pb.unit(q.double()).float() * D ** -0.5, pb.unit(k.double()).float()
        data.append((q, k, torch.randn(n, H, V, generator=g), beta, decay))
    want, last = zip(*[pb.delta_rule(q.double().repeat_interleave(H // G, 1), k.double().repeat_interleave(H // G, 1), v.double(),
                                     b.double(), d.double()) for q, k, v, b, d in data])
    if kind == "far":
        assert want[0][-1].abs().max() > 0.05
    state = torch.zeros(4, H, *ops.scan_state_shape(D, V), device="cuda")
    state[1].fill_(NAN)
    fed = [0, 0]
    for sizes in ([5, 2], [1, 1], [40, 0], [2, 17], [150, 3], [64, 65], [28, 2]):
        segs = [(s, n) for s, n in enumerate(sizes) if n]
        cat = lambda i: torch.cat([data[s][i][fed[s]:fed[s] + n].reshape(n, -1) for s, n in segs]).cuda()      # noqa: E731
        q, k, v, beta, decay = (cat(i) for i in range(5))
        rows = np.cumsum([0] + [n for _, n in segs])[:-1]
        out = torch.zeros(q.shape[0], H * V, device="cuda")
        more = {}
        words = ops.delta_chunks_scratch(max(n for _, n in segs), q.shape[0], H, D, V)
        if chunks and words:
            more = dict(scratch=torch.full((words,), NAN, device="cuda"), longest=max(n for _, n in segs), shortest=min(n for _, n in segs))
        ops.linear_scan(out, state, q, k, v, decay, beta, i32(rows), i32([n for _, n in segs]), i32([slots[s] for s, _ in segs]),
                        H, G, D, V, "delta", decay_per_head=True, **more)
        row = 0
        for s, n in segs:
            w = want[s][fed[s]:fed[s] + n].reshape(n, -1)
            err = (out[row:row + n].double().cpu() - w).abs().max() / want[s].abs().max()
            assert err < 2e-5, (sizes, s, float(err))
            fed[s] += n
            row += n
            if kind == "far" and fed[s] == lengths[s]:
                assert bu.rel(out[row - 1].double().cpu(), w[-1]) < 2e-5
    assert fed == lengths and torch.isnan(state[1]).all() and torch.isfinite(state[[0, 2, 3]]).all()
    for s in (0, 1):
        got = ops.scan_state_matrix(state[slots[s]], D, V).double().cpu()
        assert (got - last[s]).abs().max() / last[s].abs().max() < 2e-5


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n,H,V", [(5, 3, 20), (70, 16, 256), (3, 2, 7), (40, 4, 96), (1, 5, 4), (9, 2, 640), (2, 3, 1020)])
def test_heads_normed_and_gated(dtype, n, H, V):
    from hfee_amd.kernels import ops
    g = torch.Generator().manual_seed(V)
    wide = torch.randn(n, H * V + 24, generator=g).to(DT[dtype])
    o, z, w = torch.randn(n, H * V, generator=g), wide[:, 16:16 + H * V], torch.rand(V, generator=g) + 0.5
    for act, of in (("silu", pb.silu), ("sigmoid", torch.sigmoid)):
        out = torch.zeros(n, H * V, dtype=DT[dtype], device="cuda")
        ops.head_norm_gate(out, o.cuda(), wide.cuda()[:, 16:16 + H * V], w.cuda(), H, V, 1e-4, act)
        want = (pb.rms(o.double().view(n, H, V), 1e-4) * w.double()).reshape(n, -1) * of(z.double())
        assert bu.rel(out.double().cpu(), want) < (2e-6 if dtype == "float32" else 1e-2)


# ------------------------------------------------------------------ the whole model

@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    base = tmp_path_factory.mktemp("miberax")
    return {(name, dtype): bu.make_folder(base / f"{name.replace(' ', '_')}_{dtype}", cj, seed=7 + ord(name[0]), dtype=dtype,
                                          silent=bu.SILENT.get(name))
            for name, cj in list(bu.CONFIGS.items()) + list(bu.SINGLE.items()) for dtype in ("float32", "bfloat16")}


def plain_logits(folder, tokens, margins=None, moved=None):
    """The plain implementation's logits; margins: a list that receives, a position, the smallest margin by
    which any of its routers chose; moved: one that receives by how much the logits move at most, relative to the
    largest, in four draws of changing every weight at random by about twice a bfloat16's rounding."""
    cj, w = bu.load_plain(folder)
    each = []
    logits = pb.forward(tokens, w, cj, margins=each).numpy()
    if margins is not None:
        margins.extend(torch.stack(each).min(0).values.tolist() if each else [float("inf")] * len(tokens))
    if moved is not None:
        g, most = torch.Generator().manual_seed(0), np.zeros(len(tokens))
        for _ in range(4):
            noisy = {n: t.double() * (1.0 + 0.003 * torch.randn(t.shape, generator=g)) for n, t in w.items()}
            other = pb.forward(tokens, noisy, cj).numpy()
            most = np.maximum(most, np.abs(other - logits).max(1) / np.abs(logits).max(1))
        moved.extend(most.tolist())
    return logits


# In bfloat16 a router reads rounded numbers: a token whose last chosen expert and the best one not chosen score
# almost alike may go to the other one, and the states and the cache carry the difference to every token behind
# it.  So in bfloat16 a request is compared up to the first position at which a router of the plain
# implementation chose by less than NEAR_TIE, and the configurations in which every token uses every expert
# ("... every expert": nothing is chosen) are compared up to the end.  And what a head reads is divided by its own root
# mean square: where a key and a query are almost at right angles and little else has been written (a sequence's first
# tokens), the result's direction is rounding's.  So in bfloat16 the positions whose plain logits move by more than
# the tolerance under changes of the weights by such amounts are left to the 32-bit comparison.
NEAR_TIE = 0.01


class Rows(dict):
    """(request, position) -> logits of the plain implementation; `.margins`: -> the routers' smallest margin;
    `.moved`: -> see plain_logits."""
    margins: dict
    moved: dict


def add_rows(rows, folder, rid, toks, dtype, first=0):
    margins, moved = [], [] if dtype == "bfloat16" else None
    logits = plain_logits(folder, toks, margins, moved)
    rows.update({(rid, i): logits[i] for i in range(first, len(toks))})
    rows.margins.update({(rid, i): margins[i] for i in range(len(toks))})
    rows.moved.update({(rid, i): m for i, m in enumerate(moved or [])})


@pytest.fixture(scope="module")
def plain_rows(folders):
    cache = {}

    def get(name, dtype, lengths=None):
        key = (name, dtype, tuple(lengths or LENGTHS[name[0]]))
        if key not in cache:
            cj = (bu.CONFIGS.get(name) or bu.SINGLE[name])
            reqs = tu.make_requests(cj["vocab"], list(key[2]), seed=ord(name[0]))
            rows = Rows()
            rows.margins, rows.moved = {}, {}
            for rid, toks in reqs.items():
                add_rows(rows, folders[(name, dtype)], rid, toks, dtype)
            cache[key] = (reqs, rows)
        return cache[key]
    return get


def compare(got, want, dtype, what):
    """32-bit: every position within the tolerance.  bfloat16: every position before its request's first near
    tie and where rounding alone does not move it (see NEAR_TIE) within twice the tolerance and all but one in a hundred of
    them (or one) within it; over those positions the median is well within it."""
    assert set(got) == set(want), f"{what}: positions differ"
    tol = TOL[dtype]
    margins, moved = getattr(want, "margins", {}), getattr(want, "moved", {})
    errors = {key: bu.rel(got[key], want[key]) for key in want}
    keys = sorted(want)
    if dtype != "float32":
        first_tie = {}
        for rid, at in keys:
            if margins.get((rid, at), float("inf")) < NEAR_TIE:
                first_tie[rid] = min(at, first_tie.get(rid, at))
        keys = [(rid, at) for rid, at in keys if at < first_tie.get(rid, at + 1) and moved.get((rid, at), 0.0) < tol]
    over = sorted((errors[key], key) for key in keys if not errors[key] < tol)
    allowed = 0 if dtype == "float32" else max(1, len(keys) // 100)
    assert keys and len(over) <= allowed and not any(e >= 2 * tol for e, _ in over), \
        f"{what}: {len(over)} of {len(keys)} positions beyond {tol}, the worst {over[-1:]}, the first {min(k for _, k in over) if over else None}"
    median = np.median([errors[key] for key in keys])
    assert median < tol / 2, f"{what}: median relative error {median:.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(bu.SINGLE))
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
    for name in ("A", "C"):
        reqs, _ = plain_rows(name, "float32")
        runs = []
        for steps in (tu.whole(reqs), tu.portions(reqs, sizes=(2, 3, 16, 1, 15, 17, 2, 70, 64)), tu.bulk_then_tail(reqs, 20)):
            runs.append(tu.run(Replayer(folders[(name, "float32")], "float32", 448, max_requests=4), steps))
        for other in runs[1:]:
            for key in runs[0]:
                assert bu.rel(other[key], runs[0][key]) < 2e-5, (name, key)


@pytest.mark.parametrize("name", ["A", "B"])
def test_a_slot_that_is_used_again_starts_from_nothing(folders, plain_rows, name):
    """One state slot and a pool of one request's pages: every request inherits the slot and the pages of the
    one before, whose states and convolution inputs must be gone."""
    from hfee_amd.trace_replay import Replayer
    reqs, want = plain_rows(name, "float32")
    longest = max(len(t) for t in reqs.values())
    rep = Replayer(folders[(name, "float32")], "float32", (longest + 63) // 64 * 64, max_requests=1)
    got = tu.run(rep, tu.portions(reqs, sizes=(9, 2, 30)))
    compare(got, want, "float32", f"{name}: one slot for all")


def test_chunks_give_back_the_pages_they_have_passed(folders, plain_rows):
    """A chunk's cache is a window group of the manager: a request of 150 tokens holds the pages of its reach and no
    more, whether it came in portions or token by token, and its logits are the plain ones."""
    from hfee_amd.trace_replay import Replayer
    reqs, want = plain_rows("chunk", "float32", [150])
    toks = reqs["r0"]
    rep = Replayer(folders[("chunk", "float32")], "float32", 192, max_requests=2)
    assert [(g.kind, g.window) for g in rep.engine.cache.groups] == [("window", 6)]
    got, fed = {}, 0
    for n in [40, 3, 2, 50] + [1] * 55:
        rows = rep.step([("r0", toks[fed:fed + n], list(range(n)))])
        got.update({("r0", fed + i): rows[i] for i in range(n)})
        fed += n
        assert sum(p >= 0 for p in rep.engine.cache.get("r0").tables[0]) <= 2
        rep.engine.cache.check()
    compare(got, want, "float32", "chunk: a window group")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,dim,chunk,rot", [(4, 32, 50, 32), (2, 16, 33, 8), (3, 10, 48, 6), (4, 64, 0, 64)])
def test_keys_that_stand_out_around_a_chunks_edge(tmp_path, dtype, heads, dim, chunk, rot):
    """A model of one attention layer in which every query looks hardest at one token's keys (W_q and W_k alike, the
    token's embedding large in what they read): placed as a chunk's last, first and second token, at a page's borders
    and as the sequence's first, with queries inside the chunk and just behind it, in prompts and token by token."""
    from hfee_amd.trace_replay import Replayer
    size = chunk or 200
    cj = bu.config(40, 64, 1e-6, 2, [bu.bare(bu.pair(bu.attention(heads, heads, dim, 32 if dim == 64 else 16, 4.0 / dim, chunk=chunk or None,
                                                                 rot=bu.rotation(rot, 1e6, 8.0)), bu._TINY_RIGHT))])
    w = bu.make_tensors(cj, 11, silent="right")
    w["l0.mix.left.k"] = w["l0.mix.left.q"].clone()
    w["embed"][7] = w["embed"][:7].mean(0) * 3.0          # (what the queries of the others have in common)
    w["embed"][8:] += w["embed"][7]
    folder = bu.make_folder(tmp_path / "m", cj, 0, dtype, tensors=w)
    rng = np.random.default_rng(3)
    reqs = {}
    for i, at in enumerate([0, size - 1, size, size + 1, 15, 16, 2 * size - 1, 31]):
        toks = rng.integers(8, 40, size=2 * size + 9)
        toks[at] = 7
        reqs[f"r{i}"] = toks.tolist()
    want = Rows()
    want.margins, want.moved = {}, {}
    for rid, t in reqs.items():
        add_rows(want, folder, rid, t, dtype)
    room = (2 * size + 9 + 63) // 64 * 64
    for what, steps in (("whole", tu.whole(reqs)), ("tail", tu.bulk_then_tail(reqs, size + 12)), ("portions", tu.portions(reqs))):
        compare(tu.run(Replayer(folder, dtype, room, max_requests=2), steps), want, dtype, f"standing out {what}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(folders, dtype):
    """300 single tokens after a short prompt: decode steps replayed from captured graphs, across page borders and
    chunks' edges, the states carried through every replay; a second request joins on the way, so that steps of two
    rows are replayed as well."""
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
    want = Rows()
    want.margins, want.moved = {}, {}
    for rid, t, first in (("a", toks, 29), ("b", other, 9)):
        add_rows(want, folders[(name, dtype)], rid, t, dtype, first)
    compare(got, want, dtype, f"long decoding {dtype}")


@pytest.mark.parametrize("at", [0, 1, 40])
def test_an_early_token_shows_much_later_through_the_recurrence_alone(folders, at):
    """Two sequences that differ in one token only: 60 to 100 tokens later the engine's logits differ by what the plain
    implementation says, in a model whose only path back is the recurrence; in the model whose only mixer is
    attention over chunks of six they do not differ at all."""
    from hfee_amd.trace_replay import Replayer
    toks = tu.make_requests(50, [101], seed=3)["r0"]
    other = list(toks)
    other[at] = (toks[at] + 7) % 50
    for name, moves in (("delta", True), ("chunk", False)):
        folder = folders[(name, "float32")]
        rep = Replayer(folder, "float32", 256, max_requests=2)
        got = tu.run(rep, [{"entries": [("a", toks[:60], []), ("b", other[:60], [])], "end": []},
                           {"entries": [("b", other[60:], [40]), ("a", toks[60:], [40])], "end": ["a", "b"]}])
        want = plain_logits(folder, toks)[100] - plain_logits(folder, other)[100]
        if moves:
            assert np.abs(want).max() > 1e-4
            assert bu.rel(got[("a", 100)] - got[("b", 100)], want) < 2e-2
        else:
            assert np.abs(want).max() == 0.0 and np.array_equal(got[("a", 100)], got[("b", 100)])


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
    assert bu.rel(a[0], want[0]) < 3e-5 and bu.rel(a[1], want[20]) < 3e-5
    assert bu.rel(c[0], want[38]) < 3e-5 and bu.rel(c[1], want[1]) < 3e-5


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
