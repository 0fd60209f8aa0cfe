"""The Medulorn design without a GPU: the configuration's round trip and its errors, the declared tensors, the cache
manager's window that keeps a sequence's first tokens, and the plain implementation pinned by hand-worked cases: what a
query sees around a chunk's and a window's edge and of the first tokens, both sinks, the stretched rotation, the
recurrence against its closed form, the clipped expert, the router's softmax over the chosen, the token shift, the
norm behind the sum and the cap on the logits."""
import copy
import math

import numpy as np
import pytest
import torch

import medulorn_util as mu
import plain_medulorn as pm

F64 = torch.float64


def test_configuration_round_trip_and_what_it_leaves_out():
    from hfee_amd.config import config_from_dict
    for cj in list(mu.CONFIGS.values()) + list(mu.SINGLE.values()):
        cfg = config_from_dict(cj)
        assert cfg.to_dict() == cj
        assert config_from_dict(cfg.to_dict()) == cfg
    cfg = config_from_dict(mu.M_A)
    assert cfg.alpha == 1.7 and cfg.embedding_scale == 8.0 and cfg.logit_softcap == 9.0 and cfg.layers[2].mlp is None
    assert cfg.layers[1].mixer.left.keep_first == 3 and cfg.layers[1].mixer.left.rot.scaling == (4.0, 1.0, 4.0, 64.0)
    assert cfg.layers[0].mlp.shared == (64, 1.2) and cfg.layers[3].mlp.shared is None
    last = config_from_dict(mu.M_B).layers[4].mixer
    assert (last.chunk, last.rot) == (0, None) and config_from_dict(mu.M_B).logit_softcap == 0.0
    # sizes that an entry leaves out: as many key heads as heads, values as wide as keys, the whole head rotated
    cj = copy.deepcopy(mu.SINGLE["chunk"])
    for key in ("kv_heads", "vdim"):
        del cj["layers"][0]["mixer"][key]
    del cj["layers"][0]["mixer"]["rot"]["dims"]
    m = config_from_dict(cj).layers[0].mixer
    assert (m.kv_heads, m.vdim, m.rot.dims) == (3, 16, 16)


@pytest.mark.parametrize("change,message", [
    (lambda c: c["layers"][0]["mixer"].update(kv_heads=3), "multiple"),
    (lambda c: c["layers"][0]["mixer"]["rot"].update(dims=34), "do not fit"),
    (lambda c: c["layers"][0]["mixer"]["mask"].update(size=0), "positive"),
    (lambda c: c["layers"][1]["mixer"]["left"]["mask"].update(keep_first=-1), "keep_first"),
    (lambda c: c["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(low=5.0), "below high"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5]), "decay"),
    (lambda c: c["layers"][1]["mixer"]["right"].update(decay=[0.5, 1.5]), "between 0 and 1"),
    (lambda c: c["layers"][1]["mixer"].pop("right"), "right"),
    (lambda c: c["layers"][2].update(type="other"), "unknown mixer"),
    (lambda c: c["layers"][0]["mlp"].update(kind="other"), "unknown feed-forward"),
    (lambda c: c["layers"][0]["mlp"]["router"].update(top=9), "cannot use"),
    (lambda c: c["layers"][0]["mlp"]["expert"].pop("limit"), "limit"),
    (lambda c: c.update(logit_softcap=-1.0), "logit_softcap"),
    (lambda c: c.pop("width"), "width"),
])
def test_configuration_errors(change, message):
    from hfee_amd.config import ConfigError, config_from_dict
    cj = copy.deepcopy(mu.M_A)
    change(cj)
    with pytest.raises(ConfigError, match=message):
        config_from_dict(cj)


def test_declared_tensors():
    from hfee_amd.config import config_from_dict
    from hfee_amd.engine.model import declared_tensors
    shapes = {s.name: tuple(s.shape) for s in declared_tensors(config_from_dict(mu.M_A))}
    assert shapes["l0.norm1"] == shapes["l3.norm2"] == shapes["final.norm"] == () and "l2.norm2" not in shapes
    assert shapes["l0.shift"] == (64,) and shapes["l0.mix.q.b"] == (128,) and shapes["l0.mix.v.b"] == (32,)
    assert shapes["l0.mix.q.norm"] == shapes["l0.mix.k.norm"] == (32,)
    assert shapes["l1.mix.left.q.norm"] == (128,) and shapes["l1.mix.left.k.norm"] == (64,) and shapes["l1.mix.left.sink"] == (4,)
    assert "l1.mix.left.q.b" not in shapes and "l0.mix.sink" not in shapes
    assert shapes["l1.mix.right.g"] == (64, 64) and shapes["l1.mix.right.norm"] == (64,) and shapes["l1.mix.right.o"] == (64, 64)
    assert shapes["l1.mlp.gate"] == (96, 64) and shapes["l0.mlp.e5.down"] == (64, 32) and shapes["l0.mlp.router.b"] == (6,)
    assert shapes["l0.mlp.shared.up"] == (64, 64) and "l3.mlp.shared.up" not in shapes
    assert not any(n.startswith("l2.mlp") for n in shapes) and shapes["head"] == (131, 64)


# ------------------------------------------------------------------ the cache manager

def test_a_window_group_keeps_the_first_tokens():
    from hfee_amd.cache.manager import CacheError, CacheGroupSpec, CacheManager
    groups = [CacheGroupSpec("window", (2, 4), (0,), window=20, keep_first=18), CacheGroupSpec("window", (2, 4), (1,), window=20),
              CacheGroupSpec("full", (2, 4), (2,))]
    m = CacheManager(groups, 16, 12, 2)
    m.admit("a")
    first = None
    for n in [30, 1, 40, 16] + [1] * 60:
        m.reserve("a", n)
        m.commit("a", n)
        m.check()
        rc = m.get("a")
        kept, plain, full = ([b for b, p in enumerate(t) if p >= 0] for t in rc.tables)
        needed = set(range((rc.length - 20 + 1) // 16 if rc.length >= 20 else 0, -(-rc.length // 16)))
        assert set(plain) == needed and set(full) == set(range(-(-rc.length // 16)))
        assert set(kept) == needed | {0, 1}             # the first 18 tokens lie in the first two pages
        pages = rc.tables[0][:2]
        first = first or list(pages)
        assert list(pages) == first and list(rc.table_array(0)[:2]) == first
    m.release("a")
    m.check()
    assert m.free_pages() == [12, 12, 12]
    with pytest.raises(CacheError):
        CacheGroupSpec("full", (2, 4), (0,), keep_first=4)


# ------------------------------------------------------------------ what a query sees

def _one_layer(layer, width=24, vocab=40, seed=0, shift=0.0):
    cj = mu.config(vocab, width, 1e-6, 1.0, [mu.bare(layer)])
    w = {n: t.double() for n, t in mu.make_tensors(cj, seed, std=0.3).items()}
    w["l0.shift"] = torch.full_like(w["l0.shift"], shift)
    return cj, w


def _moved_by(cj, w, tokens, at, change):
    """Whether the logits at `at` move when the token at `change` is another one."""
    other = list(tokens)
    other[change] = (other[change] + 1) % cj["vocab"]
    a, b = pm.forward(tokens, w, cj)[at], pm.forward(other, w, cj)[at]
    return bool((a - b).abs().max() > 1e-9)


def test_what_a_query_sees():
    """One layer without a token shift: the logits at i move with token j exactly if i sees j."""
    tokens = list(np.random.default_rng(0).integers(0, 40, size=40))
    cj, w = _one_layer(mu.attention(2, 1, 4, 4, 0.5, chunk=7))
    assert _moved_by(cj, w, tokens, 34, 28) and not _moved_by(cj, w, tokens, 34, 27) and not _moved_by(cj, w, tokens, 34, 35)
    assert _moved_by(cj, w, tokens, 35, 35) and not _moved_by(cj, w, tokens, 35, 34) and _moved_by(cj, w, tokens, 6, 0)
    silent = mu.lightning(1, 2, 2, (0.0,))
    cj, w = _one_layer(mu.pair(mu.window(2, 1, 4, 4, 0.5, size=6, keep=3), silent, 1.0, 0.0))
    assert _moved_by(cj, w, tokens, 30, 25) and not _moved_by(cj, w, tokens, 30, 24)
    assert _moved_by(cj, w, tokens, 30, 2) and _moved_by(cj, w, tokens, 30, 0) and not _moved_by(cj, w, tokens, 30, 3)
    assert _moved_by(cj, w, tokens, 1, 0) and not _moved_by(cj, w, tokens, 0, 1)       # (a kept token that is still to come)
    # with a token shift a key carries the token before it as well
    cj, w = _one_layer(mu.attention(2, 1, 4, 4, 0.5, chunk=7), shift=0.5)
    assert _moved_by(cj, w, tokens, 34, 27) and not _moved_by(cj, w, tokens, 34, 26)
    # the recurrence reaches all the way back where a head does not decay
    cj, w = _one_layer(mu.pair(mu.window(1, 1, 4, 4, 0.5, size=1), mu.lightning(1, 4, 4, (1.0,)), 0.0, 1.0))
    assert _moved_by(cj, w, tokens, 39, 0)


def test_both_sinks_by_hand():
    s = torch.tensor([[[0.3, 0.0], [1.2, -0.4]], [[2.0, 0.0], [0.1, 0.5]]], dtype=F64)
    sight = torch.tensor([[True, False], [True, True]])
    p = pm.weigh(s, sight, torch.tensor([0.0, -1.0], dtype=F64))
    e = math.exp
    assert math.isclose(float(p[0, 0, 0]), e(0.3) / (1 + e(0.3))) and float(p[0, 0, 1]) == 0.0
    assert math.isclose(float(p[0, 1, 0]), e(1.2) / (1 + e(1.2) + e(-0.4)))
    assert math.isclose(float(p[1, 1, 1]), e(0.5) / (e(-1.0) + e(0.1) + e(0.5)))


def test_the_stretched_rotation_by_hand():
    """Wavelengths below original / high stay, those above original / low are divided, the rest is blended; the
    product's frequencies are the same."""
    from hfee_amd.parts.rotary import rope_frequencies
    rot = mu.rotation(16, 500.0, (4.0, 1.0, 4.0, 64.0))
    plain = [500.0 ** (-i / 8) for i in range(8)]
    got = pm.rotation_frequencies(rot)
    kinds = set()
    for i, f in enumerate(plain):
        wave = 2 * math.pi / f
        if wave < 16.0:
            want, kind = f, "kept"
        elif wave > 64.0:
            want, kind = f / 4.0, "divided"
        else:
            s = (64.0 / wave - 1.0) / 3.0
            want, kind = (1 - s) * f / 4.0 + s * f, "blended"
        kinds.add(kind)
        assert math.isclose(float(got[i]), want, rel_tol=1e-12)
    assert kinds == {"kept", "divided", "blended"}
    assert np.allclose(rope_frequencies(16, 500.0, ("llama3", 4.0, 1.0, 4.0, 64.0)), got.numpy(), rtol=1e-12)


def test_rotation_keeps_true_positions():
    q = torch.randn(9, 1, 6, dtype=F64, generator=torch.Generator().manual_seed(0))
    r = pm.rotate(q, {"base": 50.0, "dims": 4})
    a = 7 * 50.0 ** (-2.0 / 4)
    assert math.isclose(float(r[7, 0, 1]), float(q[7, 0, 1] * math.cos(a) - q[7, 0, 3] * math.sin(a)))
    assert math.isclose(float(r[7, 0, 3]), float(q[7, 0, 3] * math.cos(a) + q[7, 0, 1] * math.sin(a)))
    assert torch.equal(r[:, :, 4:], q[:, :, 4:]) and torch.equal(r[0], q[0])


def test_lightning_against_its_closed_form():
    cj, w = _one_layer(mu.pair(mu.window(1, 1, 4, 4, 0.5, size=1), mu.lightning(2, 4, 6, (0.9, 1.0))), seed=3)
    m, T, pre = cj["layers"][0]["mixer"]["right"], 12, "l0.mix.right."
    h = torch.randn(T, 24, dtype=F64, generator=torch.Generator().manual_seed(1))
    q, k, v = (torch.nn.functional.silu(h @ w[pre + n].T).view(T, 2, -1) for n in "qkv")
    o = torch.zeros(T, 2, 6, dtype=F64)
    for t in range(T):
        for j in range(t + 1):
            for hd, d in enumerate((0.9, 1.0)):
                o[t, hd] += d ** (t - j) * (q[t, hd] @ k[j, hd]) * v[j, hd]
    o = o.reshape(T, 12)
    o = o / torch.sqrt((o * o).mean(-1, keepdim=True) + 1e-6) * w[pre + "norm"]          # (both heads normed as one)
    want = (o * torch.sigmoid(h @ w[pre + "g"].T)) @ w[pre + "o"].T
    assert torch.allclose(pm.lightning(h, w, pre, m, 1e-6), want, atol=1e-10)


def test_the_clipped_expert_by_hand():
    eye = torch.eye(3, dtype=F64)
    w = {"gate": eye, "up": 2.0 * eye, "down": eye}
    h = torch.tensor([[3.0, -4.0, 0.25]], dtype=F64)
    got = pm.clipped_expert(h, w, "", 1.5)[0]
    want = [1.5 / (1 + math.exp(-1.702 * 1.5)) * 2.5,           # gate and up clipped from above
            -4.0 / (1 + math.exp(1.702 * 4.0)) * -0.5,          # the gate has no floor, up has
            0.25 / (1 + math.exp(-1.702 * 0.25)) * 1.5]
    assert torch.allclose(got, torch.tensor(want, dtype=F64))


def test_the_router_weighs_the_chosen_only():
    g = torch.Generator().manual_seed(0)
    h = torch.randn(5, 8, dtype=F64, generator=g)
    w = {"router": torch.randn(4, 8, dtype=F64, generator=g), "router.b": torch.zeros(4, dtype=F64)}
    chosen, weights, margin = pm.route(h, w, "", 2)
    z = h @ w["router"].T
    assert torch.equal(chosen, z.argsort(-1, descending=True)[:, :2]) and torch.allclose(weights.sum(-1), torch.ones(5, dtype=F64))
    assert torch.allclose(weights[:, 0] / weights[:, 1], torch.exp(torch.gather(z, 1, chosen)[:, 0] - torch.gather(z, 1, chosen)[:, 1]))
    assert (margin > 0).all()
    w["router.b"][3] = 100.0                      # (the bias chooses and weighs)
    chosen, weights, _ = pm.route(h, w, "", 2)
    assert (chosen[:, 0] == 3).all() and (weights[:, 0] > 1 - 1e-12).all()


def test_shift_norm_and_cap_by_hand():
    x = torch.tensor([[1.0, 2.0], [3.0, -2.0]], dtype=F64)
    assert torch.equal(pm.token_shift(x, torch.tensor([0.0, 1.0], dtype=F64)), torch.tensor([[1.0, 0.0], [3.0, 2.0]], dtype=F64))
    assert torch.allclose(pm.scalar_norm(x, torch.tensor(0.5, dtype=F64), 0.0)[0], torch.tensor([1.0, 2.0], dtype=F64) / math.sqrt(2.5) / 2)
    cj = copy.deepcopy(mu.SINGLE["chunk"])
    w = mu.make_tensors(cj, 1)
    plain = pm.forward([1, 2, 3], w, cj)
    cj["logit_softcap"] = 0.7
    assert torch.allclose(pm.forward([1, 2, 3], w, cj), 0.7 * torch.tanh(plain / 0.7))
    # the stream joins with alpha before the norm: a mixer of zeros leaves norm(alpha x), whatever alpha is
    w["l0.mix.o"] = torch.zeros_like(w["l0.mix.o"])
    streams = []
    pm.forward([1, 2, 3], w, cj, streams=streams)
    x0 = w["embed"][[1, 2, 3]].double()
    assert torch.allclose(streams[0], pm.scalar_norm(1.5 * x0, w["l0.norm1"].double(), 1e-6))


def test_a_prefix_does_not_depend_on_what_follows():
    cj = mu.M_A
    w = mu.make_tensors(cj, 5)
    tokens = list(np.random.default_rng(2).integers(0, cj["vocab"], size=50))
    full = pm.forward(tokens, w, cj)
    assert torch.allclose(pm.forward(tokens[:31], w, cj), full[:31], atol=1e-9)
