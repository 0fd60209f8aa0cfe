"""The Medulorn decoder as a list of parts.

Every layer is a "postnorm" block with a token shift: the mixer reads each token's stream mixed with that of the token
before it, x <- norm1(alpha x + mixer(h)), x <- norm2(alpha x + feed_forward(x)), with RMS norms of one number each and
one alpha for the whole model.  The mixer of a layer is grouped attention over chunks of positions
("kv_attention" with biases, a norm over each head of q and k, a chunk and a sink of zero), or two mixers side by
side ("side_by_side"): grouped attention over a sliding window that keeps the first tokens in sight ("kv_attention"
with a norm over the whole projections and a learned sink), and linear attention with a fixed decay a head
("lightning_attention").  The feed-forward is a gated one with relu ("gated_mlp"), experts with clipped gates that
a router chooses, beside one that every token uses ("routed_moe"), or none.  The lookup is scaled, the logits are
capped.  Which layer has which, and every size and constant, is config.json's.

What is fixed here is what the design fixes: the rotation's pairs (i, i + dims/2) behind the norms, biases in the
chunked attention only, the two kinds of sink, the sharpness 1.702 of the experts' gates, a softmax over the chosen
experts, a bias on the router.
"""
from __future__ import annotations

from ..config.medulorn import ChunkAttentionConfig, ClippedExpertsConfig, DenseConfig, MedulornConfig, PairConfig
from ..config.registry import register_architecture
from ..config.specs import (EmbeddingSpec, FeedForwardSpec, HeadSpec, LayerSpec, MixerSpec, ModelSpec, NormSpec, PositionSpec,
                            ScheduleEntry, params)

SHARPNESS = 1.702       # of the experts' gates: g sigmoid(1.702 g)


def _rope(head_dim: int, rot):
    if rot is None:
        return None
    scaling = None if rot.scaling is None else ("llama3", *rot.scaling)
    return PositionSpec("rope", params(head_dim=head_dim, rotary_dim=rot.dims, theta=rot.base, scaling=scaling, pairing="half"))


def _attention(cfg: MedulornConfig, m, **more) -> MixerSpec:
    names = (("q", "q"), ("k", "k"), ("v", "v"), ("o", "o"), ("q_bias", "q.b"), ("k_bias", "k.b"), ("v_bias", "v.b"),
             ("q_norm", "q.norm"), ("k_norm", "k.norm"), ("sink", "sink"))
    return MixerSpec("kv_attention", params(
        hidden=cfg.width, num_heads=m.heads, num_kv_heads=m.kv_heads, key_dim=m.dim, value_dim=m.vdim, scale=m.scale,
        norm_eps=cfg.norm_eps, names=names, **more), position=_rope(m.dim, m.rot))


def _mixer(cfg: MedulornConfig, m) -> MixerSpec:
    if isinstance(m, ChunkAttentionConfig):
        return _attention(cfg, m, bias=True, qk_norm="head", chunk=m.chunk, sink="zero")
    if isinstance(m, PairConfig):
        left = _attention(cfg, m.left, qk_norm="row", window=m.left.window, keep_first=m.left.keep_first, sink="learned")
        right = MixerSpec("lightning_attention", params(
            hidden=cfg.width, num_heads=m.right.heads, dim=m.right.dim, vdim=m.right.vdim, decay=m.right.decay,
            norm_eps=cfg.norm_eps, names=(("q", "q"), ("k", "k"), ("v", "v"), ("g", "g"), ("o", "o"), ("norm", "norm"))))
        return MixerSpec("side_by_side", params(hidden=cfg.width, left=left, right=right, left_scale=m.left_scale,
                                                right_scale=m.right_scale, names=(("left", "left."), ("right", "right."))))
    raise ValueError(f"no part for a mixer of type {m.type!r}")


def _feed_forward(cfg: MedulornConfig, mlp):
    if mlp is None:
        return None
    matrices = (("gate", "gate"), ("up", "up"), ("down", "down"))
    if isinstance(mlp, DenseConfig):
        return FeedForwardSpec("gated_mlp", params(hidden=cfg.width, intermediate=mlp.ff, activation="relu", names=matrices))
    if isinstance(mlp, ClippedExpertsConfig):
        shared = None if mlp.shared is None else (mlp.shared[0], (mlp.shared[1], SHARPNESS))
        return FeedForwardSpec("routed_moe", params(
            hidden=cfg.width, intermediate=mlp.ff, experts=mlp.experts, top=mlp.top, activation="clipped",
            numbers=(mlp.limit, SHARPNESS), score="softmax_chosen", router_bias=True, weight_on="output", shared=shared,
            names=matrices + (("expert", "e{}."), ("router", "router"), ("router_bias", "router.b"), ("shared", "shared."))))
    raise ValueError(f"no part for a feed-forward of {type(mlp).__name__}")


def medulorn_model_spec(cfg: MedulornConfig) -> ModelSpec:
    norm = NormSpec("rmsnorm", cfg.width, cfg.norm_eps, params(one_number=True))
    layers = tuple(
        LayerSpec(arrangement="postnorm", hidden=cfg.width, mixer=_mixer(cfg, layer.mixer),
                  feed_forward=_feed_forward(cfg, layer.mlp), mixer_norm=norm, feed_forward_norm=norm, prefix=f"l{i}.",
                  names=(("mixer", "mix."), ("feed_forward", "mlp."), ("mixer_norm", "norm1"), ("feed_forward_norm", "norm2"),
                         ("token_shift", "shift")),
                  params=params(alpha=cfg.alpha, token_shift=True))
        for i, layer in enumerate(cfg.layers))
    return ModelSpec(
        architecture=cfg.architecture, hidden=cfg.width, vocab=cfg.vocab, layers=layers,
        schedule=tuple(ScheduleEntry(layer=i, cache=i) for i in range(len(layers))),
        final_norm=norm, embedding_name="embed", final_norm_name="final.norm", head_name="head",
        max_positions=cfg.max_positions, eos_token_ids=tuple(cfg.eos_token_ids), bos_token_id=cfg.bos_token_id,
        embedding=EmbeddingSpec("lookup", params(scale=cfg.embedding_scale)),
        head=HeadSpec("norm_linear", params(softcap=cfg.logit_softcap)))


register_architecture("Medulorn", MedulornConfig, medulorn_model_spec)
