"""The Miberax decoder as a list of parts.

Every layer is a "prenorm" block whose norms cut a row into groups.  Its mixer is a pair ("side_by_side") whose results
are each normed over the row with a weight of their own before half their sum joins the stream: grouped attention over
chunks of positions ("kv_attention"), and the gated delta rule with one decay a head and a full gate ("gated_delta").
The feed-forward is two matrices around a polynomial of normed powers ("dense_mlp" with "poly_norm"), or experts with
clipped gates that a router chooses out of groups, among them experts that hand on their input, beside one behind a
gate of its own that every token uses ("routed_moe"), or none.  The logits come from the embedding table.  Which layer
has which, and every size and constant, is config.json's.

What is fixed here is what the design fixes: the rotation's pairs (2i, 2i + 1), half the sum of the two mixers, the
unit norm's 1e-6, the sharpness 1.702 of the experts' gates, scores by a softmax over all experts with a correction
where they are chosen, weights divided by their sum.
"""
from __future__ import annotations

from ..config.miberax import DenseConfig, ExpertsConfig, MiberaxConfig, PairConfig
from ..config.registry import register_architecture
from ..config.specs import (FeedForwardSpec, HeadSpec, LayerSpec, MixerSpec, ModelSpec, NormSpec, PositionSpec, ScheduleEntry,
                            params)

SHARPNESS = 1.702       # of the experts' gates: g sigmoid(1.702 g)
UNIT_EPS = 1e-6         # of the delta rule's unit vectors


def _rope(head_dim: int, rot):
    if rot is None:
        return None
    scaling = None if rot.factor is None else ("linear", rot.factor)
    return PositionSpec("rope", params(head_dim=head_dim, rotary_dim=rot.dims, theta=rot.base, scaling=scaling,
                                       pairing="interleaved"))


def _mixer(cfg: MiberaxConfig, m: PairConfig) -> MixerSpec:
    a, d = m.left, m.right
    same = lambda *roles: tuple((r, r) for r in roles)      # noqa: E731
    left = MixerSpec("kv_attention", params(
        hidden=cfg.width, num_heads=a.heads, num_kv_heads=a.kv_heads, key_dim=a.dim, value_dim=a.vdim, scale=a.scale,
        chunk=a.chunk, names=same("q", "k", "v", "o")), position=_rope(a.dim, a.rot))
    right = MixerSpec("gated_delta", params(
        hidden=cfg.width, num_heads=d.heads, num_qk_heads=d.kv_heads, dim=d.dim, vdim=d.vdim, conv=d.conv, unit_eps=UNIT_EPS,
        norm_eps=cfg.norm_eps, names=same("q", "k", "v", "b", "a", "g", "o", "norm", "dt_bias")
        + (("q_conv", "q.conv"), ("k_conv", "k.conv"), ("v_conv", "v.conv"), ("a_log", "A_log"))))
    return MixerSpec("side_by_side", params(
        hidden=cfg.width, left=left, right=right, left_scale=0.5, right_scale=0.5, output_norm_eps=cfg.norm_eps,
        names=(("left", "left."), ("right", "right."), ("left_norm", "left.out"), ("right_norm", "right.out"))))


def _feed_forward(cfg: MiberaxConfig, mlp):
    if mlp is None:
        return None
    if isinstance(mlp, DenseConfig):
        return FeedForwardSpec("dense_mlp", params(hidden=cfg.width, intermediate=mlp.ff, activation="poly_norm", norm_eps=cfg.norm_eps,
                                                   names=(("up", "up"), ("down", "down"), ("activation", "act"))))
    if isinstance(mlp, ExpertsConfig):
        shared = None if mlp.shared is None else (mlp.shared[0], (mlp.shared[1], SHARPNESS))
        return FeedForwardSpec("routed_moe", params(
            hidden=cfg.width, intermediate=mlp.ff, experts=mlp.experts, top=mlp.top, activation="clipped",
            numbers=(mlp.limit, SHARPNESS), score="softmax", correction=True, weight_on="output", renormalize=True,
            weight_scale=mlp.scale, identity=mlp.identity, groups=mlp.groups, shared=shared, shared_gate=shared is not None,
            names=(("gate", "gate"), ("up", "up"), ("down", "down"), ("expert", "e{}."), ("router", "router"),
                   ("correction", "correction"), ("shared", "shared."), ("shared_gate", "shared.sg"))))
    raise ValueError(f"no part for a feed-forward of {type(mlp).__name__}")


def miberax_model_spec(cfg: MiberaxConfig) -> ModelSpec:
    norm = NormSpec("rmsnorm", cfg.width, cfg.norm_eps, params(groups=cfg.norm_groups))
    layers = tuple(
        LayerSpec(arrangement="prenorm", hidden=cfg.width, mixer=_mixer(cfg, layer.mixer),
                  feed_forward=_feed_forward(cfg, layer.mlp), mixer_norm=norm, feed_forward_norm=norm, prefix=f"l{i}.",
                  names=(("mixer", "mix."), ("feed_forward", "mlp."), ("mixer_norm_tensor", "norm1"),
                         ("feed_forward_norm_tensor", "norm2")))
        for i, layer in enumerate(cfg.layers))
    return ModelSpec(
        architecture=cfg.architecture, hidden=cfg.width, vocab=cfg.vocab, layers=layers,
        schedule=tuple(ScheduleEntry(layer=i, cache=i) for i in range(len(layers))),
        final_norm=norm, embedding_name="embed", final_norm_name="final.norm", head_name=None,
        max_positions=cfg.max_positions, eos_token_ids=tuple(cfg.eos_token_ids), bos_token_id=cfg.bos_token_id,
        head=HeadSpec("norm_linear"))


register_architecture("Miberax", MiberaxConfig, miberax_model_spec)
