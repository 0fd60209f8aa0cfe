"""Feed-forwards of many small experts, of which every token uses `top`.

"table_moe": no router.  A table [vocabulary, top] of integers gives every token id its experts (the
entries of a row differ); each counts 1 / top.  Expert: down(act(gate(h)) * up(h)), act the SiLU, no
biases; the output is the weighted sum of the chosen experts' outputs, added to the residual stream in
float32.  The experts' matrices are stacked [experts, rows, columns] when they are bound; the lookup
runs on the device from the step's token ids, so a step may be replayed from a recorded graph.  A step
with more (token, expert) pairs than experts groups the pairs by expert on the device and multiplies them
in tiles on the matrix cores (bfloat16, sizes that are multiples of 32); a step of few tokens, and
float32, reads each token's experts row by row.

"routed_moe": a router chooses.  z = W_router h in float32; scores s = sigmoid(z); the `top` experts with
the largest scores are a token's, and their weights are those scores as they are (not renormalized).
Expert: down(relu(up(w h))^2), no gate and no biases: the weight w multiplies the expert's input (it joins
the up product's float32 sum, which is the same product).  The output is the sum of the chosen experts'
outputs.  It writes float32 rows (`forward_into`) for a block that norms them, or adds them to the stream.
Steps of many tokens go through the same grouped kernels as above, few tokens and float32 row by row.
Its parameters make other routed experts of it: `score` "softmax" takes the softmax of z over all experts as
the scores; `correction` adds a learned number an expert to the scores where the experts are chosen, and only
there; `activation` "silu" gives the experts a gate, down(silu(gate(h)) * up(h)); `weight_on` "output"
multiplies an expert's output by its weight instead of its input.  `score` "softmax_chosen" takes the softmax over the chosen
logits only; `router_bias` adds a learned number an expert to the logits; `activation` "clipped" with its
`numbers` (limit, sharpness) is the gate that clips both of its sides (`ops.GATE_ACTIVATIONS`); `shared` = (ff, numbers)
stands an expert beside them (the same form, its own size and numbers, tensors under the name `shared`) that
every token uses with weight one, or with `shared_gate` with sigmoid(W_sg h), one number a token.  `groups` = (count, keep):
the router's outputs form `count` equal groups of neighbours, a token's experts come from the `keep` groups with the
largest best choice scores.  `renormalize` divides the chosen scores by their sum (+ 1e-20), `weight_scale` multiplies
them then.  `identity` = I: the router has I more outputs behind the experts', which stand for experts without matrices
that hand on their input.  Where experts may hand on their input or the shared one has a gate, the experts' outputs,
those inputs, the shared expert, the addition to the stream and the norm that follows meet in one launch
(`ops.experts_join`).
"""
from __future__ import annotations

import torch

from ..config.specs import FeedForwardSpec, params
from ..kernels import ops
from ..weights.spec import TensorSpec
from .base import FeedForward, LazyNorm, register_feed_forward
from .mlp import GatedMLP


@register_feed_forward("table_moe")
class TableMoE(FeedForward):
    graph_safe = True

    def __init__(self, spec: FeedForwardSpec, prefix: str, dtype: torch.dtype):
        self.prefix, self.dtype = prefix, dtype
        self.hidden = spec.get("hidden")
        self.intermediate = spec.get("intermediate")
        self.experts, self.top = spec.get("experts"), spec.get("top")
        self.vocab = spec.get("vocab")
        if spec.get("activation", "silu") != "silu":
            raise ValueError("the experts' activation is the SiLU")
        if not 1 <= self.top <= self.experts:
            raise ValueError(f"a token uses 1 to {self.experts} experts, not {self.top}")
        given = dict(spec.get("names") or ())
        self.expert_names = given.get("expert", "experts.{}.")           # a format for the expert's number
        self.roles = {r: given.get(r, d) for r, d in dict(gate="gate_proj.weight", up="up_proj.weight",
                                                         down="down_proj.weight", table="table").items()}

    def _name(self, e: int, role: str) -> str:
        return self.prefix + self.expert_names.format(e) + self.roles[role]

    def tensor_specs(self):
        specs = []
        for e in range(self.experts):
            specs += [TensorSpec(self._name(e, "gate"), (self.intermediate, self.hidden)),
                      TensorSpec(self._name(e, "up"), (self.intermediate, self.hidden)),
                      TensorSpec(self._name(e, "down"), (self.hidden, self.intermediate))]
        specs.append(TensorSpec(self.prefix + self.roles["table"], (self.vocab, self.top), role="table",
                                init=("distinct_in_row", self.experts)))
        return specs

    def bind(self, tensors):
        E = range(self.experts)
        self.w_gate = torch.stack([tensors.pop(self._name(e, "gate")) for e in E]).contiguous()
        self.w_up = torch.stack([tensors.pop(self._name(e, "up")) for e in E]).contiguous()
        self.w_down = torch.stack([tensors.pop(self._name(e, "down")) for e in E]).contiguous()
        self.table = tensors.pop(self.prefix + self.roles["table"]).contiguous()
        lo, hi = int(self.table.min()), int(self.table.max())
        if lo < 0 or hi >= self.experts:
            raise ValueError(f"{self.prefix + self.roles['table']} names experts {lo}..{hi}, the layer has {self.experts}")

    def forward_add(self, ctx, x, h):
        hn = h.tensor() if isinstance(h, LazyNorm) else h
        n, top = ctx.n, self.top
        # more pairs than experts: grouped by expert, an expert's matrices are read once for all its tokens
        if n * top > self.experts and ops.moe_grouped_fits(self.dtype, self.hidden, self.intermediate) \
                and hn.data_ptr() % 16 == 0 and hn.stride(0) % 8 == 0:
            ws = ctx.workspace
            order = ws.flat("table_moe.order", ws.capacity * top, torch.int32)
            tiles = ws.flat("table_moe.tiles", 3 * ops.moe_group_tiles(ws.capacity, top, self.experts) + 1, torch.int32)
            act = ctx.rows("table_moe.act", top * self.intermediate)
            y = ctx.rows("table_moe.rows", top * self.hidden, torch.float32) if top > 1 else None
            ops.moe_grouped(x, hn, self.w_gate, self.w_up, self.w_down, top, order, tiles, act, y, weight=1.0 / top,
                            table=self.table, token_ids=ctx.token_ids)
            return
        act = ctx.rows("table_moe.act", self.top * self.intermediate).view(ctx.n * self.top, self.intermediate)
        ops.moe_up(act, hn, self.w_gate, self.w_up, self.top, table=self.table, token_ids=ctx.token_ids)
        ops.moe_down(x, act, self.w_down, self.top, weight=1.0 / self.top, table=self.table, token_ids=ctx.token_ids)


@register_feed_forward("routed_moe")
class RoutedMoE(FeedForward):
    """Tensor names by role: router ([experts + identity, hidden]), router_bias, correction ([experts + identity]); expert
    (a format for the expert's number), shared (a prefix), shared_gate ([1, hidden]), gate, up, down."""
    graph_safe = True

    def __init__(self, spec: FeedForwardSpec, prefix: str, dtype: torch.dtype):
        self.prefix, self.dtype = prefix, dtype
        self.hidden = spec.get("hidden")
        self.intermediate = spec.get("intermediate")
        self.experts, self.top = spec.get("experts"), spec.get("top")
        self.activation, self.score = spec.get("activation", "relu2"), spec.get("score", "sigmoid")
        self.weight_on = spec.get("weight_on", "input")
        self.has_correction = bool(spec.get("correction", False))
        self.has_router_bias = bool(spec.get("router_bias", False))
        if self.activation not in ("relu2", "silu", "clipped") or self.score not in ops.ROUTER_SCORES:
            raise ValueError("the routed experts' activation is 'relu2' (no gate), 'silu' or 'clipped' (gated), their scores "
                             f"one of {sorted(ops.ROUTER_SCORES)}")
        self.gated = self.activation != "relu2"
        self.gate = dict(activation=self.activation, numbers=spec.get("numbers")) if self.gated else {}
        if self.gated:
            ops.gate_numbers(**self.gate)
        self.identity, self.groups = int(spec.get("identity", 0) or 0), spec.get("groups")
        self.outputs = self.experts + self.identity            # of the router
        self.renormalize, self.weight_scale = bool(spec.get("renormalize", False)), float(spec.get("weight_scale", 1.0))
        if self.weight_on != ("output" if self.gated else "input"):
            raise ValueError("the weights multiply the inputs of experts without a gate and the outputs of gated ones")
        if self.renormalize and self.score == "softmax_chosen":
            raise ValueError("a softmax over the chosen experts is normalized already")
        if self.weight_scale != 1.0 and not self.renormalize:
            raise ValueError("weight_scale multiplies renormalized weights")
        if self.groups is not None:
            count, keep = self.groups
            if not 1 <= keep <= count or self.outputs % count or keep * (self.outputs // count) < self.top:
                raise ValueError(f"{self.outputs} router outputs in {count} equal groups of which {keep} are kept cannot give "
                                 f"a token {self.top} experts")
        if self.identity and not self.gated:
            raise ValueError("experts that hand on their input stand beside gated ones")
        if self.has_correction and self.score == "softmax_chosen":
            raise ValueError("a softmax over the chosen experts takes no correction")
        if not 1 <= self.top <= self.outputs:
            raise ValueError(f"a token uses 1 to {self.outputs} experts, not {self.top}")
        given = dict(spec.get("names") or ())
        self.expert_names = given.get("expert", "experts.{}.")
        self.roles = {r: given.get(r, d) for r, d in dict(gate="gate_proj.weight", up="up_proj.weight", down="down_proj.weight",
                                                         router="router.weight", router_bias="router.bias",
                                                         correction="router.correction", shared="shared_expert.",
                                                         shared_gate="shared_expert_gate.weight").items()}
        self.output_bias = None
        self.correction = self.router_bias = None
        self.shared = None
        if spec.get("shared") is not None:
            if not self.gated:
                raise ValueError("an expert that every token uses is a gated one")
            ff, numbers = spec.get("shared")
            self.shared = GatedMLP(FeedForwardSpec("gated_mlp", params(
                hidden=self.hidden, intermediate=ff, activation=self.activation, numbers=numbers,
                names=tuple((r, self.roles[r]) for r in ("gate", "up", "down")))), prefix + self.roles["shared"], dtype)

        self.has_shared_gate = bool(spec.get("shared_gate", False))
        if self.has_shared_gate and self.shared is None:
            raise ValueError("shared_gate is the gate of an expert that every token uses")
        self.emits_norm = self.joins = bool(self.identity or self.has_shared_gate)      # (that launch holds whole rows)

    def _name(self, e: int, role: str) -> str:
        return self.prefix + self.expert_names.format(e) + self.roles[role]

    def tensor_specs(self):
        specs = []
        for e in range(self.experts):
            if self.gated:
                specs.append(TensorSpec(self._name(e, "gate"), (self.intermediate, self.hidden)))
            specs += [TensorSpec(self._name(e, "up"), (self.intermediate, self.hidden)),
                      TensorSpec(self._name(e, "down"), (self.hidden, self.intermediate))]
        specs.append(TensorSpec(self.prefix + self.roles["router"], (self.outputs, self.hidden)))
        if self.has_correction:
            specs.append(TensorSpec(self.prefix + self.roles["correction"], (self.outputs,), role="vector"))
        if self.has_router_bias:
            specs.append(TensorSpec(self.prefix + self.roles["router_bias"], (self.outputs,), role="vector"))
        if self.shared is not None:
            specs += self.shared.tensor_specs()
        if self.has_shared_gate:
            specs.append(TensorSpec(self.prefix + self.roles["shared_gate"], (1, self.hidden)))
        return specs

    def bind(self, tensors):
        E = range(self.experts)
        self.w_gate = torch.stack([tensors.pop(self._name(e, "gate")) for e in E]).contiguous() if self.gated else None
        self.w_up = torch.stack([tensors.pop(self._name(e, "up")) for e in E]).contiguous()
        self.w_down = torch.stack([tensors.pop(self._name(e, "down")) for e in E]).contiguous()
        self.w_router = tensors.pop(self.prefix + self.roles["router"]).contiguous()
        if self.has_shared_gate:        # (one more row of the router's product)
            self.w_router = torch.cat([self.w_router, tensors.pop(self.prefix + self.roles["shared_gate"])], dim=0).contiguous()
        if self.has_correction:
            self.correction = tensors.pop(self.prefix + self.roles["correction"]).to(torch.float32).contiguous()
        if self.has_router_bias:
            self.router_bias = tensors.pop(self.prefix + self.roles["router_bias"]).to(torch.float32).contiguous()
        if self.shared is not None:
            self.shared.bind(tensors)

    def _choose(self, ctx, hn):
        """(chosen, weights, the shared expert's gate before its sigmoid or None)."""
        n, top = ctx.n, self.top
        made = ctx.rows("routed_moe.logits", self.w_router.shape[0], torch.float32)
        ops.linear(made, hn, self.w_router)
        logits = made[:, :self.outputs]
        ws = ctx.workspace
        chosen = ws.flat("routed_moe.chosen", ws.capacity * top, torch.int32)[:n * top].view(n, top)
        weights = ws.flat("routed_moe.weights", ws.capacity * top, torch.float32)[:n * top].view(n, top)
        ops.router_topk(chosen, weights, logits, top, score=self.score, correction=self.correction, bias=self.router_bias,
                        groups=self.groups, renormalize=self.renormalize, scale=self.weight_scale)
        return chosen, weights, made[:, self.outputs] if self.has_shared_gate else None

    def _grouped(self, n, hn) -> bool:
        return (n * self.top > self.experts and ops.moe_grouped_fits(self.dtype, self.hidden, self.intermediate)
                and hn.data_ptr() % 16 == 0 and hn.stride(0) % 8 == 0)

    def _join(self, ctx, x, h, then):
        """x += everything the experts make of h, and the norm that follows."""
        hn = h.tensor() if isinstance(h, LazyNorm) else h
        n, top, ws = ctx.n, self.top, ctx.workspace
        shared = None
        if self.shared is not None:
            shared = ctx.rows("routed_moe.shared", self.hidden, torch.float32)
            self.shared.forward_into(ctx, shared, hn)
        chosen, weights, gate = self._choose(ctx, hn)
        grouped = self._grouped(n, hn)
        if grouped:
            order = ws.flat("table_moe.order", ws.capacity * top, torch.int32)
            tiles = ws.flat("table_moe.tiles", 3 * ops.moe_group_tiles(ws.capacity, top, self.experts) + 1, torch.int32)
            act = ctx.rows("table_moe.act", top * self.intermediate)
            y = ctx.rows("table_moe.rows", top * self.hidden, torch.float32).view(n * top, self.hidden)
            ops.moe_grouped(None, hn, self.w_gate, self.w_up, self.w_down, top, order, tiles, act, y, chosen=chosen, **self.gate)
        else:
            act = ctx.rows("table_moe.act", top * self.intermediate).view(n * top, self.intermediate)
            ops.moe_up(act, hn, self.w_gate, self.w_up, top, chosen=chosen, **self.gate)
            y = ctx.rows("routed_moe.summed", self.hidden, torch.float32)
            ops.moe_down(y, act, self.w_down, top, pair_weights=weights, chosen=chosen, accumulate=False)
        ops.experts_join(x, y, chosen, weights, self.experts, hn, summed=not grouped, shared=shared, gate=gate,
                         **(then.offer_rows() if then is not None else {}))

    def _run(self, ctx, out, h, add: bool):
        if self.joins:
            if not add:
                out.zero_()
            return self._join(ctx, out, h, None)
        hn = h.tensor() if isinstance(h, LazyNorm) else h
        n, top = ctx.n, self.top
        if self.shared is not None:         # (its last product fills the rows, or adds to them; the experts' sum joins)
            self.shared._run(ctx, out, hn, None, add=add)
            add = True
        chosen, weights, _ = self._choose(ctx, hn)
        # (gated experts: the weight meets the output; experts without a gate: the input)
        on_input = None if self.gated else weights
        on_output = weights if self.gated else None
        if self._grouped(n, hn):
            ws = ctx.workspace
            order = ws.flat("table_moe.order", ws.capacity * top, torch.int32)
            tiles = ws.flat("table_moe.tiles", 3 * ops.moe_group_tiles(ws.capacity, top, self.experts) + 1, torch.int32)
            act = ctx.rows("table_moe.act", top * self.intermediate)
            y = ctx.rows("table_moe.rows", top * self.hidden, torch.float32) if top > 1 else None
            if not add:
                out.zero_()
            ops.moe_grouped(out, hn, self.w_gate, self.w_up, self.w_down, top, order, tiles, act, y, weight=1.0, chosen=chosen,
                            in_weights=on_input, pair_weights=on_output, **self.gate)
            return
        act = ctx.rows("table_moe.act", top * self.intermediate).view(n * top, self.intermediate)
        ops.moe_up(act, hn, self.w_gate, self.w_up, top, chosen=chosen, in_weights=on_input, **self.gate)
        ops.moe_down(out, act, self.w_down, top, weight=1.0, pair_weights=on_output, chosen=chosen, accumulate=add)

    def forward_into(self, ctx, out, h):
        self._run(ctx, out, h, add=False)

    def forward_add(self, ctx, x, h, then=None):
        if self.joins:
            self._join(ctx, x, h, then)
        else:
            self._run(ctx, x, h, add=True)
