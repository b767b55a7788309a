"""Feed-forward parts.  A feed-forward adds its output into the residual stream."""

from __future__ import annotations

from typing import Dict, Optional

import torch

from ..ops import kernels, residual
from ..ops.linear import LazyNorm, as_tensor, linear, linear_add, linear_xielu, packed_weight, plain_residual
from .base import MATRIX, Part, StepContext, TABLE, VECTOR, WeightRequest, register_feed_forward

# activations of the dense feed-forward: an epilogue of the product kernels, or (None) one that brings coefficients
# (ops.linear.linear_xielu: the tiled kernel's epilogue, elsewhere a kernel of its own behind the product)
_ACTIVATIONS = {"gelu_tanh": kernels.EPI_GELU, "relu2": kernels.EPI_RELU2, "xielu": None}
# activations of experts without a gate: epilogues of the grouped products as well
_EXPERT_ACTIVATIONS = {"relu2": kernels.EPI_RELU2}


class FeedForward(Part):
    category = "feed_forward"

    def forward_add(self, ctx: StepContext, h: torch.Tensor, x: torch.Tensor) -> None:
        """x[:n_rows] += ff(h[:n_rows]); h is a tensor or an ops.linear.LazyNorm (see Mixer.forward_add)."""
        raise NotImplementedError


@register_feed_forward("dense_mlp")
class DenseMLP(FeedForward):
    """u = h Wfc^T (+ b); g = 0.5 u (1 + tanh(sqrt(2/pi)(u + 0.044715 u^3))); m = g Wproj^T (+ b)
    (reference: src/minigpt_infer/model.py:96-101; there the hidden size is 4*n_embd, here it is
    a parameter).  With activation "xielu" g is instead, from two stored numbers (p, q) (the tensor `act`),
    softplus(p) u^2 + u / 2 for u > 0 and (1/2 + softplus(q)) (exp(u) - 1 - u) + u / 2 for u <= 0; with "relu2"
    it is max(u, 0)^2."""

    graph_safe = True

    plan_safe = True
    takes_pending_residual = True

    def __init__(self, width: int, hidden: int, bias: bool, activation: str = "gelu_tanh") -> None:
        if activation not in _ACTIVATIONS:
            raise ValueError(f"activation {activation!r} has no kernel epilogue; known: {sorted(_ACTIVATIONS)}")
        self.width, self.hidden, self.has_bias = int(width), int(hidden), bool(bias)
        self.activation = activation
        self.fc_weight = self.fc_bias = self.proj_weight = self.proj_bias = None

    def weight_requests(self) -> Dict[str, WeightRequest]:
        req = {"fc_weight": WeightRequest((self.hidden, self.width), MATRIX),
               "proj_weight": WeightRequest((self.width, self.hidden), MATRIX)}
        if self.has_bias:
            req["fc_bias"] = WeightRequest((self.hidden,), VECTOR)
            req["proj_bias"] = WeightRequest((self.width,), VECTOR)
        if self.activation == "xielu":
            req["act"] = WeightRequest((2,), VECTOR)
        return req

    def bind(self, tensors):
        super().bind(tensors)
        if self.activation == "xielu":
            # the two branches' coefficients, made once: softplus(p) and 1/2 + softplus(q)
            sp = torch.nn.functional.softplus(tensors["act"].to(torch.float32))
            self.act_coef = torch.stack([sp[0], sp[1] + 0.5]).contiguous()
        return None

    def _forward_add_fused(self, ctx: StepContext, h, x: torch.Tensor) -> bool:
        """A decode-only step of few rows: one kernel from the residual (a sum, as the kernels
        before left it) through LayerNorm, both products and the activation to this part's addition
        to the residual, left as one partial sum per 64 hidden units.  False, with nothing launched,
        where that kernel does not apply."""
        parts_n = kernels.fused_mlp_parts(self.hidden)
        if not (isinstance(h, LazyNorm) and h._tensor is None and h.rows is None and h.x is x
                and getattr(h.norm, "fusable_layer_norm", False) and parts_n and residual.usable(ctx, self.width, parts_n)
                and self.activation == "gelu_tanh" and self.fc_weight.dtype == torch.bfloat16
                and self.proj_weight.dtype == torch.bfloat16):
            return False
        wfc, wproj = packed_weight(self.fc_weight, ctx), packed_weight(self.proj_weight, ctx)
        if wfc is None or wproj is None:
            return False
        n = ctx.n_rows
        if ctx.pending is not None and ctx.pending.base is None:
            residual.settle(ctx, x, n)      # table rows: this kernel reads residual rows only
        pending, settled = residual.take(ctx, x)
        parts = residual.parts_buffer(ctx, "feed_forward_parts", parts_n, n, self.width)
        if not kernels.fused_mlp_decode(pending, settled, h.norm.weight, h.norm.bias, h.norm.eps, wfc, self.fc_bias,
                                        wproj, self.proj_bias, parts, n, self.hidden):
            return False
        ctx.pending = residual.PendingSums(settled, parts, parts_n)
        return True

    def forward_add(self, ctx: StepContext, h: torch.Tensor, x: torch.Tensor) -> None:
        if self._forward_add_fused(ctx, h, x):
            return
        plain_residual(ctx, h, x)
        n = ctx.n_rows
        u = ctx.workspace.get("ff_hidden", n, self.hidden, ctx.dtype)
        if self.activation == "xielu":
            linear_xielu(ctx, h, self.fc_weight, self.fc_bias, u, n, self.act_coef)
        else:
            linear(ctx, h, self.fc_weight, self.fc_bias, u, n, _ACTIVATIONS[self.activation])
        # (a caller that hands over a LazyNorm of x itself knows that x may be left as a sum)
        linear_add(ctx, u, self.proj_weight, self.proj_bias, x, n,
                   may_leave_parts=isinstance(h, LazyNorm) and h.x is x)


def _gated(ctx: StepContext, h, in_weight: torch.Tensor, down_weight: torch.Tensor, x: torch.Tensor, n: int,
           hidden: int, **unit) -> None:
    """x += (act(h Wgate^T) * (h Wup^T)) Wdown^T with the gate and up matrices stacked in in_weight; `unit`: the
    activation and its constants, as ops.kernels.gated_unit takes them."""
    act = ctx.workspace.get("gated_act", n, hidden, ctx.dtype)
    few = not ctx.exact and n <= kernels.GATED_FEW_ROWS and kernels.gated_few_rows(as_tensor(ctx, h), in_weight, act, n, hidden, **unit)
    if not few:
        z = ctx.workspace.get("gated_z", n, 2 * hidden, ctx.dtype)
        linear(ctx, h, in_weight, None, z, n)
        kernels.gated_unit(z, act, n, hidden, fast=not ctx.exact, **unit)
    linear_add(ctx, act, down_weight, None, x, n)


def _unit_options(activation: str, limit: Optional[float], sharpness: float) -> Dict[str, object]:
    """The gated unit's activation and constants as ops.kernels.gated_unit takes them."""
    if activation not in kernels.GATE_ACTIVATIONS:
        raise ValueError(f"gated unit: activation {activation!r} is none of {sorted(kernels.GATE_ACTIVATIONS)}")
    if activation != "clamped_swish":
        return {"activation": activation}
    if limit is None or not float(limit) > 0.0:
        raise ValueError(f"gated unit: a clamped swish needs a positive limit, got {limit!r}")
    return {"activation": activation, "limit": float(limit), "sharpness": float(sharpness)}


def _stack_gate_up(part: Part, tensors, gate: str, up: str):
    """One matrix [2 * hidden, width] from a gate and an up matrix; the two names become views of it."""
    joint = torch.cat([tensors[gate], tensors[up]], dim=0).contiguous()
    hidden = tensors[gate].shape[0]
    views = {gate: joint[:hidden], up: joint[hidden:]}
    for name, view in views.items():
        setattr(part, name, view)
    return joint, views


@register_feed_forward("gated_mlp")
class GatedMLP(FeedForward):
    """m = (act(h Wgate^T) * (h Wup^T)) Wdown^T, no biases; act is silu(v) = v sigmoid(v) unless
    `activation` names relu or gelu_tanh; the unit's nonlinearity and product in float32.  "clamped_swish" (with
    `limit` and `sharpness`) is the unit g sigmoid(sharpness g) (u + 1), g = min(h Wgate^T, limit), u = h Wup^T held within
    -limit .. limit."""

    graph_safe = True
    plan_safe = True

    def __init__(self, width: int, hidden: int, activation: str = "silu", limit: Optional[float] = None,
                 sharpness: float = 1.0) -> None:
        self.width, self.hidden = int(width), int(hidden)
        self.unit = _unit_options(activation, limit, sharpness)
        self.activation = activation
        self.in_weight = None

    def weight_requests(self) -> Dict[str, WeightRequest]:
        return {"gate_weight": WeightRequest((self.hidden, self.width), MATRIX),
                "up_weight": WeightRequest((self.hidden, self.width), MATRIX),
                "down_weight": WeightRequest((self.width, self.hidden), MATRIX)}

    def bind(self, tensors):
        super().bind(tensors)
        self.in_weight, views = _stack_gate_up(self, tensors, "gate_weight", "up_weight")
        return views

    def forward_add(self, ctx: StepContext, h, x: torch.Tensor) -> None:
        plain_residual(ctx, h, x)
        _gated(ctx, h, self.in_weight, self.down_weight, x, ctx.n_rows, self.hidden, **self.unit)


@register_feed_forward("table_experts")
class TableExperts(FeedForward):
    """A mixture of gated feed-forwards without a router: row id_t of an integer table [vocab, top]
    names the experts of token t, each weighted 1 / top; a shared expert (shared_hidden > 0) takes
    every token and is added.

    The (token, choice) pairs are sorted by expert on the device, every expert multiplies its run
    of pairs by its own matrices (csrc/hip/experts.hip), and the pairs' outputs are added up per
    token in the order of the table's columns."""

    graph_safe = True
    plan_safe = True

    def __init__(self, width: int, hidden: int, n_experts: int, top: int, vocab_size: int,
                 shared_hidden: int = 0) -> None:
        self.width, self.hidden, self.n_experts, self.top = int(width), int(hidden), int(n_experts), int(top)
        self.vocab_size, self.shared_hidden = int(vocab_size), int(shared_hidden)
        if not 0 < self.top <= self.n_experts <= kernels.MAX_EXPERTS:
            raise ValueError(f"top {self.top} of {self.n_experts} experts: need 0 < top <= experts <= {kernels.MAX_EXPERTS}")
        # an expert is a gated unit; without the gate (a subclass says so) it is down(act(up h)) with this activation
        self.gated, self.epilogue = True, kernels.EPI_NONE
        self.unit = self.shared_unit = {"activation": "silu"}     # the gated unit of the experts, and of the shared one
        self.gates_shared = False       # the shared expert's output is multiplied by a number per token
        self.in_weights = self.down_weights = self.shared_in_weight = None

    def weight_requests(self) -> Dict[str, WeightRequest]:
        req = {"table": WeightRequest((self.vocab_size, self.top), TABLE)}
        for e in range(self.n_experts):
            if self.gated:
                req[f"e{e}_gate"] = WeightRequest((self.hidden, self.width), MATRIX)
            req[f"e{e}_up"] = WeightRequest((self.hidden, self.width), MATRIX)
            req[f"e{e}_down"] = WeightRequest((self.width, self.hidden), MATRIX)
        if self.shared_hidden:
            if self.gated:
                req["shared_gate"] = WeightRequest((self.shared_hidden, self.width), MATRIX)
            req["shared_up"] = WeightRequest((self.shared_hidden, self.width), MATRIX)
            req["shared_down"] = WeightRequest((self.width, self.shared_hidden), MATRIX)
        return req

    def bind(self, tensors):
        self.table = tensors["table"]
        if self.table.dtype != torch.int32:
            raise ValueError("the experts' table must hold integers")
        return self._bind_experts(tensors)

    def _bind_experts(self, tensors):
        f, views = self.hidden, {}
        # [experts, 2 * hidden, width] (without gates [experts, hidden, width]) and [experts, width, hidden]: an
        # expert's matrices lie together
        if self.gated:
            self.in_weights = torch.stack([torch.cat([tensors[f"e{e}_gate"], tensors[f"e{e}_up"]], dim=0)
                                           for e in range(self.n_experts)]).contiguous()
        else:
            self.in_weights = torch.stack([tensors[f"e{e}_up"] for e in range(self.n_experts)]).contiguous()
        self.down_weights = torch.stack([tensors[f"e{e}_down"] for e in range(self.n_experts)]).contiguous()
        for e in range(self.n_experts):
            if self.gated:
                views[f"e{e}_gate"], views[f"e{e}_up"] = self.in_weights[e, :f], self.in_weights[e, f:]
            else:
                views[f"e{e}_up"] = self.in_weights[e]
            views[f"e{e}_down"] = self.down_weights[e]
        if self.shared_hidden:
            self.shared_down = tensors["shared_down"]
            if self.gated:
                self.shared_in_weight, shared = _stack_gate_up(self, tensors, "shared_gate", "shared_up")
                views.update(shared)
            else:
                self.shared_in_weight = tensors["shared_up"]
        return views

    def token_matrix_elements(self) -> int:
        """Matrix elements one token goes through: its `top` experts and the shared one."""
        return (3 if self.gated else 2) * self.width * (self.top * self.hidden + self.shared_hidden)

    def forward_add(self, ctx: StepContext, h, x: torch.Tensor) -> None:
        plain_residual(ctx, h, x)
        hn = as_tensor(ctx, h)
        self._experts_add(ctx, hn, x, ctx.n_rows, ctx.token_ids, self.table, None, 1.0 / self.top)

    def _experts_add(self, ctx: StepContext, hn: torch.Tensor, x: torch.Tensor, n: int, ids, table: torch.Tensor,
                     pair_weight, combine_weight: float, out_weight=None, shared_gate=None, routed=None) -> None:
        """x += combine_weight * sum over token n's experts (row ids[n] of the table, or row n without ids) of
        v expert(w h), w = pair_weight[n][choice] and v = out_weight[n][choice] (None: 1), plus the shared expert
        (times shared_gate[n]).  routed: the slots of _slots, if the pairs are sorted already."""
        ws = ctx.workspace
        fast = not ctx.exact and ctx.dtype == torch.bfloat16
        if routed is None and fast and n * self.top >= self.TILED_FROM_PAIRS and self.width % 16 == 0 and self.hidden % 16 == 0 \
                and self._forward_tiled(ctx, hn, x, n, ids, table, pair_weight, combine_weight, out_weight, shared_gate):
            return
        slot_token, slot_pair, tile_expert, slots, tile = routed or self._slots(ctx, n)
        if routed is None:
            kernels.expert_route(ids, ctx.q_req, table, n, self.n_experts, slot_token, slot_pair, tile_expert, tile)
        act = ws.get("expert_act", slots, self.hidden, ctx.dtype)
        rows, places = hn, slot_token
        if pair_weight is not None:
            # the weight multiplies the expert's input: every pair's row is made first, scaled, in the experts' order
            rows, places = ws.get("expert_rows", slots, self.width, ctx.dtype), None
            kernels.gather_scale_rows(hn, slot_token, slot_pair, pair_weight, rows, slots)
        # few pairs an expert: the unit is made where the gate's and the up product's sums meet
        done = (self.gated and fast and tile == 16
                and kernels.gated_few_rows(rows, self.in_weights, act, 0, self.hidden, a_rows=places, tile_expert=tile_expert,
                                           slot_token=slot_token, n_slots=slots, **self.unit))
        if not done:
            z = ws.get("expert_z", slots, 2 * self.hidden, ctx.dtype) if self.gated else act
            kernels.grouped_linear(rows, places, self.in_weights, tile_expert, slot_token, z, None, slots, tile, fast, self.epilogue)
        if self.gated and not done:
            kernels.gated_unit(z, act, slots, self.hidden, fast=not ctx.exact, **self.unit)
        pair_out = ws.get("expert_pair_out", n * self.top, self.width, torch.float32)
        kernels.grouped_linear(act, None, self.down_weights, tile_expert, slot_token, pair_out, slot_pair, slots,
                               tile, fast)
        extra = self._shared_add(ctx, hn, x, n)
        kernels.expert_combine(pair_out, x, n, self.top, combine_weight, q_req=ctx.q_req, pair_weight=out_weight,
                               extra=extra, extra_gate=shared_gate)

    def _slots(self, ctx: StepContext, n: int):
        """Buffers for the sorted pairs of n tokens: (slot_token, slot_pair, tile_expert, slots, slots a tile)."""
        # tiles of 64 slots for the MFMA kernel of few rows, of 16 for the general one, and for the MFMA kernels too
        # where an expert gets 16 pairs at most on average (a decode step): a tile's empty slots are loaded and
        # multiplied like the used ones
        ws = ctx.workspace
        fast = not ctx.exact and ctx.dtype == torch.bfloat16
        tile = 64 if fast and n * self.top > 16 * self.n_experts else 16
        slots = kernels.expert_slots(n, self.top, self.n_experts, tile)
        return (ws.get("expert_slot_token", slots, 1, torch.int32).view(-1), ws.get("expert_slot_pair", slots, 1, torch.int32).view(-1),
                ws.get("expert_tile", slots // tile, 1, torch.int32).view(-1), slots, tile)

    def _shared_add(self, ctx: StepContext, hn: torch.Tensor, x: torch.Tensor, n: int):
        """The shared expert: added into x (returns None), or, if a number per token multiplies it, as rows of its own
        that the kernel which adds up the experts' outputs takes along."""
        if not self.shared_hidden:
            return None
        if self.gated and not self.gates_shared:
            _gated(ctx, hn, self.shared_in_weight, self.shared_down, x, n, self.shared_hidden, **self.shared_unit)
            return None
        act = ctx.workspace.get("shared_act", n, self.shared_hidden, ctx.dtype)
        if self.gated:
            z = ctx.workspace.get("shared_z", n, 2 * self.shared_hidden, ctx.dtype)
            linear(ctx, hn, self.shared_in_weight, None, z, n)
            kernels.gated_unit(z, act, n, self.shared_hidden, fast=not ctx.exact, **self.shared_unit)
        else:
            linear(ctx, hn, self.shared_in_weight, None, act, n, self.epilogue)
        if not self.gates_shared:
            linear_add(ctx, act, self.shared_down, None, x, n)
            return None
        rows = ctx.workspace.get("shared_out", n, self.width, torch.float32)
        linear(ctx, act, self.shared_down, None, rows, n)
        return rows

    # From this many (token, choice) pairs on, the experts' products go through the tiled MFMA kernel
    # of the dense layers: the pairs' rows are copied into the experts' order first, every expert's
    # run padded to whole tiles of 256 slots, so that a tile of that kernel multiplies one expert's
    # matrix.  Below it a step is a decode step or a short portion, and padding every expert to 256
    # rows would be most of the work.
    TILED_FROM_PAIRS = 512

    def _forward_tiled(self, ctx: StepContext, hn: torch.Tensor, x: torch.Tensor, n: int, ids, table: torch.Tensor,
                       pair_weight, combine_weight: float, out_weight=None, shared_gate=None) -> bool:
        ws, tile = ctx.workspace, 256
        slots = kernels.expert_slots(n, self.top, self.n_experts, tile)
        slot_token = ws.get("expert_slot_token", slots, 1, torch.int32).view(-1)
        slot_pair = ws.get("expert_slot_pair", slots, 1, torch.int32).view(-1)
        pair_slot = ws.get("expert_pair_slot", n * self.top, 1, torch.int32).view(-1)
        tile_expert = ws.get("expert_tile", slots // tile, 1, torch.int32).view(-1)
        sorted_rows = ws.get("expert_rows", slots, self.width, ctx.dtype)
        if hn.stride(0) % 8 or hn.data_ptr() % 16 or sorted_rows.data_ptr() % 16 or self.width % 8:
            return False
        kernels.expert_route(ids, ctx.q_req, table, n, self.n_experts, slot_token, slot_pair,
                             tile_expert, tile, pair_slot=pair_slot)
        if pair_weight is not None:
            kernels.gather_scale_rows(hn, slot_token, slot_pair, pair_weight, sorted_rows, slots)
        elif not kernels.gather_rows(hn, slot_token, sorted_rows, slots):
            return False
        act = ws.get("expert_act", slots, self.hidden, ctx.dtype)
        z = ws.get("expert_z", slots, 2 * self.hidden, ctx.dtype) if self.gated else act
        if not kernels.grouped_linear_tiled(sorted_rows, self.in_weights, tile_expert, slot_token, z, slots, self.epilogue):
            return False
        if self.gated:
            kernels.gated_unit(z, act, slots, self.hidden, fast=True, **self.unit)
        slot_out = ws.get("expert_slot_out", slots, self.width, torch.float32)
        if not kernels.grouped_linear_tiled(act, self.down_weights, tile_expert, slot_token, slot_out, slots):
            return False
        extra = self._shared_add(ctx, hn, x, n)
        kernels.expert_combine(slot_out, x, n, self.top, combine_weight, pair_slot=pair_slot, q_req=ctx.q_req,
                               pair_weight=out_weight, extra=extra, extra_gate=shared_gate)
        return True


@register_feed_forward("routed_experts")
class RoutedExperts(TableExperts):
    """A mixture of feed-forwards chosen by a router: scores s = sigmoid(h Wr^T), computed in
    float32; a token uses the `top` experts with the largest scores; the output is the sum over them of
    expert_e(s_e h), expert(u) = (silu(u Wgate^T) * (u Wup^T)) Wdown^T: the score multiplies the expert's
    input and is not renormalised.  A shared expert (shared_hidden > 0) takes every token unweighted.

    Options: `score` "softmax" (over all experts) or "logit"; `activation` "relu2": experts without a gate, expert(u) =
    max(u Wup^T, 0)^2 Wdown^T, or another gated unit (GatedMLP's) with its constants `limit` and `sharpness` (and
    `shared_limit` where the shared expert's differs); `group_best` 1: a group ranks by its best expert alone; `weight_on`
    "output": the weight multiplies the expert's output; `correction`: a number per expert is added to the scores
    that the choice goes by (the weights are the scores without it); `groups` = (count, keep): the experts form
    `count` equal groups of neighbours and only those of the `keep` groups whose two largest choice scores have the
    largest sums can be chosen; `normalise`: the weights are the chosen scores over (their sum + 1e-20); `scale`
    multiplies every weight; `shared_gate`: the shared expert's output is multiplied by sigmoid(h . w), one number per
    token (the router kernel computes it, as one more row of its matrix).

    The router kernel writes the step's own table of experts and scores; from there on the experts run as
    those chosen by a stored table do."""

    graph_safe = True
    plan_safe = True

    def __init__(self, width: int, hidden: int, n_experts: int, top: int, shared_hidden: int = 0,
                 score: str = "sigmoid", activation: str = "silu", weight_on: str = "input", correction: bool = False,
                 groups=None, normalise: bool = False, scale: float = 1.0, shared_gate: bool = False,
                 limit: Optional[float] = None, shared_limit: Optional[float] = None, sharpness: float = 1.0,
                 group_best: int = 2) -> None:
        super().__init__(width, hidden, n_experts, top, vocab_size=0, shared_hidden=shared_hidden)
        if score not in kernels.ROUTER_SCORES:
            raise ValueError(f"router score {score!r} is none of {sorted(kernels.ROUTER_SCORES)}")
        self.score = score
        self.gated = activation not in _EXPERT_ACTIVATIONS
        self.epilogue = kernels.EPI_NONE if self.gated else _EXPERT_ACTIVATIONS[activation]
        if self.gated:
            self.unit = _unit_options(activation, limit, sharpness)
            self.shared_unit = _unit_options(activation, limit if shared_limit is None else shared_limit, sharpness)
        if group_best not in (1, 2):
            raise ValueError("a group of experts ranks by its best one (group_best 1) or its two best (2)")
        self.group_best = int(group_best)
        if weight_on not in ("input", "output"):
            raise ValueError(f"weight_on {weight_on!r} is neither 'input' nor 'output'")
        self.weighs_output, self.has_correction = weight_on == "output", bool(correction)
        self.groups = None if groups is None else (int(groups[0]), int(groups[1]))
        if self.groups is not None:
            count, keep = self.groups
            if not 0 < keep <= count or self.n_experts % count or self.top > keep * (self.n_experts // count):
                raise ValueError(f"{self.n_experts} experts in {count} groups of which {keep} stay: need equal groups and "
                                 f"{self.top} experts left to choose")
        self.normalise, self.scale = bool(normalise), float(scale)
        self.gates_shared = bool(shared_gate) and self.shared_hidden > 0
        self.correction = self.shared_gate_weight = None

    def weight_requests(self) -> Dict[str, WeightRequest]:
        req = super().weight_requests()
        del req["table"]
        req["router_weight"] = WeightRequest((self.n_experts, self.width), MATRIX)
        if self.has_correction:
            req["correction"] = WeightRequest((self.n_experts,), VECTOR)
        if self.gates_shared:
            req["shared_gate_weight"] = WeightRequest((1, self.width), MATRIX)
        return req

    def bind(self, tensors):
        self.router_weight = tensors["router_weight"]
        self.correction = tensors.get("correction")
        self.shared_gate_weight = tensors.get("shared_gate_weight")
        return self._bind_experts(tensors)

    def token_matrix_elements(self) -> int:
        return super().token_matrix_elements() + self.n_experts * self.width

    def forward_add(self, ctx: StepContext, h, x: torch.Tensor) -> None:
        plain_residual(ctx, h, x)
        n, ws = ctx.n_rows, ctx.workspace
        hn = as_tensor(ctx, h)
        chosen = ws.get("router_chosen", n, self.top, torch.int32)
        weight = ws.get("router_weight", n, self.top, torch.float32)
        gate = ws.get("router_shared_gate", n, 1, torch.float32).view(-1) if self.gates_shared else None
        rule = dict(q_req=ctx.q_req, score=self.score, correction=self.correction, groups=self.groups, normalise=self.normalise,
                    scale=self.scale, extra=self.shared_gate_weight, extra_out=gate, group_best=self.group_best)
        # few tokens: the same launch sorts the pairs
        routed = None
        if n <= kernels.ROUTE_MAX_ROWS and n * self.top < self.TILED_FROM_PAIRS:
            routed = self._slots(ctx, n)
            if not kernels.router_topk(hn, self.router_weight, n, self.top, chosen, weight, slots=routed, **rule):
                routed = None
        if routed is None:
            kernels.router_topk(hn, self.router_weight, n, self.top, chosen, weight, **rule)
        weight = weight.view(-1)
        self._experts_add(ctx, hn, x, n, None, chosen, None if self.weighs_output else weight, 1.0,
                          out_weight=weight if self.weighs_output else None, shared_gate=gate, routed=routed)
