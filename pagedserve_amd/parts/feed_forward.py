"""Feed-forward parts."""

import torch

from ..ops import kernels
from ..weights.loader import MATRIX, VECTOR, ParamSpec
from .base import FeedForward, site_memo
from .registry import register_feed_forward

ACTIVATIONS = ("gelu_tanh", "gelu_erf", "relu2")


@register_feed_forward("dense")
class DenseFeedForward(FeedForward):
    """``residual += act(x W_up + b_up) W_down + b_down``
    (src/model/paged_decoder.py:178-179,224-228; activations ``:273-280``)."""

    graph_safe = True

    accepts_pending_norm = True

    def __init__(self, width: int, dtype, inner: int, activation: str, bias: bool = True):
        if activation not in ACTIVATIONS:
            raise ValueError(f"unknown activation {activation!r}; known: {', '.join(ACTIVATIONS)}")
        self.width = width
        self.dtype = dtype
        self.inner = inner
        self.activation = activation
        self.bias = bias
        self._memo_up, self._memo_down = {}, {}

    def parameters(self):
        params = {
            "up.weight": ParamSpec((self.inner, self.width), MATRIX),
            "down.weight": ParamSpec((self.width, self.inner), MATRIX),
        }
        if self.bias:
            params["up.bias"] = ParamSpec((self.inner,), VECTOR)
            params["down.bias"] = ParamSpec((self.width,), VECTOR)
        return params

    def bind(self, tensors):
        self.up_weight = tensors["up.weight"]
        self.down_weight = tensors["down.weight"]
        self.up_bias = tensors.get("up.bias")
        self.down_bias = tensors.get("down.bias")
        # copies in the layout that the products of few rows (decode steps) read fastest
        self.up_packed = kernels.pack_decode_weight(self.up_weight)
        self.down_packed = kernels.pack_decode_weight(self.down_weight)
        self._memo_up.clear()
        self._memo_down.clear()

    def forward(self, x, residual, ctx):
        hidden = ctx.workspace.first_rows("ffn", self.inner, self.dtype, ctx.tokens)
        # (the hidden rows belong to these two calls alone: at 17 to 64 rows the first may leave
        # them in the order in which the second reads them)
        _, hidden_packed = kernels.linear(x, self.up_weight, self.up_bias, hidden,
                                          epilogue=self.activation, packed=self.up_packed,
                                          packed_out=True, memo=site_memo(self._memo_up, ctx.workspace),
                                          shared=ctx.shared_calls)
        kernels.linear(hidden, self.down_weight, self.down_bias, residual, epilogue="residual",
                       packed=self.down_packed, a_packed=hidden_packed, memo=site_memo(self._memo_down, ctx.workspace),
                       shared=ctx.shared_calls)


@register_feed_forward("gated")
class GatedFeedForward(FeedForward):
    """``residual += W_down (act(W_gate x) * (W_up x))``, no biases; ``activation``: ``silu`` (with
    other constants of the gated unit as ``form = (limit, slope, shift)``: ``g' sigmoid(slope g') (u' +
    shift)`` of ``g' = min(W_gate x, limit)`` and ``u' = clamp(W_up x, -limit, limit)``) or
    ``gelu_tanh`` or ``relu``.  One packed product gives ``[gate | up]`` in float; the activation and the
    product of the halves are 32-bit.  ``forward(row_scale=...)``: a float per token that
    multiplies its result.  ``ride``: that many more rows of the packed product belong to the caller;
    ``forward`` returns their float columns."""

    graph_safe = True

    accepts_pending_norm = True

    def __init__(self, width: int, dtype, inner: int, activation: str = "silu", form=kernels.PLAIN_GATE,
                 ride: int = 0):
        if activation not in kernels.GATE_ACTIVATIONS:
            raise ValueError(f"unknown gate activation {activation!r}; known: "
                             f"{', '.join(kernels.GATE_ACTIVATIONS)}")
        self.width = width
        self.dtype = dtype
        self.inner = inner
        self.activation = activation
        self.form = tuple(float(value) for value in form)
        self.ride = int(ride)
        self._memo_up, self._memo_down = {}, {}

    def parameters(self):
        return {
            "gate_up.weight": ParamSpec((2 * self.inner + self.ride, self.width), MATRIX),
            "down.weight": ParamSpec((self.width, self.inner), MATRIX),
        }

    def bind(self, tensors):
        self.gate_up_weight = tensors["gate_up.weight"]
        self.down_weight = tensors["down.weight"]
        self.gate_up_packed = kernels.pack_decode_weight(self.gate_up_weight)
        self.down_packed = kernels.pack_decode_weight(self.down_weight)
        self._memo_up.clear()
        self._memo_down.clear()

    def forward(self, x, residual, ctx, row_scale=None):
        tokens = ctx.tokens
        whole, both, ridden = ctx.workspace.column_views("ffn_gate_up", 2 * self.inner + self.ride, torch.float32,
                                                         tokens, (2 * self.inner, self.ride))
        kernels.linear(x, self.gate_up_weight, None, whole, packed=self.gate_up_packed,
                       memo=site_memo(self._memo_up, ctx.workspace), shared=ctx.shared_calls)
        hidden = ctx.workspace.first_rows("ffn", self.inner, self.dtype, tokens)
        kernels.silu_gate(both, hidden, self.activation, form=self.form, row_scale=row_scale)
        kernels.linear(hidden, self.down_weight, None, residual, epilogue="residual",
                       packed=self.down_packed, memo=site_memo(self._memo_down, ctx.workspace),
                       shared=ctx.shared_calls)
        return ridden if self.ride else None


@register_feed_forward("moe")
class MixtureOfExperts(FeedForward):
    """``experts`` small feed-forwards (no biases) of which each token uses ``top``:

        s = softmax(W_router x) over all experts, the logits in 32-bit
        experts form ``groups`` equal groups of neighbours; a group's score is its largest s and
        only experts of the ``keep`` best groups may be chosen; the ``top`` largest s among them are
        residual += sum over the chosen e of (s_e * scale) * W_down,e (silu(W_gate,e x) * (W_up,e x))

    The weights are not renormalised.  The experts' matrices are stacked, ``[experts, gate rows
    | up rows, width]`` and ``[experts, width, inner]``; the choice stays on the device
    (``csrc/moe.hip``).

    Options: ``score="sigmoid"``: ``s = sigmoid(z)``; ``score="chosen_softmax"``: the choice by the
    logits, the weights the softmax over the chosen logits only; ``correction``: a number per expert
    (``router.correction``) is added to ``s`` for the choice only, the weights use ``s`` without it;
    ``group_top``: a group's score is the sum of that many of its largest choice scores;
    ``normalise``: the chosen scores are divided by their sum (+ 1e-20) before ``scale``;
    ``form="relu2"``: an expert is ``W_down,e relu(W_up,e x)^2`` (``up.weight [experts * inner,
    width]``); ``gate_form = (limit, slope, shift)``: other constants of the gated form's unit, which
    becomes ``g' sigmoid(slope g') (u' + shift)`` with ``g' = min(g, limit)`` and ``u' = clamp(u, -limit,
    limit)``; ``shared_inner > 0``: one more expert of the same form, of that inner width and with
    ``shared_limit`` in place of the limit, (``shared.*``) runs for every token with weight one, or, with
    ``shared_gate``, with the weight ``sigmoid(w x)`` of a learned row (``shared_gate.weight``), which
    the router's launch works out in 32-bit.  Steps of few tokens run the shared expert inside the
    experts' own two launches, as one more choice of every token; steps of many tokens run it as
    two dense products."""

    graph_safe = True

    accepts_pending_norm = False

    SCORES = tuple(kernels.ROUTE_SCORES)
    FORMS = ("gated_silu", "relu2")

    def __init__(self, width: int, dtype, inner: int, experts: int, top: int, groups: int = 1,
                 keep: int = 1, scale: float = 1.0, score: str = "softmax", correction: bool = False,
                 group_top: int = 1, normalise: bool = False, form: str = "gated_silu",
                 gate_form=kernels.PLAIN_GATE, shared_inner: int = 0, shared_limit=None,
                 shared_gate: bool = False):
        if groups < 1 or experts % groups:
            raise ValueError(f"{groups} groups do not divide {experts} experts")
        if not 1 <= keep <= groups:
            raise ValueError(f"keep ({keep}) must lie in 1..groups ({groups})")
        if not 1 <= top <= (experts // groups) * keep:
            raise ValueError(f"top ({top}) exceeds the experts that may be chosen")
        if score not in self.SCORES:
            raise ValueError(f"unknown router score {score!r}; known: {', '.join(self.SCORES)}")
        if form not in self.FORMS:
            raise ValueError(f"unknown expert form {form!r}; known: {', '.join(self.FORMS)}")
        if not 1 <= group_top <= 8:
            raise ValueError(f"group_top ({group_top}) must lie in 1..8")
        self.width = width
        self.dtype = dtype
        self.inner = inner
        self.experts = experts
        self.top = top
        self.groups = groups
        self.keep = keep
        self.scale = float(scale)
        self.score = score
        self.has_correction = bool(correction)
        self.group_top = int(group_top)
        self.normalise = bool(normalise)
        self.gated = form == "gated_silu"
        self.first_rows = (2 if self.gated else 1) * inner     # rows of an expert's first matrix
        self.first_name = "gate_up.weight" if self.gated else "up.weight"
        self.gate_form = tuple(float(value) for value in gate_form)
        self.shared_limit = self.gate_form[0] if shared_limit is None else float(shared_limit)
        self.shared = None
        self.shared_inner = int(shared_inner)
        self.has_shared_gate = bool(shared_gate)
        if self.has_shared_gate and not shared_inner:
            raise ValueError("a gate for the shared expert needs a shared expert")
        if shared_inner:
            if self.gated:
                self.shared = GatedFeedForward(width, dtype, shared_inner,
                                               form=(self.shared_limit,) + self.gate_form[1:])
            elif self.has_shared_gate:
                raise ValueError("a gate for the shared expert goes with the gated form")
            else:
                self.shared = DenseFeedForward(width, dtype, shared_inner, "relu2", bias=False)
        # whether the shared expert may ride along in the row kernels (at inner widths that are no
        # multiples of 8 they keep a token's hidden rows of all its experts in LDS)
        self.shared_rides = bool(shared_inner) and (
            (inner % 8 == 0 and shared_inner % 8 == 0) or (top * inner + shared_inner) * 4 <= 64 * 1024)

    def parameters(self):
        params = {
            "router.weight": ParamSpec((self.experts, self.width), VECTOR),
            self.first_name: ParamSpec((self.experts * self.first_rows, self.width), MATRIX),
            "down.weight": ParamSpec((self.experts * self.width, self.inner), MATRIX),
        }
        if self.has_correction:
            params["router.correction"] = ParamSpec((self.experts,), VECTOR)
        if self.shared is not None:
            for name, spec in self.shared.parameters().items():
                params["shared." + name] = spec
        if self.has_shared_gate:
            params["shared_gate.weight"] = ParamSpec((1, self.width), VECTOR)
        return params

    def bind(self, tensors):
        self.router_weight = tensors["router.weight"]
        self.correction = tensors["router.correction"] if self.has_correction else None
        self.first_weight = tensors[self.first_name].view(self.experts, self.first_rows, self.width)
        if self.gated:
            self.gate_up_weight = self.first_weight
        self.down_weight = tensors["down.weight"].view(self.experts, self.width, self.inner)
        if self.shared is not None:
            self.shared.bind({name: tensors["shared." + name] for name in self.shared.parameters()})
            self.shared_extra = (self.shared.gate_up_weight if self.gated else self.shared.up_weight,
                                 self.shared.down_weight)
        self.shared_gate = tensors["shared_gate.weight"].view(-1) if self.has_shared_gate else None

    def forward(self, x, residual, ctx):
        tokens = ctx.tokens
        workspace = ctx.workspace
        sorted_path = (tokens * self.top >= kernels.MOE_GROUPED_FROM
                       and kernels.moe_grouped_supported(self.dtype, self.width, self.inner))
        # few tokens: the shared expert rides along as one more choice of every token
        rides = self.shared_rides and not sorted_path
        chosen = self.top + (1 if rides else 0)
        ids = workspace.first_rows("moe_ids", chosen, torch.int32, tokens)
        weights = workspace.first_rows("moe_weights", chosen, torch.float32, tokens)
        gates = None
        if self.has_shared_gate and not rides:
            gates = workspace.rows("moe_shared_gates", 1, torch.float32).view(-1)[:tokens]
        kernels.moe_route(x, self.router_weight, self.groups, self.keep, self.top, self.scale, ids,
                          weights, score=self.score, correction=self.correction,
                          group_top=self.group_top, normalise=self.normalise, fixed=rides,
                          gate=self.shared_gate, gate_out=gates)
        hidden = workspace.rows("moe_hidden", self.top * self.inner + self.shared_inner, self.dtype)
        if sorted_path:
            most = workspace.max_rows * self.top
            # many rows: sorted by expert, tiles on the matrix cores
            tiles = kernels.moe_grouped_tiles(most, self.experts)
            kernels.moe_experts_grouped(
                x, self.first_weight, self.down_weight, ids, weights, hidden,
                workspace.rows("moe_out", self.width, torch.float32, max_rows=most),
                workspace.flat("moe_order", tiles * kernels.MOE_TILE, torch.int32),
                workspace.flat("moe_tiles", tiles, torch.int32), residual, gated=self.gated,
                form=self.gate_form)
        else:
            kernels.moe_experts(x, self.first_weight, self.down_weight, ids, weights, hidden, residual,
                                gated=self.gated, extra=self.shared_extra if rides else None,
                                form=self.gate_form, extra_limit=self.shared_limit)
        if self.shared is not None and not rides:
            if gates is not None:
                self.shared.forward(x, residual, ctx, row_scale=gates)
            else:
                self.shared.forward(x, residual, ctx)
