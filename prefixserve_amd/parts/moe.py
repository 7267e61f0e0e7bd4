"""Feed-forward as a mixture of experts: a router picks a few small feed-forwards per token."""

from __future__ import annotations

from typing import TYPE_CHECKING, Mapping

import torch

from .base import FeedForward, Runtime, WeightWant, register_feed_forward

if TYPE_CHECKING:
    from prefixserve_amd.engine.batch import StepContext


# How a router scores: the code the kernels take.
SCORES = {"sigmoid": 0, "softmax_of_chosen": 1, "softmax": 2}


class RoutedExperts(FeedForward):
    """``num_experts`` feed-forwards of inner size ``intermediate_size`` without biases, of
    which every token uses ``top_k``.

    Router: z = W_r x (+ a bias, ``router_bias``) in 32-bit; the ``top_k`` largest are taken (the
    lower index among equals). ``score`` "sigmoid": the weights are sigmoid(z) as they are, not
    renormalized; "softmax_of_chosen": the softmax over the chosen z alone; "softmax": the softmax over all z.
    ``choice_bias`` (with "softmax"): a learned number per expert (name "correction") that is added to its score for the
    choice, not for its weight. ``groups`` = {"count": G, "keep": k} (not with "softmax_of_chosen"): the experts form G
    equal groups of neighbours, a group's score is the sum of its two largest scores (``group_score`` "top2") or its
    largest ("max"), as the choice sees them, and only experts of the k best groups can be chosen. ``weight_scale``
    multiplies the weights.

    ``identity``: the router has that many rows more than there are experts, and the last ``identity`` choices are
    identity experts: their output is the token itself times the weight. They count for ``top_k`` and in the groups.

    ``weight_on`` "input": the weight multiplies the expert's input, the output is the sum over
    the chosen experts of expert(w x), which is not w expert(x) when the expert clamps; "output": the
    sum of w expert(x).

    Expert: with g = min(W_gate h, limit) and u = clamp(W_up h, -limit, limit) it is
    W_down (g sigmoid(gate_alpha g) (u + up_shift)); ``limit`` None, ``gate_alpha`` 1 and
    ``up_shift`` 0 make it W_down (silu(W_gate h) * W_up h). ``expert`` "squared_relu": no gate,
    W_down (max(W_up h, 0))^2; the three constants do not apply.

    ``shared`` = {"intermediate_size": F, "gated": bool}: one more SiLU-gated feed-forward that every
    token uses, its output times sigmoid(w . x), one number per token, when ``gated``.

    The chosen experts' outputs (and the shared one's) come back as float32 slices ``[top_k (+ 1), T,
    hidden]`` that the norm behind adds up in ascending order, so a token's sum does not depend on
    what else is in the step; in a bfloat16 step so small that the products add into the residual stream
    themselves (``ops.fuses_norm``) the experts do so too. ``names``: "router" ("router_bias"), "gate"/"up"/"down" with ``{e}``
    for the expert, "shared_gate"/"shared_up"/"shared_down" ("shared_scale": the [1, hidden] row w; "correction")."""

    takes_residual_scale = True

    def __init__(self, hidden_size: int, num_experts: int, top_k: int, intermediate_size: int,
                 names: Mapping[str, str], limit: float | None = None, gate_alpha: float = 1.702, up_shift: float = 1.0,
                 score: str = "sigmoid", renormalize: bool = False, weight_on: str = "input",
                 router_bias: bool = False, shared: Mapping[str, object] | None = None, expert: str = "gated",
                 groups: Mapping[str, int] | None = None, weight_scale: float = 1.0, choice_bias: bool = False,
                 group_score: str = "top2", identity: int = 0) -> None:
        if score not in SCORES or renormalize or weight_on not in ("input", "output"):
            raise ValueError("the router kernels score with a sigmoid or a softmax (scores kept as weights) or with the softmax over the "
                             f"chosen logits, on the experts' input or output; got score={score!r}, "
                             f"renormalize={renormalize}, weight_on={weight_on!r}")
        choices = num_experts + identity
        if num_experts < 1 or identity < 0 or not 1 <= top_k <= choices:
            raise ValueError(f"top_k {top_k} of {num_experts} experts and {identity} identity experts")
        if choice_bias and score != "softmax":
            raise ValueError("a correction of the choice goes with the softmax over all experts")
        if identity and weight_on != "output":
            raise ValueError("identity experts' weights multiply the output")
        if group_score not in ("top2", "max"):
            raise ValueError(f"a group's score is that of its two largest or of its largest, got {group_score!r}")
        if expert not in ("gated", "squared_relu"):
            raise ValueError(f"experts are gated or squared ReLU without a gate, got {expert!r}")
        if groups is not None:
            count, keep = int(groups["count"]), int(groups["keep"])
            if score == "softmax_of_chosen" or not 1 <= count <= 256 or choices % count or not 1 <= keep <= count \
                    or top_k > keep * (choices // count):
                raise ValueError(f"{choices} experts in {count} groups of which {keep} are kept, {top_k} chosen, score {score!r}")
        self.hidden_size, self.num_experts, self.top_k = int(hidden_size), int(num_experts), int(top_k)
        self.intermediate_size = int(intermediate_size)
        self.names = dict(names)
        self.limit = float("inf") if limit is None else float(limit)
        self.gate_alpha, self.up_shift = float(gate_alpha), float(up_shift)
        self.router_mode = SCORES[score]
        self.choice_bias, self.identity, self.choices = bool(choice_bias), int(identity), int(choices)
        self.weight_on_output = weight_on == "output"
        self.router_bias = bool(router_bias)
        self.shared_size = None if shared is None else int(shared["intermediate_size"])
        self.shared_gated = shared is not None and bool(shared.get("gated", False))
        self.expert = expert
        # What the calls name beyond the plain form (sigmoid scores, gated experts, weight on the input).
        self.route_options: dict[str, object] = {}
        if self.router_mode or self.router_bias:
            self.route_options["mode"] = self.router_mode
        if groups is not None:
            self.route_options.update(groups=count, keep=keep)
            if group_score == "max":
                self.route_options["group_max"] = True
        if weight_scale != 1.0:
            self.route_options["factor"] = float(weight_scale)
        self.expert_options: dict[str, object] = {}
        if self.identity:
            self.route_options["identity"] = self.expert_options["identity"] = self.identity
        if self.weight_on_output:
            self.expert_options["weight_on_output"] = True
        if expert != "gated":
            self.expert_options["kind"] = expert

    def weights(self) -> dict[str, WeightWant]:
        h, f, n = self.hidden_size, self.intermediate_size, self.names
        want = {n["router"]: WeightWant((self.choices, h))}
        if self.router_bias:
            want[n["router_bias"]] = WeightWant((self.choices,), "bias")
        if self.choice_bias:
            want[n["correction"]] = WeightWant((self.choices,), "offset")
        for e in range(self.num_experts):
            if self.expert == "gated":
                want[n["gate"].format(e=e)] = WeightWant((f, h))
            want[n["up"].format(e=e)] = WeightWant((f, h))
            want[n["down"].format(e=e)] = WeightWant((h, f))
        if self.shared_size is not None:
            want[n["shared_gate"]] = WeightWant((self.shared_size, h))
            want[n["shared_up"]] = WeightWant((self.shared_size, h))
            want[n["shared_down"]] = WeightWant((h, self.shared_size))
            if self.shared_gated:
                want[n["shared_scale"]] = WeightWant((1, h))
        return want

    def bind(self, tensors: Mapping[str, torch.Tensor], rt: Runtime) -> None:
        super().bind(tensors, rt)
        n, e_n = self.names, self.num_experts
        # The router stays 32-bit whatever the activation dtype.
        self.w_router = tensors[n["router"]].to(device=rt.device, dtype=torch.float32).contiguous()
        # ... and also stands in the activation dtype for steps whose logits a product kernel computes
        # (bfloat16 x bfloat16 products are exact in float32, where they are summed).
        self.w_router_act = self.w_router if rt.dtype == torch.float32 else rt.ops.prepare_matrix(tensors[n["router"]], rt)
        self.b_router = None
        if self.router_bias:
            self.b_router = tensors[n["router_bias"]].to(device=rt.device, dtype=torch.float32).contiguous()
        if self.choice_bias:
            self.route_options["correction"] = tensors[n["correction"]].to(device=rt.device, dtype=torch.float32).contiguous()
        # Per expert the rows of gate (where there is one), then of up: [E, 2F or F, H]; and down [E, H, F].
        first = ("gate", "up") if self.expert == "gated" else ("up",)
        self.w_in = rt.ops.prepare_matrix(torch.stack([torch.cat([tensors[n[which].format(e=e)] for which in first], dim=0)
                                                       for e in range(e_n)]), rt)
        self.w_down = rt.ops.prepare_matrix(torch.stack([tensors[n["down"].format(e=e)] for e in range(e_n)]), rt)
        self.w_shared_gate_up = self.w_shared_down = self.w_shared_scale = None
        if self.shared_size is not None:
            self.w_shared_gate_up = rt.ops.prepare_matrix(torch.cat([tensors[n["shared_gate"]], tensors[n["shared_up"]]], dim=0), rt)
            self.w_shared_down = rt.ops.prepare_matrix(tensors[n["shared_down"]], rt)
            if self.shared_gated:
                self.w_shared_scale = tensors[n["shared_scale"]].to(device=rt.device, dtype=torch.float32).reshape(-1).contiguous()

    def weight_bytes(self) -> int:
        """What a decode step of one token reads: the router, ``top_k`` experts and the shared one."""
        per_expert = (self.w_in.numel() + self.w_down.numel()) // self.num_experts * self.w_down.element_size()
        shared = 0
        if self.w_shared_gate_up is not None:
            shared = (self.w_shared_gate_up.numel() + self.w_shared_down.numel()) * self.w_shared_down.element_size()
        return self.w_router.numel() * 4 + self.top_k * per_expert + shared

    def _adds_into_stream(self, t: int, residual: torch.Tensor | None) -> bool:
        fuses = getattr(self.rt.ops, "fuses_norm", None)
        return (residual is not None and self.shared_size is None and fuses is not None
                and fuses(t, self.hidden_size, self.rt.dtype))

    def forward(self, x: torch.Tensor, ctx: "StepContext") -> torch.Tensor | None:
        rt, ops, ws = self.rt, self.rt.ops, self.rt.workspace
        t, k = x.shape[0], self.top_k
        chosen = ws.get("moe.chosen", (t, k), torch.int32)
        weight = ws.get("moe.weight", (t, k), torch.float32)
        act = ws.get("moe.act", (t * k, self.intermediate_size), rt.dtype)
        if self.b_router is not None:
            ops.moe_route(x, self.w_router, chosen, weight, self.w_router_act, bias=self.b_router, **self.route_options)
        else:
            ops.moe_route(x, self.w_router, chosen, weight, self.w_router_act, **self.route_options)
        residual = getattr(ctx, "residual", None)
        if self._adds_into_stream(t, residual):
            ops.moe_experts(x, chosen, weight, self.w_in, self.w_down, act, None, self.gate_alpha, self.limit, self.up_shift,
                            residual=residual, col_scale=getattr(ctx, "residual_scale", None), **self.expert_options)
            return None
        slices = k + (1 if self.shared_size is not None else 0)
        out = ws.get("moe.out", (slices, t, self.hidden_size), torch.float32)
        ops.moe_experts(x, chosen, weight, self.w_in, self.w_down, act, out[:k], self.gate_alpha, self.limit, self.up_shift,
                        **self.expert_options)
        if self.shared_size is not None:
            shared_act = ws.get("moe.shared_act", (t, self.shared_size), rt.dtype)
            ops.linear_swiglu(x, self.w_shared_gate_up, shared_act)
            ops.linear(shared_act, self.w_shared_down, out[k])
            if self.w_shared_scale is not None:
                ops.row_gate(out[k], x, self.w_shared_scale)
        return out


register_feed_forward("routed_experts", RoutedExperts)
