"""Feed-forwards that route every token to a few of many small experts."""
from __future__ import annotations

from typing import Optional

import torch

from ..config.spec import SILU_GLU, SwiGLUSpec
from ..kernels import ops
from ..kernels.limits import MOE_MAX_EXPERTS, beyond
from ..weights.loader import Expect
from .base import BuildContext, FeedForward, register_part
from .ffn import SwiGLU
from .linear import Linear


@register_part("routed_experts")
class RoutedExperts(FeedForward):
    """sum over a token's ``top_k`` experts of weight * expert(x), plus sigmoid(w_sg . x) * shared(x) (or shared(x) as it
    is: ``shared_gated``).  The router's last ``identity_experts`` outputs are experts that return x; ``groups`` of
    neighbouring outputs may restrict the choice to the best ones.

    An expert is down(act(gate(x), up(x))) with the clamped gated activation of ``ClampedGLUSpec`` and no biases, or
    (an activation that is not ``gated``) down(max(up(x), 0)^2) with no gate matrix.  With ``routing``
    "top_then_softmax" the router's logits get a bias, the largest are chosen and weighted by the softmax over the
    chosen ones alone; with "sigmoid_then_top" every score is the sigmoid of its own logit.  ``input_weighted``: a weight
    multiplies its expert's input; it lies beside the row's place and multiplies the first product's sums, before the
    activation.  The router's logits are a float32 product (its weight is kept in 32 bits, with the shared expert's gate vector as
    one more row); one kernel forms the softmax, adds the correction, picks the experts and their weights.  The
    tokens' rows are then grouped by expert on the device (no count travels to the host: the launch sizes depend on
    the number of tokens alone): each expert's rows fill whole tiles of the grouped products, gate/up with the
    activation in its epilogue, then down into float32 rows, which a last kernel weights and sums token by token, in
    the order of the token's choices, together with the gated shared expert.  A token's result does not depend on
    which other tokens share its expert's tiles: a row of a tile is summed on its own.  The output is float32.
    Steps of up to 64 tokens are routed and grouped in one launch; a shared expert whose activation is plain SiLU runs as
    the dense gated feed-forward does (its activation in the product's epilogue in small steps)."""
    graph_safe = True
    takes_tail = True
    kernel_modules = ("common", "gemm", "moe")

    @classmethod
    def expected_tensors(cls, spec, prefix: str, hidden_size: int):
        out = [Expect(f"{prefix}.router.weight", ((spec.router_outputs, hidden_size),))]
        if spec.routing == "top_then_softmax":
            out.append(Expect(f"{prefix}.router.bias", ((spec.num_experts,),), init="bias"))
        elif spec.corrected:
            out.append(Expect(f"{prefix}.correction", ((spec.router_outputs,),), init="bias"))
        gated = getattr(spec.activation, "gated", True)
        for number in range(spec.num_experts):
            if gated:
                out.append(Expect(f"{prefix}.e{number}.gate.weight", ((spec.expert_size, hidden_size),)))
            out += [Expect(f"{prefix}.e{number}.up.weight", ((spec.expert_size, hidden_size),)),
                    Expect(f"{prefix}.e{number}.down.weight", ((hidden_size, spec.expert_size),))]
        if spec.shared_size is not None:
            out += [Expect(f"{prefix}.shared.gate.weight", ((spec.shared_size, hidden_size),)),
                    Expect(f"{prefix}.shared.up.weight", ((spec.shared_size, hidden_size),)),
                    Expect(f"{prefix}.shared.down.weight", ((hidden_size, spec.shared_size),))]
            if spec.shared_gated:
                out.append(Expect(f"{prefix}.shared.sg.weight", ((1, hidden_size),)))
        return out

    @classmethod
    def limits(cls, spec, hidden_size: int):
        return beyond("routed_experts", "num_experts", spec.router_outputs, MOE_MAX_EXPERTS,
                      "the experts' counts and a token's scores are kept in LDS and registers")

    def __init__(self, spec, prefix: str, tensors, build: BuildContext):
        self.spec = spec
        self.build = build
        get = lambda name: tensors[f"{prefix}.{name}"]
        experts, inner, hidden = spec.num_experts, spec.expert_size, build.hidden_size
        # rows of 16-byte pieces for the bfloat16 matrix cores, else the float32 kernel (any width)
        keep = torch.float32 if (build.dtype == torch.float32 or hidden % 8 or inner % 8) else torch.bfloat16
        self.gated = getattr(spec.activation, "gated", True)
        if self.gated:
            first = [torch.cat([get(f"e{number}.gate.weight"), get(f"e{number}.up.weight")]) for number in range(experts)]
        else:
            first = [get(f"e{number}.up.weight") for number in range(experts)]
        self.gate_up = torch.stack(first).to(keep).contiguous().to(build.device)
        self.down = torch.stack([get(f"e{number}.down.weight") for number in range(experts)]) \
            .to(keep).contiguous().to(build.device)
        # the router's product has float32 sums; a weight stored in bfloat16 beside bfloat16 rows gives exact float32
        # products on the matrix cores, so it stays as it is stored; any other keeps 32 bits and the float32 kernel
        stored = {get("router.weight").dtype} | ({get("shared.sg.weight").dtype} if spec.shared_size is not None and spec.shared_gated else set())
        route_dtype = torch.bfloat16 if (build.dtype == torch.bfloat16 and stored == {torch.bfloat16} and hidden % 8 == 0) \
            else torch.float32
        router = [get("router.weight").to(route_dtype)]
        self.shared = spec.shared_size is not None
        if self.shared:
            if spec.shared_gated:
                router.append(get("shared.sg.weight").to(route_dtype).reshape(1, hidden))
            self.shared_dense = None
            if spec.shared_activation == SILU_GLU:
                named = {f"shared.{name}_proj.weight": get(f"shared.{name}.weight") for name in ("gate", "up", "down")}
                self.shared_dense = SwiGLU(SwiGLUSpec(intermediate_size=spec.shared_size), "shared", named, build)
            else:
                self.shared_gate_up = Linear([get("shared.gate.weight"), get("shared.up.weight")], [None, None], build)
                self.shared_down = Linear([get("shared.down.weight")], [None], build)
        self.router = torch.cat(router).contiguous().to(build.device)
        # what is added to a token's scores before the choice: a correction of the softmax, or the logits' bias
        self.correction = None
        if spec.corrected:
            added = "router.bias" if spec.routing == "top_then_softmax" else "correction"
            self.correction = get(added).to(torch.float32).contiguous().to(build.device)
        # rows and matrices in whole 16-byte pieces: the widest tiles of the grouped products take nothing else
        piece = 4 if keep == torch.float32 else 8
        self.whole_pieces = hidden % piece == 0 and inner % piece == 0

    def _shared_rows(self, x: torch.Tensor) -> torch.Tensor:
        if self.shared_dense is not None:
            return self.shared_dense.forward(x)
        act = self.spec.shared_activation
        gate_up = self.shared_gate_up(x)
        activated = torch.empty((x.shape[0], self.spec.shared_size), dtype=gate_up.dtype, device=x.device)
        ops.clamped_glu(gate_up, act.limit, act.alpha, act.up_offset, activated)
        return self.shared_down(activated)

    def forward(self, x: torch.Tensor, tail=None) -> Optional[torch.Tensor]:
        spec = self.spec
        tokens, hidden = x.shape
        logits = ops.linear(x, self.router, None, keep_float32=True)          # float32 [T, experts (+ 1)]
        how = dict(routing=spec.routing, renormalize=spec.renormalize, groups=spec.groups, kept_groups=spec.kept_groups)
        choice = (logits, spec.router_outputs, spec.top_k, self.correction, spec.route_scale, spec.weight_eps,
                  self.shared and spec.shared_gated)
        pad = ops.moe_tile_rows(tokens, spec.top_k, spec.num_experts, self.whole_pieces)
        if tokens <= ops.ROUTE_PLAN_TOKENS:
            _, weights, gate, plan = ops.moe_route_plan(*choice, experts_with_matrices=spec.num_experts, pad=pad,
                                                         place_weights=spec.input_weighted, **how)
        else:
            chosen, weights, gate = ops.moe_route(*choice, **how)
            plan = ops.moe_plan(chosen, spec.num_experts, pad, weights if spec.input_weighted else None)
        if spec.input_weighted:                # the weights are in the rows: the sum of the experts' outputs is plain
            weights = None
        rows = x if x.dtype == self.gate_up.dtype else x.to(self.gate_up.dtype)
        inner = torch.empty((plan.capacity, spec.expert_size), dtype=rows.dtype, device=x.device)
        ops.moe_expert_gemm(rows, plan, self.gate_up, inner, gather=True, glu=spec.activation if self.gated else None,
                            squared_relu=not self.gated, row_scale=plan.place_weight if spec.input_weighted else None)
        down = torch.empty((plan.capacity, hidden), dtype=torch.float32, device=x.device)
        ops.moe_expert_gemm(inner, plan, self.down, down, gather=False, glu=None)
        shared_rows = self._shared_rows(x) if self.shared else None
        own_rows = x if spec.identity_experts else None
        if tail is not None and (own_rows is None or own_rows.dtype == tail.dtype):
            ops.moe_combine(down, plan, weights, shared_rows, gate, None, own_rows, tail.stream_arguments())
            return None
        out = torch.empty((tokens, hidden), dtype=torch.float32, device=x.device)
        ops.moe_combine(down, plan, weights, shared_rows, gate, out, own_rows)
        return out
