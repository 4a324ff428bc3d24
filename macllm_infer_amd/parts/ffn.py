"""Dense feed-forward parts."""
from __future__ import annotations

from typing import Optional

import torch

from ..kernels import ops
from ..weights.loader import Expect
from .base import BuildContext, FeedForward, register_part
from .linear import Linear


@register_part("swiglu")
class SwiGLU(FeedForward):
    """down(act(gate(x)) * up(x)), act = SiLU or the tanh form of GELU (``activation``), or down of the clamped gated
    activation of gate(x) and up(x) (``clamp``); gate and up are one fused
    product (reference: src/decoder.rs:261-306).  ``gate_multiplier`` scales gate's output,
    ``down_multiplier`` down's output; both are folded into the weights.  When the width is a
    multiple of 8 the rows of the fused matrix are stored in tiles of 8 gate rows and 8 up rows
    (``tile``), the order the fused decode kernel wants, so that one matrix serves every path."""
    graph_safe = True
    takes_tail = True
    kernel_modules = ("common", "gemm")

    @classmethod
    def expected_tensors(cls, spec, prefix: str, hidden_size: int):
        inner = spec.intermediate_size
        out = [Expect(f"{prefix}.gate_proj.weight", ((inner, hidden_size),)),
               Expect(f"{prefix}.up_proj.weight", ((inner, hidden_size),)),
               Expect(f"{prefix}.down_proj.weight", ((hidden_size, inner),))]
        if spec.bias:
            out += [Expect(f"{prefix}.gate_proj.bias", ((inner,),), init="bias"),
                    Expect(f"{prefix}.up_proj.bias", ((inner,),), init="bias"),
                    Expect(f"{prefix}.down_proj.bias", ((hidden_size,),), init="bias")]
        return out

    def __init__(self, spec, prefix: str, tensors, build: BuildContext):
        self.spec = spec
        inner = spec.intermediate_size
        get = lambda name: tensors.get(f"{prefix}.{name}")
        scale = torch.cat([torch.full((inner,), spec.gate_multiplier), torch.ones(inner)])
        self.gate_up = Linear([get("gate_proj.weight"), get("up_proj.weight")],
                              [get("gate_proj.bias"), get("up_proj.bias")], build,
                              weight_scale=scale, bias_scale=scale)
        self.down = Linear([get("down_proj.weight")], [get("down_proj.bias")], build,
                           weight_scale=spec.down_multiplier, bias_scale=spec.down_multiplier)
        self.tile = 8 if inner % 8 == 0 else 0
        if self.tile:
            order = torch.arange(2 * inner).view(2, inner // 8, 8).permute(1, 0, 2).reshape(-1).to(build.device)
            self.gate_up.weight = self.gate_up.weight[order].contiguous()
            if self.gate_up.bias is not None:
                self.gate_up.bias = self.gate_up.bias[order].contiguous()
            if self.gate_up.bias16 is not None:
                self.gate_up.bias16 = self.gate_up.bias16[order].contiguous()

    def gated_projections(self):
        if self.spec.activation != "silu":          # the fused decode kernels apply SiLU
            return None
        return self.gate_up, self.down, self.tile

    def forward(self, x: torch.Tensor, tail=None) -> Optional[torch.Tensor]:
        activated = self.activated(x)
        if tail is not None and tail.project(self.down, activated):
            return None
        return self.down(activated)

    def activated(self, x: torch.Tensor) -> torch.Tensor:
        """act(gate(x)) * up(x)."""
        rows, width = x.shape
        if (self.tile == 8 and x.dtype == torch.bfloat16 and self.gate_up.weight.dtype == torch.bfloat16
                and rows <= ops.SKINNY_ROWS and width % 32 == 0
                and x.stride(1) == 1 and x.stride(0) % 8 == 0 and x.data_ptr() % 16 == 0
                and ops.fused_gemm_supported(False, rows, width)):
            # a step of a few rows: the gate's activation and the product with the up half in the skinny kernel's
            # epilogue (the weight rows already lie in its tiles of 8 gate and 8 up rows)
            activated = torch.empty((rows, self.spec.intermediate_size), dtype=x.dtype, device=x.device)
            ops.fused_gemm(self.gate_up.weight, self.gate_up.bias, activated, x=x, epilogue=ops.EPI_SWIGLU,
                           gate_activation=self.spec.activation, clamp=self.spec.clamp)
            return activated
        gate_up = self.gate_up(x)
        activated = torch.empty((x.shape[0], self.spec.intermediate_size), dtype=gate_up.dtype, device=x.device)
        ops.swiglu(gate_up, activated, self.tile, activation=self.spec.activation, clamp=self.spec.clamp)
        return activated


@register_part("polynorm_ffn")
class PolyNormFFN(FeedForward):
    """down(act(up(x))) with act(z) = c0 N(z) + c1 N(z^2) + c2 N(z^3) + c3: powers element by element, N divides
    a token's row of inner values by its root mean square (three sums of squares over the row, in float32, one
    kernel).  The four numbers are the tensor ``act``."""
    graph_safe = True
    kernel_modules = ("common", "gemm")

    @classmethod
    def expected_tensors(cls, spec, prefix: str, hidden_size: int):
        inner = spec.intermediate_size
        return [Expect(f"{prefix}.up.weight", ((inner, hidden_size),)),
                Expect(f"{prefix}.down.weight", ((hidden_size, inner),)),
                Expect(f"{prefix}.act", ((4,),), init="scale")]

    def __init__(self, spec, prefix: str, tensors, build: BuildContext):
        self.spec = spec
        self.up = Linear([tensors[f"{prefix}.up.weight"]], [None], build)
        self.down = Linear([tensors[f"{prefix}.down.weight"]], [None], build)
        self.coefficients = tensors[f"{prefix}.act"].to(torch.float32).contiguous().to(build.device)

    def forward(self, x: torch.Tensor) -> torch.Tensor:
        inner = self.up(x)
        activated = torch.empty_like(inner)
        ops.polynorm(inner, self.coefficients, self.spec.eps, activated)
        return self.down(activated)
