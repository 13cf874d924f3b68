"""Feed-forward parts of decoders with an fp32 residual stream: a dense gated one, and routed experts with a biased router and an
optional shared expert.  forward(h) returns what the launch that finishes the residual adds up (kernels.residual_norm takes
one addend, kernels.residual_rms up to two): rows, split-K partials, or weighted expert rows.

Modules take their tensors from `get(name, shape, init)` (harness/weights.py)."""
from __future__ import annotations

from typing import Callable

import torch
from torch import nn

from .. import kernels
from .activation import SiluAndMul, rows_vectorisable

BF = torch.bfloat16


class DenseMLP(nn.Module):
    """down(silu(gate h) * (up h)), with biases or without."""

    def __init__(self, width: int, ff: int, get: Callable, linear: Callable, bias: bool = True):
        super().__init__()
        gate_up_b = torch.cat([get("gate.b", (ff,), "zeros"), get("up.b", (ff,), "zeros")], 0) if bias else None
        self.gate_up = linear(torch.cat([get("gate", (ff, width)), get("up", (ff, width))], 0), gate_up_b)
        self.down = linear(get("down", (width, ff)), get("down.b", (width,), "zeros") if bias else None)
        self.act = SiluAndMul()

    def forward(self, h: torch.Tensor):
        if self.gate_up.streams(h):                     # decode: bias, silu and the product in the weight stream's epilogue
            b = self.gate_up.bias.data if self.gate_up.bias is not None else None
            return self.down.forward_partials(kernels.wstream_gemm(h, self.gate_up.weight.data, b, epilogue="silu_and_mul"))
        g = self.gate_up(h)
        if g.dtype == BF and (g.shape[1] // 2) % 8 == 0 and rows_vectorisable(g, g.shape[1]):
            return self.down(kernels.silu_and_mul(g, round_intermediate=False))
        return self.down(kernels.gate_mul(g))


class RoutedMLP(nn.Module):
    """`top` of `experts` small gated parts per token, weighted by the softmax over the chosen router logits, plus a shared part every
    token takes.  The experts' rows are padded with zeros to whole matrix tiles (silu(0) * 0 adds nothing)."""

    def __init__(self, width: int, m: dict, get: Callable, linear: Callable):
        super().__init__()
        E, self.top = m["router"]["experts"], m["router"]["top"]
        ff = m["expert"]["ff"]
        if not 1 <= self.top <= E or E > 256 or self.top > 64:
            raise ValueError(f"router: {self.top} of {E} experts (at most 64 of 256)")
        self.router = nn.Parameter(get("router", (E, width)).contiguous(), requires_grad=False)
        self.router_bias = get("router.b", (E,), "zeros").float()
        first = get("e0.gate", (ff, width))
        pad = -ff % 64 if first.dtype == BF else 0
        w13 = torch.zeros((E, 2 * (ff + pad), width), dtype=first.dtype, device=first.device)
        w2 = torch.zeros((E, width, ff + pad), dtype=first.dtype, device=first.device)
        for e in range(E):
            w13[e, :ff] = first if e == 0 else get(f"e{e}.gate", (ff, width))
            w13[e, ff + pad:2 * ff + pad] = get(f"e{e}.up", (ff, width))
            w2[e, :, :ff] = get(f"e{e}.down", (width, ff))
        self.w13, self.w2 = nn.Parameter(w13, requires_grad=False), nn.Parameter(w2, requires_grad=False)
        shared = m.get("shared")
        self.shared = None if shared is None else DenseMLP(width, shared["ff"], lambda n, s, init=None: get("shared." + n, s, init), linear, bias=False)
        self.plain_experts = False          # tests: the form without matrix instructions

    def forward(self, h: torch.Tensor) -> tuple:
        weights, ids = kernels.moe_route(h, self.router.data, self.router_bias, self.top)
        rows = kernels.ExpertRows(kernels.routed_experts(h, self.w13.data, self.w2.data, ids, self.plain_experts), weights)
        return (rows,) if self.shared is None else (rows, self.shared(h))     # (the shared part's partials are the last product)
