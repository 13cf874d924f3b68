"""Feed-forward parts of decoders with an fp32 residual stream: a dense gated one, and routed experts behind a softmax router with a
bias or a sigmoid router with a correction, with an optional shared expert; the gated activation is a parameter (kernels.Glu).  forward(h) returns what the launch that finishes the residual adds up (kernels.residual_norm takes
one addend, kernels.residual_rms up to two): rows, split-K partials, or weighted expert rows.

Modules take their tensors from `get(name, shape, init)` (harness/weights.py)."""
from __future__ import annotations

from typing import Callable

import torch
from torch import nn

from .. import kernels
from .activation import rows_vectorisable

BF = torch.bfloat16


class DenseMLP(nn.Module):
    """down(act(gate h, up h)), with biases or without."""

    def __init__(self, width: int, ff: int, get: Callable, linear: Callable, bias: bool = True, act: kernels.Glu = kernels.SILU):
        super().__init__()
        gate_up_b = torch.cat([get("gate.b", (ff,), "zeros"), get("up.b", (ff,), "zeros")], 0) if bias else None
        self.gate_up = linear(torch.cat([get("gate", (ff, width)), get("up", (ff, width))], 0), gate_up_b)
        self.down = linear(get("down", (width, ff)), get("down.b", (width,), "zeros") if bias else None)
        self.act = act

    def forward(self, h: torch.Tensor):
        if self.gate_up.streams(h):                     # decode: bias, silu and the product in the weight stream's epilogue
            b = self.gate_up.bias.data if self.gate_up.bias is not None else None
            return self.down.forward_partials(kernels.wstream_gemm(h, self.gate_up.weight.data, b, epilogue="silu_and_mul", act=self.act))
        g = self.gate_up(h)
        if g.dtype == BF and (g.shape[1] // 2) % 8 == 0 and rows_vectorisable(g, g.shape[1]):
            return self.down(kernels.glu_and_mul(g, self.act))
        return self.down(kernels.gate_mul(g, self.act))


class RoutedMLP(nn.Module):
    """`top` of `experts` small gated parts per token plus a shared part every token takes.  scores="softmax": weighted by the softmax over
    the chosen router logits, which have a bias; "sigmoid": sigmoid scores times router.scale, chosen with a correction out of the best
    router.groups.keep of groups.count groups (kernels.SigmoidScores).  act(constants of an expert) is its activation.  The experts' rows
    are padded with zeros to whole matrix tiles (every activation makes nothing of zero columns)."""

    def __init__(self, width: int, m: dict, get: Callable, linear: Callable, scores: str = "softmax",
                 act: Callable[[dict], kernels.Glu] = lambda expert: kernels.SILU):
        super().__init__()
        r = m["router"]
        E, self.top = r["experts"], r["top"]
        ff, self.act = m["expert"]["ff"], act(m["expert"])
        if not 1 <= self.top <= E or E > 256 or self.top > 64:
            raise ValueError(f"router: {self.top} of {E} experts (at most 64 of 256)")
        self.router = nn.Parameter(get("router", (E, width)).contiguous(), requires_grad=False)
        self.router_bias = self.scores = None
        if scores == "sigmoid":
            groups = r.get("groups") or dict(count=1, keep=1)
            count, keep = groups["count"], groups["keep"]
            if not 1 <= keep <= count or E % count or self.top > keep * (E // count):
                raise ValueError(f"router: {self.top} of {E} experts out of {keep} of {count} groups")
            self.scores = kernels.SigmoidScores(get("correction", (E,), "zeros").float(), count, keep, r.get("scale", 1.0))
        else:
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
        self.shared = None if shared is None else DenseMLP(width, shared["ff"], lambda n, s, init=None: get("shared." + n, s, init), linear, bias=False,
                                                          act=act(shared))
        self.plain_experts = False          # tests: the form without matrix instructions

    def forward(self, h: torch.Tensor) -> tuple:
        weights, ids = kernels.moe_route(h, self.router.data, self.router_bias, self.top, self.scores)
        rows = kernels.ExpertRows(kernels.routed_experts(h, self.w13.data, self.w2.data, ids, self.plain_experts, self.act), weights)
        return (rows,) if self.shared is None else (rows, self.shared(h))     # (the shared part's partials are the last product)
