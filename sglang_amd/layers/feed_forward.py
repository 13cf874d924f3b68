"""Feed-forward parts of decoders with an fp32 residual stream: a dense one, and routed experts behind a softmax router with a
bias or a router of sigmoid or softmax scores with a correction, with an optional shared expert; the activation is a parameter, gated
(kernels.Glu) or not (kernels.Pointwise).  forward(h) returns what the launch that finishes the residual adds up (kernels.residual_norm takes
one addend, kernels.residual_rms up to two): rows, split-K partials, or weighted expert rows.

Modules take their tensors from `get(name, shape, init)` (harness/weights.py)."""
from __future__ import annotations

from typing import Callable, Union

import torch
from torch import nn

from .. import kernels
from .activation import rows_vectorisable

BF = torch.bfloat16


class DenseMLP(nn.Module):
    """down(act(gate h, up h)) or down(act(up h)), with biases or without."""

    def __init__(self, width: int, ff: int, get: Callable, linear: Callable, bias: bool = True,
                 act: Union[kernels.Glu, kernels.Pointwise] = kernels.SILU):
        super().__init__()
        names = ("gate", "up") if act.gated else ("up",)
        gate_up_b = torch.cat([get(n + ".b", (ff,), "zeros") for n in names], 0) if bias else None
        self.gate_up = linear(torch.cat([get(n, (ff, width)) for n in names], 0), gate_up_b)
        self.down = linear(get("down", (width, ff)), get("down.b", (width,), "zeros") if bias else None)
        self.act = act

    def forward(self, h: torch.Tensor):
        if self.gate_up.streams(h):                     # decode: bias, silu and the product in the weight stream's epilogue
            b = self.gate_up.bias.data if self.gate_up.bias is not None else None
            return self.down.forward_partials(kernels.wstream_gemm(h, self.gate_up.weight.data, b, epilogue="silu_and_mul" if self.act.gated else "none",
                                                                   act=self.act))
        g = self.gate_up(h)
        if not self.act.gated:
            return self.down(kernels.squared_relu_(g))
        if g.dtype == BF and (g.shape[1] // 2) % 8 == 0 and rows_vectorisable(g, g.shape[1]):
            return self.down(kernels.glu_and_mul(g, self.act))
        return self.down(kernels.gate_mul(g, self.act))


class RoutedMLP(nn.Module):
    """`top` of `experts` small gated parts per token plus a shared part every token takes.  scores="softmax": weighted by the softmax over
    the chosen router logits, which have a bias; "sigmoid": sigmoid scores times router.scale, chosen with a correction out of the best
    router.groups.keep of groups.count groups (kernels.SigmoidScores); "softmax_all": the same with the softmax over all experts as the scores
    (kernels.SoftmaxScores).  The last router.identity members of the router are identities: they hand on the input.  shared_gate: the shared
    part counts times the sigmoid of one more row ("shared.sg"), which joins the router's.  act(constants of an expert) is its activation.  The
    experts' rows are padded with zeros to whole matrix tiles (every activation makes nothing of zero columns)."""

    def __init__(self, width: int, m: dict, get: Callable, linear: Callable, scores: str = "softmax",
                 act: Callable[[dict], Union[kernels.Glu, kernels.Pointwise]] = lambda expert: kernels.SILU, shared_gate: bool = False):
        super().__init__()
        r, shared = m["router"], m.get("shared")
        E, self.top, self.identities = r["experts"], r["top"], r.get("identity", 0)
        R, self.shared_gate = E + self.identities, shared_gate and shared is not None
        ff, self.act = m["expert"]["ff"], act(m["expert"])
        if E < 1 or not 1 <= self.top <= R or R + self.shared_gate > 256 or self.top > 64:
            raise ValueError(f"router: {self.top} of {R} experts (at most 64 of 256, a shared part's gate among them)")
        self.router = get("router", (R, width))
        if self.shared_gate:
            self.router = torch.cat([self.router, get("shared.sg", (1, width))], 0)
        self.router = nn.Parameter(self.router.contiguous(), requires_grad=False)
        self.router_bias = self.scores = None
        if scores in ("sigmoid", "softmax_all"):
            groups = r.get("groups") or dict(count=1, keep=1)
            count, keep = groups["count"], groups["keep"]
            if not 1 <= keep <= count or R % count or self.top > keep * (R // count):
                raise ValueError(f"router: {self.top} of {R} experts out of {keep} of {count} groups")
            kind = kernels.SigmoidScores if scores == "sigmoid" else kernels.SoftmaxScores
            self.scores = kind(get("correction", (R,), "zeros").float(), count, keep, r.get("scale", 1.0))
        else:
            self.router_bias = get("router.b", (R,), "zeros").float()
        names = ("gate", "up") if self.act.gated else ("up",)
        pad = -ff % 64 if self.router.dtype == BF else 0
        w13 = torch.zeros((E, len(names) * (ff + pad), width), dtype=self.router.dtype, device=self.router.device)
        w2 = torch.zeros((E, width, ff + pad), dtype=self.router.dtype, device=self.router.device)
        for e in range(E):
            for k, n in enumerate(names):
                w13[e, k * (ff + pad):k * (ff + pad) + ff] = get(f"e{e}.{n}", (ff, width))
            w2[e, :, :ff] = get(f"e{e}.down", (width, ff))
        self.w13, self.w2 = nn.Parameter(w13, requires_grad=False), nn.Parameter(w2, requires_grad=False)
        self.shared = None if shared is None else DenseMLP(width, shared["ff"], lambda n, s, init=None: get("shared." + n, s, init), linear, bias=False,
                                                          act=act(shared))
        self.plain_experts = False          # tests: the form without matrix instructions

    def forward(self, h: torch.Tensor) -> tuple:
        weights, ids, *gate = kernels.moe_route(h, self.router.data, self.router_bias, self.top, self.scores, self.identities, self.shared_gate)
        out = kernels.routed_experts(h, self.w13.data, self.w2.data, ids, self.plain_experts, self.act)
        rows = kernels.ExpertRows(out, weights, ids, h) if self.identities else kernels.ExpertRows(out, weights)
        if self.shared is None:
            return (rows,)
        shared = self.shared(h)                            # (its partials are the last product)
        return rows, kernels.Scaled(shared, gate[0]) if gate else shared
