"""Token mixers beside RadixAttention: latent attention, grouped-query attention with sizes of its own, the gated delta rule, Mamba-2, a
matrix memory with exponential gates, and the last beside attention.  A mixer owns its projections and constants; caches, states and kernel dispatch belong to the attention backend (layers/attention/hybrid_backend.py).

Every module takes its tensors from `get(name, shape, init)` (harness/weights.py) and merges the projections that share an
input into one product, its rows padded to a multiple of 16."""
from __future__ import annotations

import math
from typing import Callable, List, Optional, Union

import torch
from torch import nn

from .. import kernels
from ..mem_cache.memory_pool import StateSpec


def merged_rows(parts: List[torch.Tensor]) -> torch.Tensor:
    """The parts' rows on top of each other, padded with zero rows to a multiple of 16 (whole weight tiles)."""
    rows = sum(p.shape[0] for p in parts)
    pad = -rows % 16
    if pad:
        parts = parts + [torch.zeros((pad, parts[0].shape[1]), dtype=parts[0].dtype, device=parts[0].device)]
    return torch.cat(parts, 0).contiguous()


def conv_taps(w: torch.Tensor) -> torch.Tensor:
    """[channels, taps] with the current token last -> fp32 [taps, channels] with the current token first."""
    return w.float().flip(1).t().contiguous()


def yarn_frequencies(f: torch.Tensor, dims: int, base: float, s: dict):
    """The frequencies f [dims / 2] with the slow ones divided by s['factor'] (YaRN), and the factor on cos and sin.  Pairs that turn more
    than s['fast'] times over s['original'] positions keep theirs, those below s['slow'] turns are divided, a ramp lies between."""
    def pair(turns: float) -> float:
        return dims * math.log(s["original"] / (2.0 * math.pi * turns)) / (2.0 * math.log(base))

    lo, hi = max(math.floor(pair(s["fast"])), 0), min(math.ceil(pair(s["slow"])), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / s["factor"] * ramp + f * (1.0 - ramp), 0.1 * math.log(s["factor"]) + 1.0


def scaled_frequencies(f: torch.Tensor, dims: int, base: float, s: dict):
    """The frequencies under a scaling, and the factor on cos and sin: YaRN, or (no original length) all divided by s['factor']."""
    if "original" in s:
        return yarn_frequencies(f, dims, base, s)
    return f / s["factor"], 1.0


def rotary_table(positions: int, dims: int, base: float, device, scaling: Optional[dict] = None) -> torch.Tensor:
    """fp32 cos | sin of p * base^(-2i / dims), evaluated in double so that far positions keep their angle; `scaling` as in
    scaled_frequencies."""
    f, factor = float(base) ** (-2.0 * torch.arange(dims // 2, dtype=torch.float64) / dims), 1.0
    if scaling is not None:
        f, factor = scaled_frequencies(f, dims, float(base), scaling)
    a = torch.arange(positions, dtype=torch.float64)[:, None] * f[None, :]
    return (torch.cat([a.cos(), a.sin()], 1) * factor).to(torch.float32).contiguous().to(device)


class LatentAttention(nn.Module):
    """Latent attention.  Queries come from the input and turn in neighbouring pairs, or (q_latent) through a normed latent of their own
    (q_rank) and turn by halves; `sink`: a learned score a head in the softmax denominator."""

    def __init__(self, width: int, m: dict, eps: float, get: Callable, linear: Callable, max_positions: int, device, *, q_latent: bool = False,
                 sink: bool = False):
        super().__init__()
        self.heads, self.dim, self.rot_dim, self.vdim, self.rank = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        self.window, self.scale, self.eps = (m.get("mask") or {}).get("size", 0), float(m["scale"]), eps
        dims = m["rot"]["dims"]
        if dims % 2 or dims > self.rot_dim:
            raise ValueError(f"latent attention: {dims} rotated dimensions in a rotated part of {self.rot_dim}")
        H = self.heads
        self.q_rows, self.dkv_rows = H * (self.dim + self.rot_dim), self.rank + self.rot_dim
        self.q_norm = self.up_proj = None
        if q_latent:
            q_rank = m["q_rank"]
            self.in_proj = linear(merged_rows([get("dq", (q_rank, width)), get("dkv", (self.dkv_rows, width))]))
            self.q_norm = get("dq.norm", (q_rank,), "ones").float()
            self.up_proj = linear(merged_rows([get("uq", (self.q_rows, q_rank))]))
        else:
            self.in_proj = linear(merged_rows([get("q", (self.q_rows, width)), get("dkv", (self.dkv_rows, width))]))
        self.sinks = get("sink", (H,)).float() if sink else None
        self.norm_weight = get("dkv.norm", (self.rank,), "ones").float()
        uk = get("uk", (H * self.dim, self.rank))
        self.w_absorb = uk.view(H, self.dim, self.rank).transpose(1, 2).contiguous()       # [H, rank, dim]
        uv = get("uv", (H * self.vdim, self.rank))
        self.w_value = uv.view(H, self.vdim, self.rank).contiguous()
        # long extends expand keys and values per head with one library product; decodes and short extends stay absorbed
        self.w_expand = None
        if uv.dtype == torch.bfloat16 and self.rank % 8 == 0 and kernels.latent_prefill_supported(self.dim, self.rot_dim, self.vdim):
            self.w_expand = torch.cat([uk, uv], 0).contiguous()
        self.o_proj = linear(get("o", (width, H * self.vdim)))
        self.cos_sin = rotary_table(max_positions, dims, m["rot"]["base"], device, m["rot"].get("scaling"))

    @property
    def cache_dim(self) -> int:
        return self.rank + self.rot_dim

    def forward(self, h: torch.Tensor, run_id: int, fb) -> torch.Tensor:
        if self.up_proj is not None:
            return self.o_proj.forward_partials(fb.attn_backend.query_latent_attention(self, self.in_proj.forward_partials(h), run_id, fb))
        p = self.in_proj(h)
        o = fb.attn_backend.latent_attention(self, p[:, :self.q_rows], p[:, self.q_rows:self.q_rows + self.dkv_rows], run_id, fb)
        return self.o_proj.forward_partials(o)


def padded_heads(w: torch.Tensor, heads: int, dim: int, to: int, axis: int) -> torch.Tensor:
    """Zeros behind every head of `dim` rows (axis 0) or columns (axis 1) up to `to`."""
    if dim == to:
        return w
    split = w.unflatten(axis, (heads, dim))
    out = split.new_zeros(split.shape[:axis] + (heads, to) + split.shape[axis + 2:])
    out.narrow(axis + 1, 0, dim).copy_(split)
    return out.flatten(axis, axis + 1)


class GroupedAttention(nn.Module):
    """Grouped-query attention: own key and value widths, an optional sliding window (mask.size, with mask.keep_first first tokens that stay
    visible), an optional soft cap of the scores
    (softcap), an optional sink (a score in the softmax denominator that carries no value: a constant, or "learned", one a head), an
    optional sigmoid gate on the heads' outputs ("elements", or "heads": one number each), biases on queries, keys and values,
    rotation by halves (rot), and an RMS norm a head on queries and keys: "before" the rotation, with weights, or "after" it, without.
    value_is_key: the values are the keys as projected.  offsets: a learned number a head ("pb") joins the scores, and a key's weight is
    their sigmoid instead of the softmax.  Head vectors are padded with zeros to multiples of 8 elements, in the projections and in the cache.

    `beside` are weights of another mixer that reads the same input: their columns follow this one's in the projection.  A mixer that is part
    of another one (out_scale: its factor there) leaves the output projection to it."""

    def __init__(self, width: int, m: dict, eps: float, get: Callable, linear: Callable, max_positions: int, device, *,
                 sink: Union[None, float, str] = None, gate: Optional[str] = None, bias: bool = False, rotary: bool = False,
                 qk_norm: Optional[str] = None, value_is_key: bool = False, offsets: bool = False, beside: Optional[List[torch.Tensor]] = None,
                 out_scale: Optional[float] = None):
        super().__init__()
        self.heads, self.kv_heads, dim, vdim = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        self.keep_first = (m.get("mask") or {}).get("keep_first", 0)
        self.value_is_key, self.out_scale = value_is_key, 1.0 if out_scale is None else float(out_scale)
        if value_is_key and vdim != dim:
            raise ValueError(f"grouped attention: values of {vdim} that are keys of {dim}")
        self.window, self.scale, self.cap, self.eps = (m.get("mask") or {}).get("size", 0), float(m["scale"]), m.get("softcap"), eps
        H, G = self.heads, self.kv_heads
        if H % G:
            raise ValueError(f"grouped attention: {H} query heads over {G} key heads")
        self.kd, self.vd, self.group = dim + -dim % 8, vdim + -vdim % 8, H // G
        self.sink = get("sink", (H,)).float() if sink == "learned" else sink
        self.offsets = get("pb", (H,)).float() if offsets else None
        heads = (("q", H, dim, self.kd), ("k", G, dim, self.kd)) + (() if value_is_key else (("v", G, vdim, self.vd),))
        parts = [padded_heads(get(n, (c * d, width)), c, d, to, 0) for n, c, d, to in heads]
        biases = [padded_heads(get(n + ".b", (c * d,), "zeros")[:, None], c, d, to, 0) for n, c, d, to in heads] if bias else []
        self.gate_cols = {None: 0, "heads": H, "elements": H * self.vd}[gate]
        if gate == "heads":
            parts.append(get("g", (H, width)))
        elif gate == "elements":
            parts.append(padded_heads(get("g", (H * vdim, width)), H, vdim, self.vd, 0))
        if bias and gate is not None:
            biases.append(torch.zeros_like(parts[-1][:, :1]))
        self.beside_cols = sum(w.shape[0] for w in beside or ())
        if self.beside_cols:
            if gate is not None:
                raise ValueError("grouped attention: a gate beside another mixer's columns")
            parts += beside
            biases += [torch.zeros_like(w[:, :1]) for w in beside] if bias else []
        self.in_proj = linear(merged_rows(parts), merged_rows(biases)[:, 0].contiguous()) if bias else linear(merged_rows(parts))
        self.dim, self.cos_sin, self.norms, self.norm_after = dim, None, None, qk_norm == "after"
        if rotary:
            rot = m["rot"]
            if rot["dims"] % 2 or rot["dims"] > dim:
                raise ValueError(f"grouped attention: {rot['dims']} rotated dimensions in heads of {dim}")
            if rot["dims"]:
                self.cos_sin = rotary_table(max_positions, rot["dims"], rot["base"], device, rot.get("scaling"))
        if qk_norm == "before":
            self.norms = tuple(padded_heads(get(n, (dim,), "ones").float(), 1, dim, self.kd, 0) for n in ("q.norm", "k.norm"))
        self.prepared = rotary or qk_norm is not None or value_is_key or self.beside_cols > 0      # a launch between the projection and attention
        o = padded_heads(get("o", (width, H * vdim)), H, vdim, self.vd, 1).contiguous()
        self.o_proj, self.out_weight = (linear(o), None) if out_scale is None else (None, o)
        self.matrix = self.in_proj.weight.dtype == torch.bfloat16 and self.scale > 0 and kernels.grouped_attention_matrix_form(self.kd, self.vd)
        self.prefill = self.matrix and kernels.grouped_prefill_supported(self.kd, self.vd, self.group)

    @property
    def cache_spec(self):
        return self.kv_heads, self.kd, self.vd

    def forward(self, h: torch.Tensor, run_id: int, fb) -> torch.Tensor:
        if self.prepared:
            o, _ = fb.attn_backend.prepared_attention(self, self.in_proj.forward_partials(h), run_id, fb)
            return self.o_proj.forward_partials(o)
        p = self.in_proj(h)
        a = self.heads * self.kd
        b = a + self.kv_heads * self.kd
        c = b + self.kv_heads * self.vd
        gate = p[:, c:c + self.gate_cols] if self.gate_cols else None
        return self.o_proj.forward_partials(fb.attn_backend.grouped_attention(self, p[:, :a], p[:, a:b], p[:, b:c], gate, run_id, fb))


class GatedDelta(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, get: Callable, linear: Callable, max_positions: int, device):
        super().__init__()
        self.heads, self.kv_heads, self.dim, self.vdim, self.taps, self.eps = m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["conv"], eps
        if self.heads % self.kv_heads:
            raise ValueError(f"gated delta rule: {self.heads} value heads over {self.kv_heads} key heads")
        qk, v, H = self.kv_heads * self.dim, self.heads * self.vdim, self.heads
        self.conv_channels, self.v_rows = 2 * qk + v, v
        self.in_proj = linear(merged_rows([get("q", (qk, width)), get("k", (qk, width)), get("v", (v, width)), get("g", (v, width)),
                                           get("b", (H, width)), get("a", (H, width))]))
        self.conv_weight = conv_taps(torch.cat([get(f"{n}.conv", (r, self.taps), "conv") for n, r in (("q", qk), ("k", qk), ("v", v))], 0))
        self.A_log, self.dt_bias = get("A_log", (H,), "decay").float(), get("dt_bias", (H,), "step").float()
        self.norm_weight = get("norm", (self.vdim,), "ones").float()
        self.o_proj = linear(get("o", (width, v)))

    @property
    def state_spec(self):
        return self.heads, self.dim, self.vdim, self.taps, self.conv_channels

    def forward(self, h: torch.Tensor, run_id: int, fb) -> torch.Tensor:
        p = self.in_proj(h)
        c, v, H = self.conv_channels, self.v_rows, self.heads
        o = fb.attn_backend.gated_delta(self, p[:, :c], p[:, c + v:c + v + H], p[:, c + v + H:c + v + 2 * H], run_id, fb)
        return self.o_proj.forward_partials(kernels.gated_rmsnorm(o, p[:, c:c + v], self.norm_weight, H, self.eps, gate_first=False))


class Mamba2(nn.Module):
    def __init__(self, width: int, m: dict, eps: float, get: Callable, linear: Callable, max_positions: int, device):
        super().__init__()
        self.heads, self.vdim, self.state, self.groups, self.taps = m["heads"], m["vdim"], m["state"], m["groups"], m["conv"]
        self.norm_groups, self.eps = m["norm_groups"], eps
        self.inner = self.heads * self.vdim
        if self.heads % self.groups or self.inner % self.norm_groups:
            raise ValueError(f"mamba2: {self.heads} heads in {self.groups} groups, {self.inner} channels in {self.norm_groups} norm groups")
        self.conv_channels = self.inner + 2 * self.groups * self.state
        self.in_proj = linear(merged_rows([get("in", (self.inner + self.conv_channels + self.heads, width))]))
        self.conv_weight = conv_taps(get("conv", (self.conv_channels, self.taps), "conv"))
        self.conv_bias = get("conv.b", (self.conv_channels,), "zeros").float()
        self.A_log, self.dt_bias = get("A_log", (self.heads,), "decay").float(), get("dt_bias", (self.heads,), "step").float()
        self.D = get("D", (self.heads,), "ones").float()
        self.norm_weight = get("norm", (self.inner,), "ones").float()
        self.o_proj = linear(get("o", (width, self.inner)))

    @property
    def state_spec(self):
        return self.heads, self.state, self.vdim, self.taps, self.conv_channels

    def forward(self, h: torch.Tensor, run_id: int, fb) -> torch.Tensor:
        p = self.in_proj(h)
        i, c = self.inner, self.conv_channels
        y = fb.attn_backend.mamba2(self, p[:, i:i + c], p[:, i + c:i + c + self.heads], run_id, fb)
        return self.o_proj.forward_partials(kernels.gated_rmsnorm(y, p[:, :i], self.norm_weight, self.norm_groups, self.eps, gate_first=True))


class MatrixMemory(nn.Module):
    """A matrix memory with exponential gates (mLSTM), read through an RMS norm a head and a sigmoid gate.  It has no projection of its own:
    `parts` are the rows [q | k | v | gate | input gates | forget gates] of the one it shares, `out_weight` goes into a common output
    projection.  out_scale: the factor of its output there (it rides on the norm's weights)."""

    def __init__(self, width: int, m: dict, eps: float, get: Callable, out_scale: float = 1.0):
        super().__init__()
        self.heads, self.dim, self.vdim, self.cap, self.eps = m["heads"], m["dim"], m["vdim"], float(m["gate_cap"]), eps
        H, qk, v = self.heads, self.heads * self.dim, self.heads * self.vdim
        self.parts = [get(n, (rows, width)) for n, rows in (("q", qk), ("k", qk), ("v", v), ("g", v), ("i", H), ("f", H))]
        self.starts = [0, qk, 2 * qk, 2 * qk + v, 2 * qk + 2 * v, 2 * qk + 2 * v + H, 2 * qk + 2 * v + 2 * H]
        self.bias_i, self.bias_f = get("i.b", (H,), "zeros").float(), get("f.b", (H,), "zeros").float()
        self.norm_weight = get("norm", (v,), "ones").float() * out_scale
        self.out_weight = get("o", (width, v))

    @property
    def state_spec(self) -> StateSpec:
        return StateSpec(self.heads, self.dim, self.vdim, norm=True)

    def forward(self, p: torch.Tensor, run_id: int, fb, out: torch.Tensor) -> torch.Tensor:
        q, k, v, g, i, f = (p[:, a:b] for a, b in zip(self.starts, self.starts[1:]))
        o = fb.attn_backend.matrix_memory(self, q, k, v, i, f, run_id, fb)
        return kernels.gated_rmsnorm(o, g, self.norm_weight, self.heads, self.eps, gate_first=False, out=out, sigmoid_gate=True)


class Parallel(nn.Module):
    """Attention and a matrix memory side by side on one input: left_scale * attention + right_scale * memory.  One projection in front of
    both, one behind both: the factors ride on the heads' outputs, which are rounded behind them.  The bias of the output projection is left
    to the launch that sums the residual (out_bias)."""

    def __init__(self, width: int, m: dict, eps: float, get: Callable, linear: Callable, max_positions: int, device, **attention):
        super().__init__()

        def side(name):
            return lambda n, shape, init=None: get(f"{name}.{n}", shape, init)

        ls = float(m["left_scale"])
        self.right = MatrixMemory(width, m["right"], eps, side("right"), float(m["right_scale"]))
        self.left = GroupedAttention(width, m["left"], eps, side("left"), linear, max_positions, device, beside=self.right.parts, out_scale=ls, **attention)
        self.out_bias = side("left")("o.b", (width,), "zeros").float() * ls
        self.right.parts = None                            # (they are in the projection)
        a, b = self.left.out_weight, self.right.out_weight
        self.split, used = a.shape[1], a.shape[1] + b.shape[1]
        self.pad = -used % 8
        self.o_proj = linear(torch.cat([a, b] + ([a.new_zeros((width, self.pad))] if self.pad else []), 1).contiguous())
        self.left.out_weight = self.right.out_weight = None

    @property
    def cache_spec(self):
        return self.left.cache_spec

    @property
    def state_spec(self):
        return self.right.state_spec

    def forward(self, h: torch.Tensor, run_id, fb) -> torch.Tensor:
        """run_id: (of the attention's cache, of the memory's state)."""
        both = (torch.zeros if self.pad else torch.empty)((h.shape[0], self.o_proj.weight.shape[1]), dtype=h.dtype, device=h.device)
        a, b = self.split, both.shape[1] - self.pad
        _, rest = fb.attn_backend.prepared_attention(self.left, self.left.in_proj.forward_partials(h), run_id[0], fb, out=both[:, :a])
        self.right(rest, run_id[1], fb, both[:, a:b])
        return self.o_proj.forward_partials(both)


MIXERS = {"latent_attention": LatentAttention, "delta": GatedDelta, "mamba2": Mamba2}
