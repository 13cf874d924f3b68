"""Dugalix: a small decoder whose mixers read a blend of every token with the one in front.  Layers mix with windowed attention whose weights
are sigmoids of the scores and whose values are the keys, or with windowed softmax attention that keeps the first tokens beside a matrix
memory with exponential gates; feed-forwards are squared-relu layers, dense or routed among experts and identities with a gated
shared part.  Every sublayer is normed in front and behind; norm weights are stored around zero.

One launch between two sublayers sums what the first left (rows, split-K partials, expert rows, input rows), norms it, adds it to the fp32
residual and norms that for the next: kernels.residual_rms.  In decode batches it also blends the row with the one in front, which it
takes from the request's state; batches with longer portions take a launch for that (kernels.token_shift)."""
from __future__ import annotations

from dataclasses import dataclass
from functools import partial
from typing import Any, Dict, List, Optional

import torch
from torch import nn

from .. import kernels
from ..layers.attention.hybrid_backend import HybridAttnBackend
from ..layers.feed_forward import DenseMLP, RoutedMLP
from ..layers.mixers import GroupedAttention, Parallel
from ..layers.sampler import LogitsProcessorOutput
from ..mem_cache.memory_pool import GroupedTokenToKVPool, HybridReqToTokenPool
from .layered import LayeredConfig

BF = torch.bfloat16
MIXERS = {
    "attention": partial(GroupedAttention, rotary=True, value_is_key=True, offsets=True),
    "parallel": partial(Parallel, rotary=True, bias=True),
}
SQUARED_RELU = kernels.Pointwise("squared_relu")


@dataclass
class DugalixConfig(LayeredConfig):
    residual_mult: float = 1.0

    @classmethod
    def from_dict(cls, d: Dict[str, Any], name: str = "dugalix") -> "DugalixConfig":
        cfg = cls(name, d["vocab"], d["width"], d["layers"], d["norm"]["eps"], None, float(d["residual_mult"]))
        cfg.check(MIXERS, ("dense", "moe"))
        return cfg


def _sizes(name: str, width: int, heads: int, kv_heads: int, ff: int, experts: int, top: int, expert_ff: int, shared_ff: int, window: int,
           memory_heads: int, pattern: str) -> DugalixConfig:
    """pattern: two letters a layer, mixer (a sigmoid attention, p parallel) and feed-forward (d dense, m routed)."""
    mixers = {
        "a": ("attention", dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, mask=dict(size=window),
                                rot=dict(base=500000.0, dims=64))),
        "p": ("parallel", dict(left=dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, mask=dict(size=window, keep_first=4),
                                         rot=dict(base=500000.0, dims=128, scaling=dict(factor=8.0))),
                               right=dict(heads=memory_heads, dim=128, vdim=128, gate_cap=15.0), left_scale=0.7, right_scale=0.7)),
    }
    mlps = {"d": dict(kind="dense", ff=ff),
            "m": dict(kind="moe", expert=dict(ff=expert_ff), shared=dict(ff=shared_ff),
                      router=dict(experts=experts, identity=8, top=top, groups=dict(count=4, keep=2)))}
    layers = [dict(type=mixers[m][0], mixer=mixers[m][1], mlp=mlps[f]) for m, f in pattern.split()]
    return DugalixConfig(name, 32000, width, layers, 1e-6, None, 0.7)


CONFIGS: Dict[str, DugalixConfig] = {
    # sizes that resemble real models' layers, for throughput runs with random weights
    "dugalix-1b": _sizes("dugalix-1b", 2048, 16, 4, 12288, 32, 4, 1536, 3072, 1024, 8, "ad pm am pm ad pm am pm am pm"),
    "dugalix-8b": _sizes("dugalix-8b", 4096, 32, 8, 21504, 32, 4, 3072, 6144, 4096, 16, "ad pm am pm ad pm am pm am pm"),
}


class _Layer(nn.Module):
    def __init__(self, cfg: DugalixConfig, i: int, get, linear, max_positions: int, device):
        super().__init__()
        lay, W = cfg.layers[i], cfg.hidden_size

        def sub(kind):
            return lambda name, shape, init=None: get(f"l{i}.{kind}.{name}", shape, init)

        def norm(name):
            return 1.0 + get(f"l{i}.{name}", (W,), "zeros").float()

        self.recurrent = lay["type"] == "parallel"
        self.shift = get(f"l{i}.shift", (W,), "zeros").float()
        self.norm1, self.norm1b = norm("norm1"), norm("norm1b")
        self.mixer = MIXERS[lay["type"]](W, lay["mixer"], cfg.eps, sub("mix"), linear, max_positions, device)
        self.out_bias = getattr(self.mixer, "out_bias", None)
        self.mlp = self.norm2 = self.norm2b = None
        m = lay.get("mlp")
        if m is not None:
            self.norm2, self.norm2b = norm("norm2"), norm("norm2b")
            self.mlp = (RoutedMLP(W, m, sub("mlp"), linear, scores="softmax_all", act=lambda expert: SQUARED_RELU, shared_gate=True)
                        if m["kind"] == "moe" else DenseMLP(W, m["ff"], sub("mlp"), linear, bias=False, act=SQUARED_RELU))


class DugalixForCausalLM(nn.Module):
    supports_prefix_cache = False      # a recurrent state cannot be rewound to a shared prefix

    def __init__(self, cfg: DugalixConfig, device, init_device=None, tp_rank: int = 0, tp_size: int = 1, *, weights=None,
                 dtype: torch.dtype = BF, max_context_len: int = 8192):
        super().__init__()
        from .models import Linear
        from .weights import SyntheticWeights

        if tp_size != 1:
            raise NotImplementedError("Dugalix runs on one GPU per replica (tensor parallelism of its recurrent layers is not built)")
        self.config, self.device, self.dtype = cfg, device, dtype
        src = weights if weights is not None else SyntheticWeights(device, dtype, init_device)
        W = cfg.hidden_size
        self.embed_tokens = nn.Parameter(src.get("embed", (cfg.vocab_size, W)), requires_grad=False)
        self.layers = nn.ModuleList([_Layer(cfg, i, src.get, Linear, max_context_len, device) for i in range(len(cfg.layers))])
        self.norm = 1.0 + src.get("final.norm", (W,), "zeros").float()
        self.lm_head = Linear(src.get("head", (cfg.vocab_size, W)))
        src.finish()
        # every layer has a cache; those with a memory a state of their own number beside it
        self.runs, self.kv_specs, self.state_specs = [], [], []
        for i, layer in enumerate(self.layers):
            self.runs.append((layer, (i, len(self.state_specs)) if layer.recurrent else i))
            self.kv_specs.append(layer.mixer.cache_spec)
            if layer.recurrent:
                self.state_specs.append(layer.mixer.state_spec)
        self.layer_trace: Optional[List[torch.Tensor]] = None     # tests: [] records the residual behind every layer

    # ------------------------------------------------------------------ what ModelRunner builds around a model
    def create_req_to_token_pool(self, size: int, max_context_len: int, device):
        return HybridReqToTokenPool(size, max_context_len, device, self.state_specs, self.dtype, [self.config.hidden_size] * len(self.layers))

    def create_kv_pool(self, size: int, page_size: int, kv_cache_dtype: str, device, use_hnd: bool):
        if kv_cache_dtype not in ("auto", "bfloat16", "float32") or use_hnd:
            raise NotImplementedError("the cache is token-major in the model's own type")
        return GroupedTokenToKVPool(size, page_size, self.dtype, self.kv_specs, device)

    def create_attn_backend(self, runner):
        return HybridAttnBackend(runner)

    # ------------------------------------------------------------------ forward
    def forward_hidden(self, input_ids: torch.Tensor, positions: torch.Tensor, forward_batch) -> torch.Tensor:
        T, W, eps, m, fb = input_ids.shape[0], self.config.hidden_size, self.config.eps, self.config.residual_mult, forward_batch
        backend = fb.attn_backend
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)
        h = torch.empty((T, W), dtype=self.dtype, device=self.device)
        blended = torch.empty_like(h) if backend.segments.start is not None else None

        def opening(k: int) -> dict:
            """What the launch that finishes the residual in front of layer k also produces."""
            if k == len(self.runs):
                return dict(h=h, norm=self.norm)
            layer = self.runs[k][0]
            return dict(h=h, norm=layer.norm1, shift=backend.token_shift(layer.shift, k, fb))

        kernels.residual_rms(x, eps, embed=(input_ids, self.embed_tokens.data, 1.0), **opening(0))
        for k, (layer, run_id) in enumerate(self.runs):
            mixed = h if blended is None else backend.shift_rows(h, layer.shift, k, fb, blended)
            y = (layer.mixer(mixed, run_id, fb),)
            after = opening(k + 1)
            if layer.mlp is None:
                kernels.residual_rms(x, eps, add=y, bias=layer.out_bias, post=(layer.norm1b, m), **after)
            else:
                kernels.residual_rms(x, eps, add=y, bias=layer.out_bias, post=(layer.norm1b, m), h=h, norm=layer.norm2)
                y = layer.mlp(h)
                kernels.residual_rms(x, eps, add=y if isinstance(y, tuple) else (y,), post=(layer.norm2b, m), **after)
            if self.layer_trace is not None:
                self.layer_trace.append(x.clone())
        return h

    def compute_logits(self, hidden: torch.Tensor, forward_batch) -> LogitsProcessorOutput:
        rows = forward_batch.logits_rows
        if rows is not None:
            hidden = hidden[rows]
        elif forward_batch.forward_mode.is_extend():
            hidden = hidden[torch.cumsum(forward_batch.extend_seq_lens, dim=0, dtype=torch.int64) - 1]
        if hidden.shape[0] == 0:
            return LogitsProcessorOutput(next_token_logits=hidden.new_empty((0, self.config.vocab_size)))
        return LogitsProcessorOutput(next_token_logits=self.lm_head(hidden))

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, forward_batch) -> LogitsProcessorOutput:
        return self.compute_logits(self.forward_hidden(input_ids, positions, forward_batch), forward_batch)
