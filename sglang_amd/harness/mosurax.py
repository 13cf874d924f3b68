"""Mosurax: a small looped decoder with learned positions.  Every layer is windowed grouped-query attention with a sink and an output
gate in front of a dense or a routed feed-forward; a span of layers runs several times in a row with the same weights, every
pass with its own cache, behind the embedding output and a vector of its own; the residual stream is fp32 with an RMS norm in
front of every sublayer, and the logits are soft-capped.

The model is a list of layer RUNS.  One launch between two sublayers closes the one (residual add) and opens the next (what a
pass adds, input norm): kernels.residual_rms; it also sums the split-K partials of decode projections and the experts' rows."""
from __future__ import annotations

from dataclasses import dataclass
from functools import partial
from typing import Any, Dict, List, Optional

import torch
from torch import nn

from .. import kernels
from ..layers.attention.hybrid_backend import HybridAttnBackend
from ..layers.feed_forward import DenseMLP, RoutedMLP
from ..layers.mixers import GroupedAttention
from ..layers.sampler import LogitsProcessorOutput
from ..mem_cache.memory_pool import GroupedTokenToKVPool, ReqToTokenPool
from .layered import LayeredConfig

BF = torch.bfloat16
MIXERS = {"attention": partial(GroupedAttention, sink=0.0, gate="elements")}


@dataclass
class MosuraxConfig(LayeredConfig):
    max_positions: int = 2048
    logit_softcap: Optional[float] = None

    @classmethod
    def from_dict(cls, d: Dict[str, Any], name: str = "mosurax") -> "MosuraxConfig":
        cfg = cls(name, d["vocab"], d["width"], d["layers"], d["norm"]["eps"], d.get("loop"), d["max_positions"], d.get("logit_softcap"))
        cfg.check(MIXERS, ("dense", "moe"))
        return cfg


def _sizes(name: str, width: int, heads: int, kv_heads: int, ff: int, experts: int, top: int, expert_ff: int, shared_ff: int, window: int,
           pattern: str, loop=None) -> MosuraxConfig:
    mlps = {"d": dict(kind="dense", ff=ff),
            "m": dict(kind="moe", expert=dict(ff=expert_ff), router=dict(experts=experts, top=top), shared=dict(ff=shared_ff))}
    mixer = dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, mask=dict(size=window))
    return MosuraxConfig(name, 32000, width, [dict(type="attention", mixer=mixer, mlp=mlps[c]) for c in pattern], 1e-6, loop, 8192, 30.0)


CONFIGS: Dict[str, MosuraxConfig] = {
    # sizes that resemble real models' layers, for throughput runs with random weights
    "mosurax-1b": _sizes("mosurax-1b", 2048, 16, 4, 8192, 32, 4, 1024, 2048, 1024, "dmdmdm", dict(start=1, stop=5, times=2)),
    "mosurax-8b": _sizes("mosurax-8b", 4096, 32, 8, 14336, 32, 4, 2048, 4096, 4096, "dmdmdm", dict(start=1, stop=5, times=2)),
}


class _Layer(nn.Module):
    def __init__(self, cfg: MosuraxConfig, i: int, get, linear, max_positions: int, device):
        super().__init__()
        lay, W = cfg.layers[i], cfg.hidden_size

        def sub(kind):
            return lambda name, shape, init=None: get(f"l{i}.{kind}.{name}", shape, init)

        self.norm1 = get(f"l{i}.norm1", (W,), "ones").float()
        self.mixer = MIXERS[lay["type"]](W, lay["mixer"], cfg.eps, sub("mix"), linear, max_positions, device)
        self.mlp = self.norm2 = None
        m = lay.get("mlp")
        if m is not None:
            self.norm2 = get(f"l{i}.norm2", (W,), "ones").float()
            self.mlp = RoutedMLP(W, m, sub("mlp"), linear) if m["kind"] == "moe" else DenseMLP(W, m["ff"], sub("mlp"), linear, bias=False)


class MosuraxForCausalLM(nn.Module):
    supports_prefix_cache = True       # keys and values of a position depend on the tokens up to it alone

    def __init__(self, cfg: MosuraxConfig, device, init_device=None, tp_rank: int = 0, tp_size: int = 1, *, weights=None,
                 dtype: torch.dtype = BF, max_context_len: int = 8192):
        super().__init__()
        from .models import Linear
        from .weights import SyntheticWeights

        if tp_size != 1:
            raise NotImplementedError("Mosurax runs on one GPU per replica (tensor parallelism is not built for it)")
        self.config, self.device, self.dtype = cfg, device, dtype
        src = weights if weights is not None else SyntheticWeights(device, dtype, init_device)
        W = cfg.hidden_size
        self.embed_tokens = nn.Parameter(src.get("embed", (cfg.vocab_size, W)), requires_grad=False)
        self.position_table = nn.Parameter(src.get("pos", (cfg.max_positions, W)), requires_grad=False)
        self.layers = nn.ModuleList([_Layer(cfg, i, src.get, Linear, max_context_len, device) for i in range(len(cfg.layers))])
        self.norm = src.get("final.norm", (W,), "ones").float()
        self.lm_head = Linear(src.get("head", (cfg.vocab_size, W)))
        self.loop_step = src.get("loop.step", (cfg.loop["times"], W)).float().contiguous() if cfg.loop is not None else None
        src.finish()
        # one cache per RUN of a layer
        self.runs = [(self.layers[i], run_id, t) for run_id, (i, t) in enumerate(cfg.runs())]
        self.layer_trace: Optional[List[torch.Tensor]] = None     # tests: [] records the residual behind every run

    # ------------------------------------------------------------------ what ModelRunner builds around a model
    def create_req_to_token_pool(self, size: int, max_context_len: int, device):
        return ReqToTokenPool(size, min(max_context_len, self.config.max_positions), device)

    def create_kv_pool(self, size: int, page_size: int, kv_cache_dtype: str, device, use_hnd: bool):
        if kv_cache_dtype not in ("auto", "bfloat16", "float32") or use_hnd:
            raise NotImplementedError("the cache is token-major in the model's own type")
        return GroupedTokenToKVPool(size, page_size, self.dtype, [layer.mixer.cache_spec for layer, _, _ in self.runs], device)

    def create_attn_backend(self, runner):
        return HybridAttnBackend(runner)

    # ------------------------------------------------------------------ forward
    def forward_hidden(self, input_ids: torch.Tensor, positions: torch.Tensor, forward_batch) -> torch.Tensor:
        T, W, eps = input_ids.shape[0], self.config.hidden_size, self.config.eps
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)
        h = torch.empty((T, W), dtype=self.dtype, device=self.device)
        again = any(t for _, _, t in self.runs)            # some pass is not the first: it needs the embedding output
        x0 = torch.empty_like(x) if again else None

        def opening(k: int) -> dict:
            """What the launch that finishes the residual in front of run k also does: a pass's additions, the run's input norm (or the
            final norm)."""
            if k == len(self.runs):
                return dict(norm=self.norm, h=h)
            layer, _, t = self.runs[k]
            return dict(norm=layer.norm1, h=h, extra=x0 if t else None, step=self.loop_step[t] if t is not None else None)

        kernels.residual_rms(x, eps, embed=(input_ids, self.embed_tokens.data, 1.0), pos=(positions, self.position_table.data), save=x0, **opening(0))
        for k, (layer, run_id, _) in enumerate(self.runs):
            y = (layer.mixer(h, run_id, forward_batch),)
            if layer.mlp is not None:
                kernels.residual_rms(x, eps, add=y, norm=layer.norm2, h=h)
                y = layer.mlp(h)
                y = y if isinstance(y, tuple) else (y,)
            if self.layer_trace is not None:
                kernels.residual_rms(x, eps, add=y)
                self.layer_trace.append(x.clone())
                y = ()
            kernels.residual_rms(x, eps, add=y, **opening(k + 1))
        return h

    def compute_logits(self, hidden: torch.Tensor, forward_batch) -> LogitsProcessorOutput:
        rows = forward_batch.logits_rows
        if rows is not None:
            hidden = hidden[rows]
        elif forward_batch.forward_mode.is_extend():
            hidden = hidden[torch.cumsum(forward_batch.extend_seq_lens, dim=0, dtype=torch.int64) - 1]
        if hidden.shape[0] == 0:
            return LogitsProcessorOutput(next_token_logits=hidden.new_empty((0, self.config.vocab_size)))
        cap = self.config.logit_softcap
        return LogitsProcessorOutput(next_token_logits=kernels.soft_cap(self.lm_head.forward_partials(hidden), cap) if cap else self.lm_head(hidden))

    def forward(self, input_ids: torch.Tensor, positions: torch.Tensor, forward_batch) -> LogitsProcessorOutput:
        return self.compute_logits(self.forward_hidden(input_ids, positions, forward_batch), forward_batch)
