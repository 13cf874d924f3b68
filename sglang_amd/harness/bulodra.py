"""Bulodra: a small decoder with bigram embeddings whose sublayers read the residual stream itself and are normed behind.  Layers mix with
rotary grouped-query attention (biases, norms on queries and keys, a learned sink a head), latent attention with query latents, or
windowed soft-capped attention with a gate a head, in any order; feed-forwards are dense or routed by sigmoid scores within groups of
experts.

One launch between two sublayers sums what the first left (rows, split-K partials, expert rows), norms it, adds it to the fp32
residual and hands the new stream to the next: kernels.residual_rms."""
from __future__ import annotations

from dataclasses import dataclass
from functools import partial
from typing import Any, Dict, List, Optional

import torch
from torch import nn

from .. import kernels
from ..layers.attention.hybrid_backend import HybridAttnBackend
from ..layers.feed_forward import DenseMLP, RoutedMLP
from ..layers.mixers import GroupedAttention, LatentAttention
from ..layers.sampler import LogitsProcessorOutput
from ..mem_cache.memory_pool import LayeredTokenToKVPool, ReqToTokenPool
from .layered import LayeredConfig

BF = torch.bfloat16
MIXERS = {
    "attention": partial(GroupedAttention, bias=True, rotary=True, qk_norm="before", sink="learned"),
    "latent_attention": partial(LatentAttention, q_latent=True, sink=True),
    "attention_2": partial(GroupedAttention, rotary=True, qk_norm="after", gate="heads"),
}
GELU = kernels.Glu("gelu_tanh")
SWISH_ALPHA = 1.702


def expert_activation(expert: dict) -> kernels.Glu:
    return kernels.Glu("clamped_swish", expert["limit"], SWISH_ALPHA)


@dataclass
class BulodraConfig(LayeredConfig):
    residual_mult: float = 1.0
    logit_scale: float = 1.0
    bigram: Optional[Dict[str, int]] = None      # buckets, mul_prev, mul_cur

    @classmethod
    def from_dict(cls, d: Dict[str, Any], name: str = "bulodra") -> "BulodraConfig":
        b = d["embedding"]["bigram"]
        cfg = cls(name, d["vocab"], d["width"], d["layers"], d["norm"]["eps"], None, float(d["residual_mult"]), float(d["logit_scale"]),
                  {k: int(b[k]) for k in ("buckets", "mul_prev", "mul_cur")})
        cfg.check(MIXERS, ("dense", "moe"))
        return cfg


def _sizes(name: str, width: int, heads: int, kv_heads: int, ff: int, experts: int, top: int, expert_ff: int, shared_ff: int, window: int,
           q_rank: int, kv_rank: int, pattern: str) -> BulodraConfig:
    """pattern: two letters a layer, mixer (c capped and windowed, a attention, l latent) and feed-forward (d dense, m routed)."""
    yarn = dict(factor=4.0, original=4096, fast=32.0, slow=1.0)
    mixers = {
        "c": ("attention_2", dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, softcap=30.0, mask=dict(size=window),
                                  rot=dict(base=10000.0, dims=64))),
        "a": ("attention", dict(heads=heads, kv_heads=kv_heads, dim=128, vdim=128, scale=128 ** -0.5, rot=dict(base=500000.0, dims=128, scaling=yarn))),
        "l": ("latent_attention", dict(heads=heads, dim=128, rot_dim=64, vdim=128, kv_rank=kv_rank, q_rank=q_rank, scale=192 ** -0.5,
                                       rot=dict(base=500000.0, dims=64, scaling=yarn))),
    }
    mlps = {"d": dict(kind="dense", ff=ff),
            "m": dict(kind="moe", expert=dict(ff=expert_ff, limit=7.0), shared=dict(ff=shared_ff, limit=7.0),
                      router=dict(experts=experts, top=top, scale=2.5, groups=dict(count=4, keep=2)))}
    layers = [dict(type=mixers[m][0], mixer=mixers[m][1], mlp=mlps[f]) for m, f in pattern.split()]
    return BulodraConfig(name, 32000, width, layers, 1e-6, None, 0.7, 1.0, dict(buckets=65521, mul_prev=31337, mul_cur=8191))


CONFIGS: Dict[str, BulodraConfig] = {
    # sizes that resemble real models' layers, for throughput runs with random weights
    "bulodra-1b": _sizes("bulodra-1b", 2048, 16, 4, 8192, 32, 4, 1024, 2048, 1024, 768, 512, "cd cm am lm cm cd cm am lm cm"),
    "bulodra-8b": _sizes("bulodra-8b", 4096, 32, 8, 14336, 32, 4, 2048, 4096, 4096, 1536, 512, "cd cm am lm cm cd cm am lm cm"),
}


class _Layer(nn.Module):
    def __init__(self, cfg: BulodraConfig, i: int, get, linear, max_positions: int, device):
        super().__init__()
        lay, W = cfg.layers[i], cfg.hidden_size

        def sub(kind):
            return lambda name, shape, init=None: get(f"l{i}.{kind}.{name}", shape, init)

        self.latent = lay["type"] == "latent_attention"
        self.norm1 = get(f"l{i}.norm1", (W,), "ones").float()
        self.mixer = MIXERS[lay["type"]](W, lay["mixer"], cfg.eps, sub("mix"), linear, max_positions, device)
        self.mlp = self.norm2 = None
        m = lay.get("mlp")
        if m is not None:
            self.norm2 = get(f"l{i}.norm2", (W,), "ones").float()
            self.mlp = (RoutedMLP(W, m, sub("mlp"), linear, scores="sigmoid", act=expert_activation) if m["kind"] == "moe"
                        else DenseMLP(W, m["ff"], sub("mlp"), linear, bias=False, act=GELU))


class BulodraForCausalLM(nn.Module):
    supports_prefix_cache = True       # keys, values, latents and the token in front depend on the tokens up to a position alone

    def __init__(self, cfg: BulodraConfig, device, init_device=None, tp_rank: int = 0, tp_size: int = 1, *, weights=None,
                 dtype: torch.dtype = BF, max_context_len: int = 8192):
        super().__init__()
        from .models import Linear
        from .weights import SyntheticWeights

        if tp_size != 1:
            raise NotImplementedError("Bulodra runs on one GPU per replica (tensor parallelism is not built for it)")
        self.config, self.device, self.dtype = cfg, device, dtype
        src = weights if weights is not None else SyntheticWeights(device, dtype, init_device)
        W = cfg.hidden_size
        self.embed_tokens = nn.Parameter(src.get("embed", (cfg.vocab_size, W)), requires_grad=False)
        self.bigram_table = nn.Parameter(src.get("bigram", (cfg.bigram["buckets"] + 1, W)), requires_grad=False)
        self.layers = nn.ModuleList([_Layer(cfg, i, src.get, Linear, max_context_len, device) for i in range(len(cfg.layers))])
        # the factor on the logits rides on the last norm's weights
        self.norm = src.get("final.norm", (W,), "ones").float() * cfg.logit_scale
        self.lm_head = Linear(src.get("head", (cfg.vocab_size, W)))
        src.finish()
        # a run number per kind of cache
        self.runs, self.kv_specs, self.latent_dims = [], [], []
        for layer in self.layers:
            if layer.latent:
                self.runs.append((layer, len(self.latent_dims)))
                self.latent_dims.append(layer.mixer.cache_dim)
            else:
                self.runs.append((layer, len(self.kv_specs)))
                self.kv_specs.append(layer.mixer.cache_spec)
        self.layer_trace: Optional[List[torch.Tensor]] = None     # tests: [] records the residual behind every layer

    # ------------------------------------------------------------------ what ModelRunner builds around a model
    def create_req_to_token_pool(self, size: int, max_context_len: int, device):
        return ReqToTokenPool(size, max_context_len, device)

    def create_kv_pool(self, size: int, page_size: int, kv_cache_dtype: str, device, use_hnd: bool):
        if kv_cache_dtype not in ("auto", "bfloat16", "float32") or use_hnd:
            raise NotImplementedError("the cache is token-major in the model's own type")
        return LayeredTokenToKVPool(size, page_size, self.dtype, self.kv_specs, self.latent_dims, device, keep_tokens=True)

    def create_attn_backend(self, runner):
        return HybridAttnBackend(runner)

    # ------------------------------------------------------------------ forward
    def forward_hidden(self, input_ids: torch.Tensor, positions: torch.Tensor, forward_batch) -> torch.Tensor:
        T, W, eps, m, fb = input_ids.shape[0], self.config.hidden_size, self.config.eps, self.config.residual_mult, forward_batch
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)
        h = torch.empty((T, W), dtype=self.dtype, device=self.device)
        b = self.config.bigram
        pairs = kernels.bigram_rows(input_ids, positions, fb.out_cache_loc, fb.req_to_token_pool.req_to_token, fb.req_pool_indices,
                                    fb.attn_backend.segments.tok_seg, fb.token_to_kv_pool.slot_ids, b["mul_prev"], b["mul_cur"], b["buckets"])
        last = dict(h=h, norm=self.norm)
        kernels.residual_rms(x, eps, embed=(input_ids, self.embed_tokens.data, 1.0), pos=(pairs, self.bigram_table.data),
                             **(dict(h=h) if self.runs else last))
        for k, (layer, run_id) in enumerate(self.runs):
            out = dict(h=h) if k + 1 < len(self.runs) else last
            y = (layer.mixer(h, run_id, fb),)
            kernels.residual_rms(x, eps, add=y, post=(layer.norm1, m), **(out if layer.mlp is None else dict(h=h)))
            if layer.mlp is not None:
                y = layer.mlp(h)
                kernels.residual_rms(x, eps, add=y if isinstance(y, tuple) else (y,), post=(layer.norm2, m), **out)
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
