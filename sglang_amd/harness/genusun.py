"""Genusun: a small hybrid decoder.  Layers mix with windowed latent attention, a gated delta rule or Mamba-2, in any order;
a span of layers runs several times in a row with the same weights, every pass with its own cache and state; the residual
stream is fp32 with a layer norm in front of and behind every sublayer.

The model is a list of layer RUNS.  One launch between two sublayers closes the one (norm of its output, residual add) and
opens the next (its input norm): kernels.residual_norm; in decode batches it also sums the projection's split-K partials."""
from __future__ import annotations

from dataclasses import dataclass
from typing import Any, Dict, List, Optional

import torch
from torch import nn

from .. import kernels
from ..layers.attention.hybrid_backend import HybridAttnBackend
from ..layers.feed_forward import DenseMLP
from ..layers.mixers import MIXERS
from ..layers.sampler import LogitsProcessorOutput
from ..mem_cache.memory_pool import HybridReqToTokenPool, LatentTokenToKVPool
from .layered import LayeredConfig

BF = torch.bfloat16


@dataclass
class GenusunConfig(LayeredConfig):
    embedding_scale: float = 1.0

    @classmethod
    def from_dict(cls, d: Dict[str, Any], name: str = "genusun") -> "GenusunConfig":
        cfg = cls(name, d["vocab"], d["width"], d["layers"], d["norm"]["eps"], d.get("loop"), d["embedding"]["scale"])
        cfg.check(MIXERS, ("dense",))
        return cfg


def _sizes(name: str, width: int, vocab: int, ff: int, heads: int, mamba_heads: int, delta_heads: int, rank: int, window: int,
           pattern: str, loop=None) -> GenusunConfig:
    mixers = {
        "m": dict(type="mamba2", mlp=None, mixer=dict(heads=mamba_heads, vdim=64, state=128, groups=8, norm_groups=8, conv=4)),
        "d": dict(type="delta", mlp=None, mixer=dict(heads=delta_heads, kv_heads=delta_heads // 2, dim=128, vdim=128, conv=4)),
        "a": dict(type="latent_attention", mlp=dict(kind="dense", ff=ff),
                  mixer=dict(heads=heads, dim=128, rot_dim=64, vdim=128, kv_rank=rank, scale=192 ** -0.5, mask=dict(size=window),
                             rot=dict(base=10000.0, dims=64))),
    }
    return GenusunConfig(name, vocab, width, [mixers[c] for c in pattern], 1e-6, loop, width ** 0.5)


CONFIGS: Dict[str, GenusunConfig] = {
    # sizes that resemble real models' layers, for throughput runs with random weights
    "genusun-1b": _sizes("genusun-1b", 2048, 32000, 8192, 16, 64, 16, 512, 1024, "mmamdm", dict(start=1, stop=4, times=2)),
    "genusun-8b": _sizes("genusun-8b", 4096, 32000, 14336, 32, 128, 32, 512, 4096, "mmamdm", dict(start=1, stop=4, times=2)),
}


class _Norm(nn.Module):
    """Layer-norm parameters in fp32; applied by kernels.residual_norm."""

    def __init__(self, get, name: str, width: int):
        super().__init__()
        self.weight, self.bias = get(name, (width,), "ones").float(), get(name + ".b", (width,), "zeros").float()

    @property
    def wb(self):
        return self.weight, self.bias


class _Layer(nn.Module):
    def __init__(self, cfg: GenusunConfig, i: int, get, linear, max_positions: int, device):
        super().__init__()
        lay, W = cfg.layers[i], cfg.hidden_size

        def sub(kind):
            return lambda name, shape, init=None: get(f"l{i}.{kind}.{name}", shape, init)

        self.kind = lay["type"]
        self.norm1, self.norm1b = _Norm(get, f"l{i}.norm1", W), _Norm(get, f"l{i}.norm1b", W)
        self.mixer = MIXERS[lay["type"]](W, lay["mixer"], cfg.eps, sub("mix"), linear, max_positions, device)
        self.mlp = None
        if lay.get("mlp") is not None:
            self.norm2, self.norm2b = _Norm(get, f"l{i}.norm2", W), _Norm(get, f"l{i}.norm2b", W)
            self.mlp = DenseMLP(W, lay["mlp"]["ff"], sub("mlp"), linear)


class GenusunForCausalLM(nn.Module):
    supports_prefix_cache = False      # a recurrent state cannot be rewound to a shared prefix

    def __init__(self, cfg: GenusunConfig, device, init_device=None, tp_rank: int = 0, tp_size: int = 1, *, weights=None,
                 dtype: torch.dtype = BF, max_context_len: int = 8192):
        super().__init__()
        from .models import Linear
        from .weights import SyntheticWeights

        if tp_size != 1:
            raise NotImplementedError("Genusun runs on one GPU per replica (tensor parallelism of its recurrent layers is not built)")
        self.config, self.device, self.dtype = cfg, device, dtype
        src = weights if weights is not None else SyntheticWeights(device, dtype, init_device)
        W = cfg.hidden_size
        self.embed_tokens = nn.Parameter(src.get("embed", (cfg.vocab_size, W)), requires_grad=False)
        self.layers = nn.ModuleList([_Layer(cfg, i, src.get, Linear, max_context_len, device) for i in range(len(cfg.layers))])
        self.norm = _Norm(src.get, "final.norm", W)
        self.lm_head = Linear(src.get("head", (cfg.vocab_size, W)))
        self.loop_in = self.loop_step = None
        if cfg.loop is not None:
            self.loop_in = Linear(src.get("loop.in", (W, 2 * W)))
            self.loop_step = src.get("loop.step", (cfg.loop["times"], W)).float().contiguous()
        src.finish()
        # one cache / state per RUN of a layer
        self.runs, self.latent_dims, self.state_specs = [], [], []
        for i, t in cfg.runs():
            layer = self.layers[i]
            if layer.kind == "latent_attention":
                self.runs.append((layer, len(self.latent_dims), t))
                self.latent_dims.append(layer.mixer.cache_dim)
            else:
                self.runs.append((layer, len(self.state_specs), t))
                self.state_specs.append(layer.mixer.state_spec)
        self.layer_trace: Optional[List[torch.Tensor]] = None     # tests: [] records the residual behind every run

    # ------------------------------------------------------------------ what ModelRunner builds around a model
    def create_req_to_token_pool(self, size: int, max_context_len: int, device):
        return HybridReqToTokenPool(size, max_context_len, device, self.state_specs, self.dtype)

    def create_kv_pool(self, size: int, page_size: int, kv_cache_dtype: str, device, use_hnd: bool):
        if kv_cache_dtype not in ("auto", "bfloat16", "float32") or use_hnd:
            raise NotImplementedError("the latent cache is token-major in the model's own type")
        return LatentTokenToKVPool(size, page_size, self.dtype, self.latent_dims, device)

    def create_attn_backend(self, runner):
        return HybridAttnBackend(runner)

    # ------------------------------------------------------------------ forward
    def forward_hidden(self, input_ids: torch.Tensor, positions: torch.Tensor, forward_batch) -> torch.Tensor:
        T, W, eps = input_ids.shape[0], self.config.hidden_size, self.config.eps
        x = torch.empty((T, W), dtype=torch.float32, device=self.device)
        h = torch.empty((T, W), dtype=self.dtype, device=self.device)
        both = torch.empty((T, 2 * W), dtype=self.dtype, device=self.device) if self.loop_in is not None else None

        def opening(k: int) -> dict:
            """What the launch that finishes the residual in front of run k also produces: the run's input norm, the residual
            copy for a pass that begins there, or the final norm."""
            if k == len(self.runs):
                return dict(norm=self.norm.wb, h=h)
            layer, _, t = self.runs[k]
            return dict(norm=layer.norm1.wb, h=h) if t is None else dict(copies=(both[:, :W], None))

        first = opening(0)
        if both is not None:
            first["copies"] = (first.get("copies", (None,))[0], both[:, W:])
        kernels.residual_norm(x, eps, embed=(input_ids, self.embed_tokens.data, self.config.embedding_scale), **first)
        for k, (layer, run_id, t) in enumerate(self.runs):
            if t is not None:
                kernels.residual_norm(x, eps, start=(self.loop_in.forward_partials(both), self.loop_step[t]), norm=layer.norm1.wb, h=h)
            y = layer.mixer(h, run_id, forward_batch)
            if layer.mlp is not None:
                kernels.residual_norm(x, eps, add=(y, *layer.norm1b.wb), norm=layer.norm2.wb, h=h)
                y = layer.mlp(h)
                kernels.residual_norm(x, eps, add=(y, *layer.norm2b.wb), **opening(k + 1))
            else:
                kernels.residual_norm(x, eps, add=(y, *layer.norm1b.wb), **opening(k + 1))
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
