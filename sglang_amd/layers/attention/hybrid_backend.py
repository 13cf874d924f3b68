"""Attention backend of models that mix latent or grouped-query attention of any sizes with recurrent layers.

Per forward it holds what every mixer needs of the batch: the segments of the packed tokens (none for a decode batch: one
token per request), the request rows (= state slots) and the positions.  Like HipAttnBackend nothing is gathered on the host
per step: the kernels walk req_to_token[req_pool_indices[b], :] and the state slots on the device, so a decode step is
capturable as it is."""
from __future__ import annotations

import torch

from ... import kernels
from .base_attn_backend import AttentionBackend


class HybridAttnBackend(AttentionBackend):
    needs_cpu_seq_lens = True

    def __init__(self, model_runner):
        super().__init__()
        self.device = model_runner.device
        self.req_to_token_pool = model_runner.req_to_token_pool
        self.token_to_kv_pool = model_runner.token_to_kv_pool
        self.state_pool = getattr(model_runner.req_to_token_pool, "state_pool", None)      # (models without recurrent layers)
        self.max_context_len = model_runner.req_to_token_pool.max_context_len
        self.segments = kernels.Segments()
        self._extend = None            # (prefix lengths, extend lengths) of the current extend batch
        self._keys = {}                # window -> kernels.VisibleKeys of the current extend batch
        self._blocks = {}              # (window, group) -> kernels.QueryBlocks of the current extend batch
        self.latent_form = None        # tests: "absorbed" / "expanded" forces the form of every extend
        self.grouped_form = None       # tests: "rows" / "prefill" / "plain" forces the form of grouped-query attention

    # ------------------------------------------------------------------ per-step metadata
    def init_forward_metadata_out_graph(self, forward_batch, in_capture: bool = False):
        mode = forward_batch.forward_mode
        if getattr(mode, "is_target_verify", lambda: False)():
            raise NotImplementedError("a tree of draft tokens cannot be verified here: recurrent layers hold one state per request, and these "
                                      "attention kernels take no tree mask")
        if mode.is_decode() or mode.is_idle():
            self.segments = kernels.Segments()
            return
        self._extend, self._keys, self._blocks = (list(forward_batch.extend_prefix_lens_cpu), list(forward_batch.extend_seq_lens_cpu)), {}, {}
        lens = torch.tensor(forward_batch.extend_seq_lens_cpu, dtype=torch.int64)
        tok_seg = torch.repeat_interleave(torch.arange(len(lens), dtype=torch.int32), lens)
        self.segments = kernels.Segments(tok_seg.to(self.device, non_blocking=True), forward_batch.extend_start_loc.to(torch.int32),
                                         forward_batch.extend_seq_lens.to(torch.int32), int(lens.max()))

    def init_forward_metadata_in_graph(self, forward_batch):
        if forward_batch.forward_mode.is_decode():
            self.segments = kernels.Segments()

    def init_cuda_graph_state(self, max_bs: int, max_num_tokens: int):
        pass

    def get_cuda_graph_seq_len_fill_value(self):
        return 1            # a padded row decodes position 0 in slot 0 / row 0: state starts from zero, one visible key

    # ------------------------------------------------------------------ mixers
    def latent_attention(self, layer, q: torch.Tensor, dkv: torch.Tensor, run_id: int, forward_batch) -> torch.Tensor:
        """q [T, heads * (dim + rot)] and dkv [T, rank + rot] as projected -> values [T, heads * vdim]."""
        cache = self.token_to_kv_pool.get_latent_buffer(run_id)
        kernels.latent_prepare(q, dkv, layer.norm_weight, layer.cos_sin, forward_batch.positions, forward_batch.out_cache_loc, cache,
                               layer.heads, layer.dim, layer.rot_dim, layer.eps)
        return self._latent(layer, q, cache, forward_batch)

    def query_latent_attention(self, layer, p, run_id: int, forward_batch) -> torch.Tensor:
        """p: the projection [query latent | latent | rotated key part], rows or Partials -> values [T, heads * vdim]."""
        cache, pos = self.token_to_kv_pool.get_latent_buffer(run_id), forward_batch.positions
        cq = kernels.latent_down(p, layer.q_norm, layer.norm_weight, layer.cos_sin, pos, forward_batch.out_cache_loc, cache, layer.rot_dim, layer.eps)
        dk = layer.dim + layer.rot_dim
        q, _ = kernels.head_prepare(layer.up_proj.forward_partials(cq), layer.heads, dk, dk, pos, layer.cos_sin, layer.eps, rot_off=layer.dim)
        return self._latent(layer, q, cache, forward_batch)

    def _latent(self, layer, q: torch.Tensor, cache: torch.Tensor, forward_batch) -> torch.Tensor:
        """Turned queries [T, heads * (dim + rot)] over the stored rows -> values [T, heads * vdim]."""
        if forward_batch.forward_mode.is_extend() and self._expanded(layer):
            keys = self._keys.get(layer.window)
            if keys is None:
                keys = self._keys[layer.window] = kernels.VisibleKeys(*self._extend, layer.window, self.device)
            lat = kernels.latent_gather(cache, self.req_to_token_pool.req_to_token, forward_batch.req_pool_indices, keys)
            kv = torch.nn.functional.linear(lat[:, :layer.rank], layer.w_expand)
            return kernels.latent_prefill(q, lat, kv, keys, forward_batch.positions, self.segments, layer.heads, layer.dim, layer.rot_dim,
                                          layer.rank, layer.vdim, layer.window, layer.scale, sinks=layer.sinks)
        T = q.shape[0]
        q3 = q.view(T, layer.heads, layer.dim + layer.rot_dim) if q.is_contiguous() else q.unflatten(1, (layer.heads, layer.dim + layer.rot_dim))
        qc = kernels.head_gemm(q3[:, :, :layer.dim], layer.w_absorb)
        oc = kernels.latent_attention(qc, q3[:, :, layer.dim:], cache, self.req_to_token_pool.req_to_token, forward_batch.req_pool_indices,
                                      forward_batch.positions, self.segments, layer.window, layer.scale, self._splits(layer, T), sinks=layer.sinks)
        return kernels.head_gemm(oc, layer.w_value).view(T, layer.heads * layer.vdim)

    # Extends shorter than this go token by token, like decode batches; longer ones as tiles of query rows.
    PREFILL_MIN_TOKENS = 16

    def grouped_attention(self, layer, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, gate, run_id: int, forward_batch) -> torch.Tensor:
        """q [T, heads * kd], k [T, kv_heads * kd], v [T, kv_heads * vd] and the gate [T, heads * vd] as projected -> gated values
        [T, heads * vd].  A decode step on the matrix form stores its own keys and values on the way."""
        rows = self.token_to_kv_pool.get_kv_rows(run_id)
        if layer.matrix and self.grouped_form != "plain" and forward_batch.forward_mode.is_decode():
            return self._grouped(layer, q, gate, rows, (k, v, forward_batch.out_cache_loc), forward_batch)
        kernels.grouped_kv_store(k, v, rows, forward_batch.out_cache_loc, layer.kv_heads)
        return self._grouped(layer, q, gate, rows, None, forward_batch)

    def prepared_attention(self, layer, p, run_id: int, forward_batch, out=None):
        """p: the projection [queries | keys | values | gate, or columns of a mixer beside], rows or Partials -> gated values [T, heads * vd] (in the
        rows `out` if given), and the columns beside as rows (or None); one launch norms, turns and stores in front of attention."""
        tail = layer.gate_cols + layer.beside_cols
        rows = self.token_to_kv_pool.get_kv_rows(run_id)
        q, gate = kernels.head_prepare(p, layer.heads, layer.dim, layer.kd, forward_batch.positions, layer.cos_sin, layer.eps, norms=layer.norms,
                                       norm_after=layer.norm_after, gate_cols=(tail + 7) // 8 * 8, value_is_key=layer.value_is_key,
                                       kv=(layer.kv_heads, layer.vd, rows, forward_batch.out_cache_loc))
        beside, gate = (gate[:, :tail], None) if layer.beside_cols else (None, gate[:, :tail] if gate is not None else None)
        return self._grouped(layer, q, gate, rows, None, forward_batch, out), beside

    def _grouped(self, layer, q: torch.Tensor, gate, rows: torch.Tensor, new, forward_batch, out=None) -> torch.Tensor:
        """Queries over the stored rows, and over the step's own keys and values `new` of a decode batch that are not stored yet."""
        T, form = q.shape[0], self.grouped_form
        matrix = layer.matrix and form != "plain"
        sizes = (layer.heads, layer.kv_heads, layer.kd, layer.vd, layer.window, layer.scale)
        variant = dict(sink=layer.sink, gate=gate, cap=layer.cap, keep=layer.keep_first, offsets=layer.offsets, out_scale=layer.out_scale, out=out)
        where = (rows, self.req_to_token_pool.req_to_token, forward_batch.req_pool_indices, forward_batch.positions, self.segments)
        if (matrix and layer.prefill and forward_batch.forward_mode.is_extend()
                and (max(self._extend[1]) >= self.PREFILL_MIN_TOKENS if form is None else form == "prefill")):
            key = (layer.window, layer.group)
            if key not in self._blocks:
                self._blocks[key] = kernels.QueryBlocks(*self._extend, layer.window, layer.group, self.device)
            return kernels.grouped_prefill(q, *where, self._blocks[key], *sizes, **variant)
        return kernels.grouped_attention(q, *where, *sizes, new=new, splits=self._grouped_splits(layer, T, matrix),
                                         plain=not matrix, **variant)

    def _grouped_splits(self, layer, tokens: int, matrix: bool) -> int:
        """Workgroups enough for the chip on small batches, never shorter than 128 keys; a function of the batch size and the context
        bound only (fixed inside a captured graph)."""
        keys = min(layer.window + layer.keep_first, self.max_context_len) if layer.window > 0 else self.max_context_len
        groups = layer.kv_heads * ((layer.group + 15) // 16) if matrix else layer.heads
        want = (512 + tokens * groups - 1) // (tokens * groups)
        return max(1, min(want, (keys + 127) // 128, 32))

    def _expanded(self, layer) -> bool:
        """Which form of an extend costs less: per (query, key) pair the absorbed form multiplies 2 rank + rot elements, the
        expanded one dim + rot + vdim, but that one first expands every visible key (a library product: half price)."""
        if layer.w_expand is None or layer.scale <= 0:
            return False
        if self.latent_form is not None:
            return self.latent_form == "expanded"
        if max(self._extend[1]) < 16:
            return False
        w = layer.window if layer.window > 0 else 1 << 40
        pairs = keys = 0
        for p, n in zip(*self._extend):
            grow = max(0, min(n, w - p))                   # queries that still see every key before them
            pairs += grow * p + grow * (grow + 1) // 2 + (n - grow) * w if n > grow else grow * p + grow * (grow + 1) // 2
            keys += n + min(p, w - 1)
        absorbed = pairs * (2 * layer.rank + layer.rot_dim)
        return pairs * (layer.dim + layer.rot_dim + layer.vdim) + keys * (layer.dim + layer.vdim) * layer.rank // 2 < absorbed

    def _splits(self, layer, tokens: int) -> int:
        """Workgroups enough for the chip on small batches, never shorter than 64 keys; a function of the batch size and the
        context bound only (fixed inside a captured graph)."""
        keys = min(layer.window, self.max_context_len) if layer.window > 0 else self.max_context_len
        if layer.w_absorb.dtype == torch.float32:
            groups, fill = layer.heads, 512
        else:                      # a workgroup carries 16 heads, two of them a compute unit -- or 32 heads, one a unit
            groups, fill = ((layer.heads + 15) // 16, 512) if layer.heads <= 16 else ((layer.heads + 31) // 32, 256)
        want = (fill + tokens * groups - 1) // (tokens * groups)
        return max(1, min(want, (keys + 63) // 64, 64))

    def mamba2(self, layer, xbc: torch.Tensor, dt: torch.Tensor, run_id: int, forward_batch) -> torch.Tensor:
        slots, pos = forward_batch.req_pool_indices, forward_batch.positions
        xbc = kernels.causal_conv_silu(xbc, layer.conv_weight, layer.conv_bias, self.state_pool.conv[run_id], slots, pos, self.segments)
        return kernels.mamba2_scan(xbc, dt, layer.A_log, layer.dt_bias, layer.D, self.state_pool.state[run_id], slots, pos, self.segments,
                                   layer.groups)

    def gated_delta(self, layer, qkv: torch.Tensor, b: torch.Tensor, a: torch.Tensor, run_id: int, forward_batch) -> torch.Tensor:
        slots, pos = forward_batch.req_pool_indices, forward_batch.positions
        qkv = kernels.causal_conv_silu(qkv, layer.conv_weight, None, self.state_pool.conv[run_id], slots, pos, self.segments)
        return kernels.gated_delta_scan(qkv, b, a, layer.A_log, layer.dt_bias, self.state_pool.state[run_id], slots, pos, self.segments,
                                        layer.kv_heads, layer.dim ** -0.5)

    def matrix_memory(self, layer, q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, i: torch.Tensor, f: torch.Tensor, run_id: int,
                      forward_batch) -> torch.Tensor:
        pool = self.state_pool
        return kernels.memory_scan(q, k, v, i, f, layer.bias_i, layer.bias_f, pool.state[run_id], pool.norm[run_id], forward_batch.req_pool_indices,
                                   forward_batch.positions, self.segments, layer.cap, layer.dim ** -0.5)

    def token_shift(self, mu: torch.Tensor, layer_id: int, forward_batch):
        """What a launch that norms a batch of single tokens needs to shift them on the way (kernels.TokenShift); other batches: None."""
        if self.segments.start is not None:
            return None
        return kernels.TokenShift(mu, self.state_pool.shift[layer_id], forward_batch.req_pool_indices, forward_batch.positions)

    def shift_rows(self, h: torch.Tensor, mu: torch.Tensor, layer_id: int, forward_batch, out: torch.Tensor) -> torch.Tensor:
        """The token shift of a batch with segments."""
        return kernels.token_shift(h, mu, self.state_pool.shift[layer_id], forward_batch.req_pool_indices, forward_batch.positions, self.segments, out)
