"""Throughput of the layered designs (Genusun here, Mosurax with grouped_bench.py, Bulodra with layered_bench.py, Dugalix with
shifted_bench.py) beside the closest decoders of this framework at equal size, and every kernel of a design against its roofline beside the like kernel of such a decoder.  Run through
`bench.py --hybrid`; random weights.

The decoder beside it has the same width, feed-forward width, vocabulary and number of attention heads and as many layers as the
design executes layer runs.  One JSON line: prompt tokens / s of cold prefills, tokens / s of graph-replayed decode steps, and a
kernel table (us, fraction of the roofline: 8 TB/s HBM, 2.5 PFLOP/s bf16, 157 TFLOP/s fp32 matrix)."""
from __future__ import annotations

import json
import sys
import time

import torch

HBM, BF16_PEAK, F32_PEAK = 8.0e12, 2.5e15, 157.3e12


def _graph_us(fns, replays=5):
    """Microseconds per launch of fns (each over its own buffers), captured back to back and replayed."""
    for f in fns:
        f()
    torch.cuda.synchronize()
    st = torch.cuda.Stream()
    st.wait_stream(torch.cuda.current_stream())
    with torch.cuda.stream(st):
        g = torch.cuda.CUDAGraph()
        with torch.cuda.graph(g, stream=st):
            for f in fns:
                f()
    torch.cuda.synchronize()
    g.replay()
    best = 1e30
    for _ in range(replays):
        a, b = torch.cuda.Event(enable_timing=True), torch.cuda.Event(enable_timing=True)
        a.record()
        g.replay()
        b.record()
        b.synchronize()
        best = min(best, a.elapsed_time(b) * 1e3)
    return best / len(fns)


def _entry(us, nbytes=0.0, bf16=0.0, f32=0.0):
    floor = max(nbytes / HBM, bf16 / BF16_PEAK, f32 / F32_PEAK) * 1e6
    bound = "hbm" if floor == nbytes / HBM * 1e6 else ("mfma bf16" if floor == bf16 / BF16_PEAK * 1e6 else "mfma fp32")
    return dict(us=round(us, 1), roofline=round(floor / us, 3), bound=bound)


def _llama_beside(cfg):
    from sglang_amd.harness.models import ModelConfig

    att = next(lay for lay in cfg.layers if lay["type"] == "latent_attention")
    return ModelConfig(f"decoder-beside-{cfg.name}", cfg.hidden_size, att["mlp"]["ff"], cfg.num_hidden_layers, att["mixer"]["heads"],
                       max(1, att["mixer"]["heads"] // 4), 128, cfg.vocab_size, 1e-5, 10000.0, None, 8192)


def throughput(cfg, device, prompts, length, batch, ctx, steps=32):
    from sglang_amd.harness.engine import Engine, ModelRunner, Req

    r = ModelRunner(cfg, max_total_tokens=max(prompts * (length + 8), batch * (ctx + steps + 80)), max_running_requests=batch,
                    max_context_len=max(length, ctx + steps + 64) + 64, device=device, use_graph=True, strict_graph=True, graph_max_bs=batch,
                    disable_radix_cache=True)
    eng = Engine(r)
    g = torch.Generator().manual_seed(0)

    def make(n, m, new):
        return [Req(i, torch.randint(0, cfg.vocab_size, (m,), generator=g).tolist(), new) for i in range(n)]

    def prefill(reqs):
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        eng.prefill(reqs)
        torch.cuda.synchronize()
        return time.perf_counter() - t0

    best = 1e30
    for k in range(4):
        reqs = make(prompts, length, 1)
        dt = prefill(reqs)
        best = min(best, dt) if k else best
        eng.finish(reqs)
    reqs = make(batch, ctx, steps + 40)
    for i in range(0, batch, 8):
        eng.prefill(reqs[i:i + 8])
    for _ in range(6):
        eng.decode_step()
    torch.cuda.synchronize()
    t0 = time.perf_counter()
    for _ in range(steps):
        eng.decode_step()
    torch.cuda.synchronize()
    step = (time.perf_counter() - t0) / steps
    eng.finish(list(eng.running))
    params = sum(p.numel() for p in r.model.parameters())
    out = dict(prefill_tokens_per_s=round(prompts * length / best), prefill_ms=round(best * 1e3, 2), decode_tokens_per_s=round(batch / step),
               decode_ms=round(step * 1e3, 3), weight_gb=round(params * 2 / 1e9, 2))
    del eng, r
    torch.cuda.empty_cache()
    return out


def kernel_table(cfg, device, T=8192, segs=4, B=64, ctx=1024):
    """The design's kernels at this model's layer sizes: T prompt tokens in `segs` requests, and decode steps of B requests."""
    from sglang_amd import kernels as K

    bf = torch.bfloat16
    rnd = lambda *s, dtype=bf: (torch.randn(*s, device=device) * 0.5).to(dtype)
    W = cfg.hidden_size
    L = {lay["type"]: lay["mixer"] for lay in cfg.layers}
    ff = next(lay["mlp"]["ff"] for lay in cfg.layers if lay.get("mlp"))
    n = T // segs
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)
    seg = K.Segments(torch.repeat_interleave(torch.arange(segs, dtype=torch.int32, device=device), n), i32([i * n for i in range(segs)]),
                     i32([n] * segs), n)
    pos = torch.arange(n, device=device).repeat(segs)
    slots = torch.arange(1, segs + 1, device=device)
    dslots, dpos = torch.arange(1, B + 1, device=device), torch.full((B,), ctx - 1, device=device)
    pre, dec = {}, {}
    C = 4                                              # copies: the working set of a repeated launch leaves the caches
    ones, zeros = torch.ones(W, device=device), torch.zeros(W, device=device)

    def residual(rows, copies):
        bufs = [(torch.randn(rows, W, device=device), rnd(rows, W), torch.empty(rows, W, dtype=bf, device=device)) for _ in range(copies)]
        us = _graph_us([lambda b=b: K.residual_norm(b[0], 1e-6, add=(b[1], ones, zeros), norm=(ones, zeros), h=b[2]) for b in bufs])
        return _entry(us, rows * W * 12)

    pre["residual_norm"], dec["residual_norm"] = residual(T, C), residual(B, 64)
    m = L["mamba2"]
    H, P, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    ch, inner = H * P + 2 * G * N, H * P
    A, dtb, D = torch.randn(H, device=device) * 0.3, torch.zeros(H, device=device) - 3, torch.ones(H, device=device)
    cw, cb = torch.randn(m["conv"], ch, device=device), torch.zeros(ch, device=device)
    conv = torch.zeros(B + 1, m["conv"], ch, dtype=bf, device=device)
    proj = [rnd(T, inner + ch + H) for _ in range(C)]
    pre["causal_conv_silu"] = _entry(_graph_us([lambda p=p: K.causal_conv_silu(p[:, inner:inner + ch], cw, cb, conv, slots, pos, seg) for p in proj]), T * ch * 4)
    xbc = [rnd(T, ch) for _ in range(C)]
    st = torch.zeros(B + 1, H, N, P, device=device)
    q = 32
    fl = T * H * (4 * N * P + 1.5 * q * N / 2 + 1.5 * q * P / 2)      # the recurrence's own products in 32-token chunks
    pre["mamba2_chunk"] = _entry(_graph_us([lambda x=x, p=p: K.mamba2_scan(x, p[:, inner + ch:], A, dtb, D, st, slots, pos, seg, G) for x, p in zip(xbc, proj)]),
                                 T * (ch + inner + H) * 2, f32=fl)
    y, nw = rnd(T, inner), torch.ones(inner, device=device)
    pre["gated_rmsnorm (mamba2)"] = _entry(_graph_us([lambda p=p: K.gated_rmsnorm(y, p[:, :inner], nw, m["norm_groups"], 1e-6, True) for p in proj]), T * inner * 6)
    sts = [torch.zeros(B + 1, H, N, P, device=device) for _ in range(2)]
    dproj = rnd(B, inner + ch + H)
    s0 = K.Segments()
    dec["causal_conv_silu"] = _entry(_graph_us([lambda: K.causal_conv_silu(dproj[:, inner:inner + ch], cw, cb, conv, dslots, dpos, s0)] * 32),
                                     B * ch * (4 + 2 * m["conv"]))
    dx = rnd(B, ch)
    dec["mamba2_step"] = _entry(_graph_us([lambda s=s: K.mamba2_scan(dx, dproj[:, inner + ch:], A, dtb, D, s, dslots, dpos, s0, G) for s in sts * 4]),
                                B * H * N * P * 8)
    dec["gated_rmsnorm (mamba2)"] = _entry(_graph_us([lambda: K.gated_rmsnorm(dx[:, :inner], dproj[:, :inner], nw, m["norm_groups"], 1e-6, True)] * 32), B * inner * 6)
    del proj, xbc, st, sts, y
    m = L["delta"]
    H, KH, Kd, V = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    ch = 2 * KH * Kd + H * V
    A, dtb = torch.randn(H, device=device) * 0.3, torch.zeros(H, device=device) - 3
    qkv, ba = [rnd(T, ch) for _ in range(C)], rnd(T, 2 * H)
    st = torch.zeros(B + 1, H, Kd, V, device=device)
    fl = T * H * (6 * Kd * V + 3 * q * Kd / 2 * 2 + 3 * q * V / 2 * 2)
    pre["delta_chunk"] = _entry(_graph_us([lambda x=x: K.gated_delta_scan(x, ba[:, :H], ba[:, H:], A, dtb, st, slots, pos, seg, KH, Kd ** -0.5) for x in qkv]),
                                T * (ch + H * V + 2 * H) * 2, f32=fl)
    sts = [torch.zeros(B + 1, H, Kd, V, device=device) for _ in range(3)]
    dec["delta_step"] = _entry(_graph_us([lambda s=s: K.gated_delta_scan(qkv[0][:B], ba[:B, :H], ba[:B, H:], A, dtb, s, dslots, dpos, s0, KH, Kd ** -0.5)
                                          for s in sts * 4]), B * H * Kd * V * 8)
    y, hw = rnd(T, H * V), torch.ones(V, device=device)
    gates = [rnd(T, H * V) for _ in range(C)]
    pre["gated_rmsnorm (delta)"] = _entry(_graph_us([lambda g=g: K.gated_rmsnorm(y, g, hw, H, 1e-6, False) for g in gates]), T * H * V * 6)
    del qkv, st, sts, y, gates
    m = L["latent_attention"]
    H, Dn, R, V, rank, win = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"], m["mask"]["size"]
    dk, row = Dn + R, (rank + R + 31) // 32 * 32
    total = B * ctx + T + 64
    caches = [rnd(total, row) for _ in range(3)]
    r2t = torch.zeros(B + 1, max(ctx, n), dtype=torch.int32, device=device)
    perm = torch.randperm(B * ctx, device=device).int() + 1
    r2t[1:, :ctx] = perm.view(B, ctx)
    qc, qr = rnd(B, H, rank), rnd(B, H, R)
    keys = min(ctx, win)
    fl = B * keys * H * 2 * (rank + R + rank)
    groups, fill = ((H + 15) // 16, 512) if H <= 16 else ((H + 31) // 32, 256)
    splits = max(1, min((fill + B * groups - 1) // (B * groups), (keys + 63) // 64))
    dec["latent_attention (absorbed)"] = _entry(_graph_us([lambda c=c: K.latent_attention(qc, qr, c, r2t, dslots, dpos, s0, win, m["scale"], splits) for c in caches * 2]),
                                                B * keys * (rank + R) * 2, bf16=fl)
    wa, wv = [rnd(H, rank, Dn) for _ in range(16)], [rnd(H, V, rank) for _ in range(16)]
    qh, oc = rnd(B, H, Dn), rnd(B, H, rank)
    dec["head_gemm (key)"] = _entry(_graph_us([lambda w=w: K.head_gemm(qh, w) for w in wa]), H * rank * Dn * 2 + B * H * (Dn + rank) * 2)
    dec["head_gemm (value)"] = _entry(_graph_us([lambda w=w: K.head_gemm(oc, w) for w in wv]), H * rank * V * 2 + B * H * (V + rank) * 2)
    cs = torch.randn(max(ctx, n), R, device=device)
    loc = torch.arange(1, T + 1, device=device)
    dkv, nw = rnd(T, rank + R), torch.ones(rank, device=device)
    qs = [rnd(T, H * dk) for _ in range(2)]
    pre["latent_prepare"] = _entry(_graph_us([lambda x=x: K.latent_prepare(x, dkv, nw, cs, pos, loc, caches[0], H, Dn, R, 1e-6) for x in qs * 2]),
                                   T * ((rank + R) * 4 + H * R * 4))
    vis = K.VisibleKeys([0] * segs, [n] * segs, win, device)
    rr = torch.zeros(segs + 1, n, dtype=torch.int32, device=device)
    rr[1:] = (torch.randperm(T, device=device).int() + 1).view(segs, n)
    pre["latent_gather"] = _entry(_graph_us([lambda c=c: K.latent_gather(c, rr, slots, vis) for c in caches * 2]), T * row * 4)
    lat = K.latent_gather(caches[0], rr, slots, vis)
    kvs = [rnd(T, H * (Dn + V)) for _ in range(2)]
    w = min(win, n)
    pairs = segs * (w * (w + 1) / 2 + (n - w) * w)
    pre["latent_prefill"] = _entry(_graph_us([lambda kv=kv: K.latent_prefill(qs[0], lat, kv, vis, pos, seg, H, Dn, R, rank, V, win, m["scale"]) for kv in kvs * 2]),
                                   T * H * (2 * dk + 2 * V) * 2, bf16=2 * pairs * H * (dk + V))
    del caches, qs, kvs, lat
    # the like kernels of the decoder beside it, same tokens, same head count
    like_pre, like_dec = {}, {}
    Hkv, D = max(1, H // 4), 128
    kc, vc = [rnd(B * ctx + 1, Hkv, D) for _ in range(3)], [rnd(B * ctx + 1, Hkv, D) for _ in range(3)]
    qx = rnd(T, H, D)
    ox = torch.empty_like(qx)
    rr2 = torch.zeros(segs + 1, n, dtype=torch.int32, device=device)
    rr2[1:] = rr[1:]
    indptr = i32([i * n for i in range(segs + 1)])
    none = torch.zeros_like(seg.len)
    us = _graph_us([lambda k=k, v=v: K.extend_attention(qx, ox, k, v, rr2, slots, seg.len, none, indptr, n, D ** -0.5) for k, v in zip(kc, vc)])
    like_pre["extend_attention"] = _entry(us, T * (H * 2 + Hkv * 2) * D * 2, bf16=4 * H * D * segs * n * (n + 1) / 2)
    q1 = rnd(B, H, D)
    o1, lens = torch.empty_like(q1), torch.full((B,), ctx, dtype=torch.int32, device=device)
    ns = max(1, 512 // (B * Hkv))
    acc, ml = K.decode_workspace(B, H, D, ns, device)
    us = _graph_us([lambda k=k, v=v: K.decode_attention(q1, k, v, o1, r2t, dslots, lens, D ** -0.5, ns, acc, ml) for k, v in zip(kc * 2, vc * 2)])
    like_dec["decode_attention"] = _entry(us, B * ctx * Hkv * D * 4)
    wt = torch.ones(W, dtype=bf, device=device)
    for name, rows, copies, table in (("fused_add_rmsnorm", T, C, like_pre), ("fused_add_rmsnorm", B, 64, like_dec)):
        b = [(rnd(rows, W), rnd(rows, W)) for _ in range(copies)]
        table[name] = _entry(_graph_us([lambda x=x, r=r: K.fused_add_rmsnorm(x, r, wt, 1e-6) for x, r in b]), rows * W * 8)
    x = [rnd(T, 2 * ff) for _ in range(2)]
    like_pre["silu_and_mul"] = _entry(_graph_us([lambda a=a: K.silu_and_mul(a) for a in x * 2]), T * ff * 6)
    wq = [rnd(W, W) for _ in range(8)]
    xb = rnd(B, W)
    like_dec["wstream_gemm"] = _entry(_graph_us([lambda w=w: K.wstream_gemm(xb, w) for w in wq]), W * W * 2 + B * W * 4)
    return dict(prefill=pre, decode=dec, like_prefill=like_pre, like_decode=like_dec)


def run(names, device, kernels_only=False):
    from benchmarks import grouped_bench, layered_bench, shifted_bench
    from sglang_amd.harness.bulodra import BulodraConfig
    from sglang_amd.harness.dugalix import DugalixConfig
    from sglang_amd.harness.mosurax import MosuraxConfig
    from sglang_amd.harness.registry import named_config

    out = {}
    for name in names:
        cfg = named_config(name)
        key, table, beside = (("design", shifted_bench.kernel_table, shifted_bench.models_beside) if isinstance(cfg, DugalixConfig) else
                              ("design", layered_bench.kernel_table, layered_bench.models_beside) if isinstance(cfg, BulodraConfig) else
                              ("design", grouped_bench.kernel_table, grouped_bench.decoders_beside) if isinstance(cfg, MosuraxConfig) else
                              ("hybrid", kernel_table, lambda c: {"decoder_beside": _llama_beside(c)}))
        shape = dict(prompts=4, length=2048, batch=64, ctx=1024)
        r = dict(shape=shape, kernels=table(cfg, device))
        torch.cuda.empty_cache()
        print(f"{name}: kernel table done", file=sys.stderr, flush=True)
        if not kernels_only:
            for other, c in {key: cfg, **beside(cfg)}.items():
                r[other] = throughput(c, device, **shape)
                print(f"{name}: throughput of {other} done", file=sys.stderr, flush=True)
        out[name] = r
    print(json.dumps({"hybrid": out, "dtype": "bf16", "data": "synthetic (random weights and tokens)"}), flush=True)
