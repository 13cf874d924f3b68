"""The kernels of the Mosurax design against their rooflines beside the like kernels of the framework's other decoders, and the
decoders its throughput is set beside.  Run through `bench.py --hybrid mosurax-1b mosurax-8b`; random weights."""
from __future__ import annotations

import torch

from benchmarks.hybrid_bench import _entry, _graph_us


def decoders_beside(cfg):
    """Decoders of the same width, heads, window and vocabulary with as many layers as the design executes layer runs: one with its
    dense feed-forward in every layer, one with its routed experts in every layer (and no shared part)."""
    from sglang_amd.harness.models import ModelConfig

    m = cfg.layers[0]["mixer"]
    dense = next(lay["mlp"]["ff"] for lay in cfg.layers if lay["mlp"]["kind"] == "dense")
    moe = next(lay["mlp"] for lay in cfg.layers if lay["mlp"]["kind"] == "moe")

    def make(kind, ff, experts, top):
        return ModelConfig(f"{kind}-decoder-beside-{cfg.name}", cfg.hidden_size, ff, cfg.num_hidden_layers, m["heads"], m["kv_heads"], m["dim"],
                           cfg.vocab_size, 1e-5, 10000.0, None, 8192, num_local_experts=experts, num_experts_per_tok=top,
                           sliding_window=m["mask"]["size"] - 1)

    return {"dense_decoder_beside": make("dense", dense, 0, 0),
            "moe_decoder_beside": make("moe", moe["expert"]["ff"], moe["router"]["experts"], moe["router"]["top"])}


def kernel_table(cfg, device, T=8192, segs=4, B=64, ctx=1024):
    """T prompt tokens in `segs` requests, and decode steps of B requests at context `ctx`, at this model's layer sizes."""
    from sglang_amd import kernels as K
    from sglang_amd.layers.attention.hybrid_backend import HybridAttnBackend

    bf = torch.bfloat16
    rnd = lambda *s, dtype=bf: (torch.randn(*s, device=device) * 0.5).to(dtype)
    W, V = cfg.hidden_size, cfg.vocab_size
    m = cfg.layers[0]["mixer"]
    moe = next(lay["mlp"] for lay in cfg.layers if lay["mlp"]["kind"] == "moe")
    E, top, eff = moe["router"]["experts"], moe["router"]["top"], moe["expert"]["ff"]
    H, G, D, win, scale = m["heads"], m["kv_heads"], m["dim"], m["mask"]["size"], m["scale"]
    n = T // segs
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)
    seg = K.Segments(torch.repeat_interleave(torch.arange(segs, dtype=torch.int32, device=device), n), i32([i * n for i in range(segs)]),
                     i32([n] * segs), n)
    pos, slots = torch.arange(n, device=device).repeat(segs), torch.arange(1, segs + 1, device=device)
    dslots, dpos = torch.arange(1, B + 1, device=device), torch.full((B,), ctx - 1, device=device)
    pre, dec, like_pre, like_dec = {}, {}, {}, {}
    one = torch.ones(W, device=device)

    # ---- residual rows: one addend (a projection), and the experts' rows beside the shared part
    for table, like, rows, copies in ((pre, like_pre, T, 4), (dec, like_dec, B, 32)):
        bufs = [(torch.randn(rows, W, device=device), rnd(rows, W), torch.empty(rows, W, dtype=bf, device=device)) for _ in range(copies)]
        table["residual_rms"] = _entry(_graph_us([lambda b=b: K.residual_rms(b[0], 1e-6, add=(b[1],), norm=one, h=b[2]) for b in bufs]), rows * W * 12)
        wt = torch.rand(rows, top, device=device)
        ex = [rnd(rows, top, W) for _ in range(min(copies, 8))]
        table["residual_rms (expert rows)"] = _entry(_graph_us([lambda b=b, e=e: K.residual_rms(b[0], 1e-6, add=(K.ExpertRows(e, wt), b[1]), norm=one, h=b[2])
                                                                for b, e in zip(bufs * 2, ex)]), rows * W * (12 + 2 * top))
        w1 = torch.ones(W, dtype=bf, device=device)
        like["fused_add_rmsnorm"] = _entry(_graph_us([lambda b=b: K.fused_add_rmsnorm(b[1], b[2], w1, 1e-6) for b in bufs]), rows * W * 8)
        like["moe_sum_reduce"] = _entry(_graph_us([lambda b=b, e=e: K.moe_sum_reduce(e, b[2]) for b, e in zip(bufs * 2, ex)]), rows * W * (2 + 2 * top))
        del bufs, ex
    # ---- router and experts
    wr, rb = [rnd(E, W) for _ in range(8)], torch.randn(E, device=device)
    for table, like, rows in ((pre, like_pre, T), (dec, like_dec, B)):
        hs = [rnd(rows, W) for _ in range(4)]
        table["moe_route"] = _entry(_graph_us([lambda h=h, w=w: K.moe_route(h, w, rb, top) for h, w in zip(hs * 2, wr)]), rows * W * 2 + E * W * 2 + rows * top * 8,
                                    bf16=2 * rows * E * W)
        gate = K.wstream_gemm if K.wstream_preferred(rows, E, W) else torch.nn.functional.linear
        like["gate product + topk_softmax"] = _entry(_graph_us([lambda h=h, w=w: K.topk_softmax(gate(h, w), top, True) for h, w in zip(hs * 2, wr)]),
                                                     rows * W * 2 + E * W * 2 + rows * (E * 4 + top * 8), bf16=2 * rows * E * W)
        ids = torch.stack([torch.randperm(E, device=device)[:top] for _ in range(min(rows, 512))]).int().repeat((rows + 511) // 512, 1)[:rows].contiguous()
        tw = torch.full((rows, top), 1.0 / top, device=device)
        w13, w2 = [rnd(E, 2 * eff, W) for _ in range(2)], [rnd(E, W, eff) for _ in range(2)]
        fl, by = 6 * rows * top * eff * W, min(E, rows * top) * 3 * eff * W * 2 + rows * W * 2
        table["routed_experts"] = _entry(_graph_us([lambda h=h, a=a, b=b: K.routed_experts(h, a, b, ids) for h, a, b in zip(hs, w13 * 2, w2 * 2)]),
                                         by + rows * top * W * 2, bf16=fl)
        like["fused_experts"] = _entry(_graph_us([lambda h=h, a=a, b=b: K.fused_experts(h, a, b, tw, ids) for h, a, b in zip(hs, w13 * 2, w2 * 2)]),
                                       by + rows * W * 2, bf16=fl)
        del w13, w2, hs
    # ---- attention
    row = G * 2 * D
    caches = [rnd(B * ctx + 1, row) for _ in range(3)]
    kcs = [(c.view(-1, 2, G, D)[:, 0].contiguous(), c.view(-1, 2, G, D)[:, 1].contiguous()) for c in caches]
    r2t = torch.zeros(B + 1, max(ctx, n), dtype=torch.int32, device=device)
    r2t[1:, :ctx] = (torch.randperm(B * ctx, device=device).int() + 1).view(B, ctx)
    proj = [rnd(B, (2 * H + 2 * G) * D) for _ in range(2)]
    a, b, c = H * D, (H + G) * D, (H + 2 * G) * D
    keys, s0, loc = min(ctx, win), K.Segments(), r2t[1:, ctx - 1].long().contiguous()
    layer = type("L", (), dict(window=win, keep_first=0, kv_heads=G, group=H // G, heads=H))
    splits = HybridAttnBackend._grouped_splits(type("B", (), dict(max_context_len=ctx + 128)), layer, B, True)
    dec["grouped_attention"] = _entry(_graph_us([lambda p=p, x=x: K.grouped_attention(p[:, :a], x, r2t, dslots, dpos, s0, H, G, D, D, win, scale, sink=0.0, gate=p[:, c:],
                                                                                     new=(p[:, a:b], p[:, b:c], loc), splits=splits)
                                                 for p, x in zip(proj * 3, caches * 2)]), B * keys * row * 2 + B * H * D * 8, bf16=4 * B * keys * H * D)
    q1, o1, lens = rnd(B, H, D), torch.empty(B, H, D, dtype=bf, device=device), torch.full((B,), ctx, dtype=torch.int32, device=device)
    ns = max(1, 512 // (B * G))
    acc, ml = K.decode_workspace(B, H, D, ns, device)
    like_dec["decode_attention"] = _entry(_graph_us([lambda k=k, v=v: K.decode_attention(q1, k, v, o1, r2t, dslots, lens, D ** -0.5, ns, acc, ml, sliding_window=win - 1)
                                                     for k, v in kcs * 2]), B * keys * row * 2 + B * H * D * 4, bf16=4 * B * keys * H * D)
    big = [rnd(T + 1, row) for _ in range(3)]
    rr = torch.zeros(segs + 1, n, dtype=torch.int32, device=device)
    rr[1:] = (torch.randperm(T, device=device).int() + 1).view(segs, n)
    proj, ploc = [rnd(T, (2 * H + 2 * G) * D) for _ in range(2)], rr[1:].flatten().long()
    blocks = K.QueryBlocks([0] * segs, [n] * segs, win, H // G, device)
    w = min(win, n)
    pairs = segs * (w * (w + 1) / 2 + (n - w) * w)
    pre["grouped_kv_store"] = _entry(_graph_us([lambda p=p, x=x: K.grouped_kv_store(p[:, a:b], p[:, b:c], x, ploc, G) for p, x in zip(proj * 3, big * 2)]), T * row * 4)
    pre["grouped_prefill"] = _entry(_graph_us([lambda p=p, x=x: K.grouped_prefill(p[:, :a], x, rr, slots, pos, seg, blocks, H, G, D, D, win, scale, sink=0.0, gate=p[:, c:])
                                               for p, x in zip(proj * 2, big)]), T * (H * 6 + G * 4) * D, bf16=4 * pairs * H * D)
    kp = [(x.view(-1, 2, G, D)[:, 0].contiguous(), x.view(-1, 2, G, D)[:, 1].contiguous()) for x in big]
    qx, ox = rnd(T, H, D), torch.empty(T, H, D, dtype=bf, device=device)
    indptr, none = i32([i * n for i in range(segs + 1)]), torch.zeros_like(seg.len)
    for name, window, pr in (("extend_attention", -1, segs * n * (n + 1) / 2), ("extend_attention (window)", win - 1, pairs)):
        like_pre[name] = _entry(_graph_us([lambda k=k, v=v: K.extend_attention(qx, ox, k, v, rr, slots, seg.len, none, indptr, n, D ** -0.5, sliding_window=window)
                                           for k, v in kp]), T * (H * 4 + G * 4) * D, bf16=4 * pr * H * D)
    kk, vv = rnd(T, G * D), rnd(T, G * D)
    like_pre["store_kv_cache"] = _entry(_graph_us([lambda k=k, v=v: K.store_kv_cache(kk, vv, k, v, ploc) for k, v in kp * 2]), T * row * 4)
    del caches, kcs, big, kp, proj
    # ---- logits of a decode step
    zs = [K.Partials(torch.randn(1, B, V, device=device), 1, B, V, None) for _ in range(8)]
    dec["soft_cap"] = _entry(_graph_us([lambda z=z: K.soft_cap(z, 30.0) for z in zs]), B * V * 8)
    like_dec["argmax"] = _entry(_graph_us([lambda z=z: K.argmax(z.data[0]) for z in zs]), B * V * 4)
    wq = [rnd(W, W) for _ in range(8)]
    xb = rnd(B, W)
    like_dec["wstream_gemm"] = _entry(_graph_us([lambda x=x: K.wstream_gemm(xb, x) for x in wq]), W * W * 2 + B * W * 4)
    return dict(prefill=pre, decode=dec, like_prefill=like_pre, like_decode=like_dec)
