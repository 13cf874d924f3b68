"""The kernels of the Bulodra design against their rooflines beside the like kernels of the framework's closest models (Mosurax, the
latent attention of Genusun, the plain decoders), and the Mosurax model its throughput is set beside.  Run through
`bench.py --hybrid bulodra-1b bulodra-8b`; random weights."""
from __future__ import annotations

import torch

from benchmarks.hybrid_bench import _entry, _graph_us


def models_beside(cfg):
    """A Mosurax model of the same width, heads, window, vocabulary, number of layers and feed-forward of every layer."""
    from sglang_amd.harness.mosurax import MosuraxConfig

    m = next(lay["mixer"] for lay in cfg.layers if lay["type"] == "attention_2")
    mixer = {k: m[k] for k in ("heads", "kv_heads", "dim", "vdim", "scale", "mask")}
    layers = [dict(type="attention", mixer=mixer, mlp=lay["mlp"]) for lay in cfg.layers]
    return {"mosurax_beside": MosuraxConfig(f"mosurax-beside-{cfg.name}", cfg.vocab_size, cfg.hidden_size, layers, cfg.eps, None, 8192, 30.0)}


def kernel_table(cfg, device, T=8192, segs=4, B=64, ctx=1024):
    """T prompt tokens in `segs` requests, and decode steps of B requests at context `ctx`, at this model's layer sizes."""
    from sglang_amd import kernels as K
    from sglang_amd.harness.bulodra import GELU, expert_activation
    from sglang_amd.layers.attention.hybrid_backend import HybridAttnBackend

    bf = torch.bfloat16
    rnd = lambda *s, dtype=bf: (torch.randn(*s, device=device) * 0.5).to(dtype)
    W, n = cfg.hidden_size, T // segs
    capped, plain, lat = (next(lay["mixer"] for lay in cfg.layers if lay["type"] == t) for t in ("attention_2", "attention", "latent_attention"))
    ff = next(lay["mlp"]["ff"] for lay in cfg.layers if lay["mlp"]["kind"] == "dense")
    moe = next(lay["mlp"] for lay in cfg.layers if lay["mlp"]["kind"] == "moe")
    E, top, eff, sff = moe["router"]["experts"], moe["router"]["top"], moe["expert"]["ff"], moe["shared"]["ff"]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)
    seg = K.Segments(torch.repeat_interleave(torch.arange(segs, dtype=torch.int32, device=device), n), i32([i * n for i in range(segs)]),
                     i32([n] * segs), n)
    pos, slots = torch.arange(n, device=device).repeat(segs), torch.arange(1, segs + 1, device=device)
    dslots, dpos, s0 = torch.arange(1, B + 1, device=device), torch.full((B,), ctx - 1, device=device), K.Segments()
    pre, dec, like_pre, like_dec = {}, {}, {}, {}
    one, eps = torch.ones(W, device=device), 1e-6

    # ---- residual rows: the sublayer's sum normed and added; decode from split-K partials of the output projection
    for table, like, rows, copies in ((pre, like_pre, T, 4), (dec, like_dec, B, 32)):
        bufs = [(torch.randn(rows, W, device=device), rnd(rows, W), torch.empty(rows, W, dtype=bf, device=device)) for _ in range(copies)]
        wt, ex = torch.rand(rows, top, device=device), [rnd(rows, top, W) for _ in range(min(copies, 8))]
        for to, kw, tag in ((table, dict(post=(one, 0.7)), "residual_rms (post)"), (like, dict(norm=one), "residual_rms")):
            to[tag] = _entry(_graph_us([lambda b=b: K.residual_rms(b[0], eps, add=(b[1],), h=b[2], **kw) for b in bufs]), rows * W * 12)
            to[tag + " (expert rows)"] = _entry(_graph_us([lambda b=b, e=e: K.residual_rms(b[0], eps, add=(K.ExpertRows(e, wt), b[1]), h=b[2], **kw)
                                                           for b, e in zip(bufs * 2, ex)]), rows * W * (12 + 2 * top))
        w1 = torch.ones(W, dtype=bf, device=device)
        like["fused_add_rmsnorm"] = _entry(_graph_us([lambda b=b: K.fused_add_rmsnorm(b[1], b[2], w1, eps) for b in bufs]), rows * W * 8)
        del bufs, ex
    # ---- activations
    x = [rnd(T, 2 * ff) for _ in range(2)]
    pre["glu_and_mul (gelu)"] = _entry(_graph_us([lambda a=a: K.glu_and_mul(a, GELU) for a in x * 2]), T * ff * 6)
    like_pre["silu_and_mul"] = _entry(_graph_us([lambda a=a: K.silu_and_mul(a) for a in x * 2]), T * ff * 6)
    x, act = [rnd(T, 2 * sff) for _ in range(4)], expert_activation(moe["shared"])
    pre["glu_and_mul (clamped, shared expert)"] = _entry(_graph_us([lambda a=a: K.glu_and_mul(a, act) for a in x]), T * sff * 6)
    like_pre["silu_and_mul (shared expert)"] = _entry(_graph_us([lambda a=a: K.silu_and_mul(a) for a in x]), T * sff * 6)
    xb, wg = rnd(B, W), [rnd(2 * ff, W) for _ in range(3)]
    dec["wstream_gemm (gelu)"] = _entry(_graph_us([lambda w=w: K.wstream_gemm(xb, w, epilogue="silu_and_mul", act=GELU) for w in wg]), 2 * ff * W * 2)
    like_dec["wstream_gemm (silu)"] = _entry(_graph_us([lambda w=w: K.wstream_gemm(xb, w, epilogue="silu_and_mul") for w in wg]), 2 * ff * W * 2)
    del x, wg
    # ---- router and experts
    wr, rb = [rnd(E, W) for _ in range(8)], torch.randn(E, device=device)
    r = moe["router"]
    scores, act = K.SigmoidScores(rb, r["groups"]["count"], r["groups"]["keep"], r["scale"]), expert_activation(moe["expert"])
    for table, like, rows in ((pre, like_pre, T), (dec, like_dec, B)):
        hs = [rnd(rows, W) for _ in range(4)]
        by, fl = rows * W * 2 + E * W * 2 + rows * top * 8, 2 * rows * E * W
        table["moe_route (groups)"] = _entry(_graph_us([lambda h=h, w=w: K.moe_route(h, w, None, top, scores) for h, w in zip(hs * 2, wr)]), by, bf16=fl)
        like["moe_route"] = _entry(_graph_us([lambda h=h, w=w: K.moe_route(h, w, rb, top) for h, w in zip(hs * 2, wr)]), by, bf16=fl)
        ids = torch.stack([torch.randperm(E, device=device)[:top] for _ in range(min(rows, 512))]).int().repeat((rows + 511) // 512, 1)[:rows].contiguous()
        w13, w2 = [rnd(E, 2 * eff, W) for _ in range(2)], [rnd(E, W, eff) for _ in range(2)]
        fl, by = 6 * rows * top * eff * W, min(E, rows * top) * 3 * eff * W * 2 + rows * W * 2 + rows * top * W * 2
        for to, a_, tag in ((table, act, "routed_experts (clamped)"), (like, K.SILU, "routed_experts")):
            to[tag] = _entry(_graph_us([lambda h=h, a=a, b=b: K.routed_experts(h, a, b, ids, act=a_) for h, a, b in zip(hs, w13 * 2, w2 * 2)]), by, bf16=fl)
        del w13, w2, hs
    # ---- grouped attention, whole causal with sinks and windowed with cap and gate
    H, G, D = plain["heads"], plain["kv_heads"], plain["dim"]
    row, cols = G * 2 * D, (H + 2 * G) * D
    win, cap, hgate = capped["mask"]["size"], capped["softcap"], (H + 7) // 8 * 8
    cos, half = torch.randn(max(ctx, n), plain["rot"]["dims"], device=device), torch.randn(max(ctx, n), capped["rot"]["dims"], device=device)
    qk = (torch.ones(D, device=device), torch.ones(D, device=device))
    sinks = torch.randn(H, device=device)
    rr = torch.zeros(segs + 1, n, dtype=torch.int32, device=device)
    rr[1:] = (torch.randperm(T, device=device).int() + 1).view(segs, n)
    ploc, big, proj = rr[1:].flatten().long(), [rnd(T + 1, row) for _ in range(3)], [rnd(T, cols + hgate) for _ in range(2)]
    by = T * cols * 4
    pre["head_prepare (norm, turn)"] = _entry(_graph_us([lambda p=p, x=x: K.head_prepare(p, H, D, D, pos, cos, eps, norms=qk, kv=(G, D, x, ploc))
                                                         for p, x in zip(proj * 3, big * 2)]), by)
    pre["head_prepare (turn, norm)"] = _entry(_graph_us([lambda p=p, x=x: K.head_prepare(p, H, D, D, pos, half, eps, norm_after=True, gate_cols=hgate, kv=(G, D, x, ploc))
                                                         for p, x in zip(proj * 3, big * 2)]), by)
    kcs = [(x[:, :G * D].contiguous(), x[:, G * D:].contiguous()) for x in big]
    like_pre["rotary_embedding + store"] = _entry(_graph_us([lambda p=p, k=k, v=v: K.rotary_embedding(pos, p[:, :H * D], p[:, H * D:(H + G) * D], D, cos, value=p[:, (H + G) * D:cols],
                                                                                                    k_cache=k, v_cache=v, cache_loc=ploc)
                                                             for p, (k, v) in zip(proj * 3, kcs * 2)]), by)
    w = min(win, n)
    pairs, causal = segs * (w * (w + 1) / 2 + (n - w) * w), segs * n * (n + 1) / 2
    b_win, b_all = (K.QueryBlocks([0] * segs, [n] * segs, v, H // G, device) for v in (win, 0))
    io = T * (H * 4 + G * 4) * D
    gates = [p[:, cols:cols + H] for p in proj]
    pf = lambda p, x, b, v, **kw: K.grouped_prefill(p[:, :H * D], x, rr, slots, pos, seg, b, H, G, D, D, v, D ** -0.5, **kw)
    pre["grouped_prefill (sinks)"] = _entry(_graph_us([lambda p=p, x=x: pf(p, x, b_all, 0, sink=sinks) for p, x in zip(proj * 2, big)]), io, bf16=4 * causal * H * D)
    pre["grouped_prefill (window, cap)"] = _entry(_graph_us([lambda p=p, x=x, g=g: pf(p, x, b_win, win, cap=cap, gate=g) for p, x, g in zip(proj * 2, big, gates * 2)]), io, bf16=4 * pairs * H * D)
    like_pre["grouped_prefill"] = _entry(_graph_us([lambda p=p, x=x: pf(p, x, b_all, 0, sink=0.0) for p, x in zip(proj * 2, big)]), io, bf16=4 * causal * H * D)
    like_pre["grouped_prefill (window)"] = _entry(_graph_us([lambda p=p, x=x: pf(p, x, b_win, win, sink=0.0) for p, x in zip(proj * 2, big)]), io, bf16=4 * pairs * H * D)
    del big, kcs, proj, gates
    caches = [rnd(B * ctx + 1, row) for _ in range(3)]
    r2t = torch.zeros(B + 1, max(ctx, n), dtype=torch.int32, device=device)
    r2t[1:, :ctx] = (torch.randperm(B * ctx, device=device).int() + 1).view(B, ctx)
    loc, qd, gd = r2t[1:, ctx - 1].long().contiguous(), rnd(B, H * D), rnd(B, H)
    backend = type("B", (), dict(max_context_len=ctx + 128))
    # a decode projection's partials, as the weight stream leaves them
    _, splits = K.choose_wstream_config(B, cols, W, True)
    parts = [K.Partials(torch.randn(splits, B, cols, device=device), splits, B, cols, None) for _ in range(8)]
    dec["head_prepare (partials)"] = _entry(_graph_us([lambda p=p: K.head_prepare(p, H, D, D, dpos, cos, eps, norms=qk, kv=(G, D, caches[0], loc)) for p in parts * 2]),
                                            B * cols * (4 * splits + 2))
    rows_ = [rnd(B, cols) for _ in range(8)]
    kc, vc = caches[0][:, :G * D].contiguous(), caches[0][:, G * D:].contiguous()
    like_dec["rotary_embedding + store"] = _entry(_graph_us([lambda p=p: K.rotary_embedding(dpos, p[:, :H * D], p[:, H * D:(H + G) * D], D, cos, value=p[:, (H + G) * D:], k_cache=kc,
                                                                                          v_cache=vc, cache_loc=loc) for p in rows_ * 2]), B * cols * 4)
    for to, name, v, kw in ((dec, "grouped_attention (sinks)", 0, dict(sink=sinks)), (dec, "grouped_attention (window, cap)", win, dict(cap=cap, gate=gd)),
                            (like_dec, "grouped_attention", 0, dict(sink=0.0)), (like_dec, "grouped_attention (window)", win, dict(sink=0.0))):
        keys = min(ctx, v) if v else ctx
        layer = type("L", (), dict(window=v, keep_first=0, kv_heads=G, group=H // G, heads=H))
        sp = HybridAttnBackend._grouped_splits(backend, layer, B, True)
        to[name] = _entry(_graph_us([lambda x=x: K.grouped_attention(qd, x, r2t, dslots, dpos, s0, H, G, D, D, v, D ** -0.5, splits=sp, **kw) for x in caches * 2]),
                          B * keys * row * 2 + B * H * D * 4, bf16=4 * B * keys * H * D)
    del caches, parts, kc, vc
    # ---- latent attention
    H, Dn, R, V, rank, qr_ = lat["heads"], lat["dim"], lat["rot_dim"], lat["vdim"], lat["kv_rank"], lat["q_rank"]
    dk, crow, sinks = Dn + R, (rank + R + 31) // 32 * 32, torch.randn(H, device=device)
    caches = [rnd(B * ctx + T + 64, crow) for _ in range(3)]
    cs = torch.randn(max(ctx, n), R, device=device)
    nq, nl = torch.ones(qr_, device=device), torch.ones(rank, device=device)
    down, qs = [rnd(T, qr_ + rank + R) for _ in range(4)], [rnd(T, H * dk) for _ in range(2)]
    pre["latent_down"] = _entry(_graph_us([lambda p=p: K.latent_down(p, nq, nl, cs, pos, ploc, caches[0], R, eps) for p in down]), T * (qr_ + rank + R) * 4)
    pre["head_prepare (turn latent queries)"] = _entry(_graph_us([lambda q=q: K.head_prepare(q, H, dk, dk, pos, cs, eps, rot_off=Dn) for q in qs * 2]), T * H * R * 4)
    like_pre["latent_prepare"] = _entry(_graph_us([lambda q=q: K.latent_prepare(q, down[0][:, :rank + R], nl, cs, pos, ploc, caches[0], H, Dn, R, eps) for q in qs * 2]),
                                        T * ((rank + R) * 4 + H * R * 4))
    vis = K.VisibleKeys([0] * segs, [n] * segs, 0, device)
    pre["latent_gather"] = _entry(_graph_us([lambda c=c: K.latent_gather(c, rr, slots, vis) for c in caches * 2]), T * crow * 4)
    gathered, kvs = K.latent_gather(caches[0], rr, slots, vis), [rnd(T, H * (Dn + V)) for _ in range(2)]
    for to, kw, tag in ((pre, dict(sinks=sinks), "latent_prefill (sinks)"), (like_pre, {}, "latent_prefill")):
        to[tag] = _entry(_graph_us([lambda kv=kv: K.latent_prefill(qs[0], gathered, kv, vis, pos, seg, H, Dn, R, rank, V, 0, lat["scale"], **kw) for kv in kvs * 2]),
                         T * H * (2 * dk + 2 * V) * 2, bf16=2 * causal * H * (dk + V))
    cols = qr_ + rank + R
    _, splits = K.choose_wstream_config(B, cols, W, True)
    parts = [K.Partials(torch.randn(splits, B, cols, device=device), splits, B, cols, None) for _ in range(8)]
    dec["latent_down (partials)"] = _entry(_graph_us([lambda p=p: K.latent_down(p, nq, nl, cs, dpos, loc, caches[0], R, eps) for p in parts * 2]), B * cols * (4 * splits + 2))
    _, splits = K.choose_wstream_config(B, H * dk, qr_, True)
    parts = [K.Partials(torch.randn(splits, B, H * dk, device=device), splits, B, H * dk, None) for _ in range(8)]
    dec["head_prepare (turn latent queries, partials)"] = _entry(_graph_us([lambda p=p: K.head_prepare(p, H, dk, dk, dpos, cs, eps, rot_off=Dn) for p in parts * 2]),
                                                                 B * H * dk * (4 * splits + 2))
    dq = [rnd(B, H * dk) for _ in range(8)]
    like_dec["latent_prepare"] = _entry(_graph_us([lambda q=q: K.latent_prepare(q, down[0][:B, :rank + R], nl, cs, dpos, loc, caches[0], H, Dn, R, eps) for q in dq * 2]),
                                        B * ((rank + R) * 4 + H * R * 4))
    qc, qr2 = rnd(B, H, rank), rnd(B, H, R)
    groups, fill = ((H + 15) // 16, 512) if H <= 16 else ((H + 31) // 32, 256)
    sp = max(1, min((fill + B * groups - 1) // (B * groups), (ctx + 63) // 64))
    for to, kw, tag in ((dec, dict(sinks=sinks), "latent_attention (sinks)"), (like_dec, {}, "latent_attention")):
        to[tag] = _entry(_graph_us([lambda c=c: K.latent_attention(qc, qr2, c, r2t, dslots, dpos, s0, 0, lat["scale"], sp, **kw) for c in caches * 2]),
                         B * ctx * (rank + R) * 2, bf16=B * ctx * H * 2 * (2 * rank + R))
    # ---- the bigram table's rows: index arithmetic, a launch; beside it another such launch
    sid = torch.zeros(B * ctx + T + 64, dtype=torch.int32, device=device)
    for to, like, ids, p_, l_, rq, sg in ((pre, like_pre, torch.randint(0, 999, (T,), device=device), pos, ploc, slots, seg.tok_seg),
                                          (dec, like_dec, torch.randint(0, 999, (B,), device=device), dpos, loc, dslots, None)):
        to["bigram_rows"] = _entry(_graph_us([lambda: K.bigram_rows(ids, p_, l_, r2t if sg is None else rr, rq, sg, sid, 31, 17, 999)] * 16), ids.numel() * 40)
        lens = torch.ones(ids.numel(), dtype=torch.int32, device=device)
        like["clamp_position"] = _entry(_graph_us([lambda: K.clamp_position(lens)] * 16), ids.numel() * 12)
    return dict(prefill=pre, decode=dec, like_prefill=like_pre, like_decode=like_dec)
