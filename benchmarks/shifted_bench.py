"""The kernels of the Dugalix design against their rooflines beside the like kernels of the framework's closest models (Mosurax, the
recurrences of Genusun, the plain decoders), and the Mosurax model its throughput is set beside.  Run through
`bench.py --hybrid dugalix-1b dugalix-8b`; random weights."""
from __future__ import annotations

import torch

from benchmarks.hybrid_bench import _entry, _graph_us


def _gated(ff: int) -> int:
    """The width at which a gated part has as many weights as one of width `ff` without a gate."""
    return ff * 2 // 3


def models_beside(cfg):
    """A Mosurax model of the same width, heads, window, vocabulary and number of layers whose feed-forwards have as many weights (its
    are gated: two thirds as wide)."""
    from sglang_amd.harness.mosurax import MosuraxConfig

    m = next(lay["mixer"] for lay in cfg.layers if lay["type"] == "attention")
    mixer = {k: m[k] for k in ("heads", "kv_heads", "dim", "vdim", "scale", "mask")}

    def feed(f):
        if f["kind"] == "dense":
            return dict(kind="dense", ff=_gated(f["ff"]))
        return dict(kind="moe", expert=dict(ff=_gated(f["expert"]["ff"])), shared=dict(ff=_gated(f["shared"]["ff"])),
                    router=dict(experts=f["router"]["experts"], top=f["router"]["top"]))

    layers = [dict(type="attention", mixer=mixer, mlp=feed(lay["mlp"])) for lay in cfg.layers]
    return {"mosurax_beside": MosuraxConfig(f"mosurax-beside-{cfg.name}", cfg.vocab_size, cfg.hidden_size, layers, cfg.eps, None, 8192, 30.0)}


def kernel_table(cfg, device, T=8192, segs=4, B=64, ctx=1024):
    """T prompt tokens in `segs` requests, and decode steps of B requests at context `ctx`, at this model's layer sizes."""
    from sglang_amd import kernels as K
    from sglang_amd.harness.dugalix import SQUARED_RELU
    from sglang_amd.layers.attention.hybrid_backend import HybridAttnBackend

    bf = torch.bfloat16
    rnd = lambda *s, dtype=bf: (torch.randn(*s, device=device) * 0.5).to(dtype)
    W, n = cfg.hidden_size, T // segs
    att, par = (next(lay["mixer"] for lay in cfg.layers if lay["type"] == t) for t in ("attention", "parallel"))
    ff = next(lay["mlp"]["ff"] for lay in cfg.layers if lay["mlp"]["kind"] == "dense")
    moe = next(lay["mlp"] for lay in cfg.layers if lay["mlp"]["kind"] == "moe")
    r = moe["router"]
    E, I, top, eff = r["experts"], r["identity"], r["top"], moe["expert"]["ff"]
    i32 = lambda v: torch.tensor(v, dtype=torch.int32, device=device)
    seg = K.Segments(torch.repeat_interleave(torch.arange(segs, dtype=torch.int32, device=device), n), i32([i * n for i in range(segs)]),
                     i32([n] * segs), n)
    pos, slots = torch.arange(n, device=device).repeat(segs), torch.arange(1, segs + 1, device=device)
    dslots, dpos, s0 = torch.arange(1, B + 1, device=device), torch.full((B,), ctx - 1, device=device), K.Segments()
    pre, dec, like_pre, like_dec = {}, {}, {}, {}
    one, eps, mu, bias = torch.ones(W, device=device), 1e-6, torch.rand(W, device=device), torch.randn(W, device=device)
    left = torch.zeros(B + 1, W, dtype=bf, device=device)

    # ---- residual rows: sum, norm, add, norm; single tokens blend with the row in front on the way, portions in a launch of their own
    for table, like, rows, copies in ((pre, like_pre, T, 4), (dec, like_dec, B, 32)):
        bufs = [(torch.randn(rows, W, device=device), rnd(rows, W), torch.empty(rows, W, dtype=bf, device=device)) for _ in range(copies)]
        wt, ex = torch.rand(rows, top + 1, device=device), [rnd(rows, top, W) for _ in range(min(copies, 8))]
        ids = torch.randint(0, E + I, (rows, top), device=device)
        ids, plain = torch.where(ids < E, ids, -1).int(), torch.rand(rows, top, device=device)
        shift = dict(shift=K.TokenShift(mu, left, dslots, dpos)) if rows == B else {}
        extra = rows * W * 4 if rows == B else 0           # the row in front, and this one for the next
        post = dict(post=(one, 0.7), norm=one)
        table["residual_rms (post, norm" + (", shift)" if shift else ")")] = _entry(
            _graph_us([lambda b=b: K.residual_rms(b[0], eps, add=(b[1],), h=b[2], bias=bias, **post, **shift) for b in bufs]), rows * W * 12 + extra)
        like["residual_rms"] = _entry(_graph_us([lambda b=b: K.residual_rms(b[0], eps, add=(b[1],), h=b[2], norm=one) for b in bufs]), rows * W * 12)
        table["residual_rms (expert and input rows)"] = _entry(
            _graph_us([lambda b=b, e=e: K.residual_rms(b[0], eps, add=(K.ExpertRows(e, wt[:, :top], ids, b[2]), K.Scaled(b[1], wt[:, top])), h=b[2], **post, **shift)
                       for b, e in zip(bufs * 2, ex)]), rows * W * (12 + 2 * top) + extra)
        like["residual_rms (expert rows)"] = _entry(_graph_us([lambda b=b, e=e: K.residual_rms(b[0], eps, add=(K.ExpertRows(e, plain), b[1]), h=b[2], norm=one)
                                                               for b, e in zip(bufs * 2, ex)]), rows * W * (12 + 2 * top))
        del bufs, ex
    x, out = [rnd(T, W) for _ in range(4)], torch.empty(T, W, dtype=bf, device=device)
    pre["token_shift"] = _entry(_graph_us([lambda a=a: K.token_shift(a, mu, left, slots, pos, seg, out) for a in x]), T * W * 4)
    taps, ring = torch.randn(2, W, device=device), torch.zeros(B + 1, 2, W, dtype=bf, device=device)
    like_pre["causal_conv_silu (2 taps)"] = _entry(_graph_us([lambda a=a: K.causal_conv_silu(a, taps, None, ring, slots, pos, seg) for a in x]), T * W * 4)
    # ---- activations
    x = [rnd(T, ff) for _ in range(2)]
    pre["squared_relu"] = _entry(_graph_us([lambda a=a: K.squared_relu_(a) for a in x * 2]), T * ff * 4)
    x = [rnd(T, 2 * _gated(ff)) for _ in range(2)]
    like_pre["silu_and_mul"] = _entry(_graph_us([lambda a=a: K.silu_and_mul(a) for a in x * 2]), T * _gated(ff) * 6)
    xb, wu = rnd(B, W), [rnd(ff, W) for _ in range(3)]
    dec["wstream_gemm (squared relu)"] = _entry(_graph_us([lambda w=w: K.wstream_gemm(xb, w, act=SQUARED_RELU) for w in wu * 2]), ff * W * 2 + B * (W + ff) * 2)
    wg = [rnd(2 * _gated(ff), W) for _ in range(3)]
    like_dec["wstream_gemm (silu)"] = _entry(_graph_us([lambda w=w: K.wstream_gemm(xb, w, epilogue="silu_and_mul") for w in wg * 2]),
                                             2 * _gated(ff) * W * 2 + B * (W + _gated(ff)) * 2)
    del x, wu, wg
    # ---- router and experts
    wr, wl, rb = [rnd(E + I + 1, W) for _ in range(8)], [rnd(E, W) for _ in range(8)], torch.randn(E, device=device)
    scores = K.SoftmaxScores(torch.randn(E + I, device=device) * 0.1, r["groups"]["count"], r["groups"]["keep"])
    for table, like, rows in ((pre, like_pre, T), (dec, like_dec, B)):
        hs = [rnd(rows, W) for _ in range(4)]
        table["moe_route (softmax scores, groups, gate)"] = _entry(_graph_us([lambda h=h, w=w: K.moe_route(h, w, None, top, scores, I, True) for h, w in zip(hs * 2, wr)]),
                                                                   rows * W * 2 + (E + I + 1) * W * 2 + rows * (top * 8 + 4), bf16=2 * rows * (E + I + 1) * W)
        like["moe_route"] = _entry(_graph_us([lambda h=h, w=w: K.moe_route(h, w, rb, top) for h, w in zip(hs * 2, wl)]), rows * W * 2 + E * W * 2 + rows * top * 8,
                                   bf16=2 * rows * E * W)
        ids = torch.stack([torch.randperm(E, device=device)[:top] for _ in range(min(rows, 512))]).int().repeat((rows + 511) // 512, 1)[:rows].contiguous()
        for to, act, width, up, tag in ((table, SQUARED_RELU, eff, 1, "routed_experts (squared relu)"), (like, K.SILU, _gated(eff), 2, "routed_experts")):
            w13, w2 = [rnd(E, up * width, W) for _ in range(2)], [rnd(E, W, width) for _ in range(2)]
            by = min(E, rows * top) * (up + 1) * width * W * 2 + rows * W * 2 + rows * top * W * 2
            to[tag] = _entry(_graph_us([lambda h=h, a=a, b=b: K.routed_experts(h, a, b, ids, act=act) for h, a, b in zip(hs, w13 * 2, w2 * 2)]), by,
                             bf16=2 * (up + 1) * rows * top * width * W)
            del w13, w2
        del hs
    # ---- attention: sigmoid weights over keys that are the values, a window beside kept tokens
    H, G, D, win, scale = att["heads"], att["kv_heads"], att["dim"], att["mask"]["size"], att["scale"]
    keep, offsets, row = par["left"]["mask"]["keep_first"], torch.randn(H, device=device), G * 2 * D
    mem = par["right"]
    MH, MD, MV = mem["heads"], mem["dim"], mem["vdim"]
    beside = 2 * MH * MD + 2 * MH * MV + 2 * MH
    tail = (beside + 7) // 8 * 8
    half, full = torch.randn(max(ctx, n), att["rot"]["dims"], device=device), torch.randn(max(ctx, n), par["left"]["rot"]["dims"], device=device)
    rr = torch.zeros(segs + 1, n, dtype=torch.int32, device=device)
    rr[1:] = (torch.randperm(T, device=device).int() + 1).view(segs, n)
    ploc, big = rr[1:].flatten().long(), [rnd(T + 1, row) for _ in range(3)]
    two, three = (H + G) * D, (H + 2 * G) * D
    proj, wide = [rnd(T, two) for _ in range(2)], [rnd(T, three + tail) for _ in range(2)]
    pre["head_prepare (turn, values are keys)"] = _entry(_graph_us([lambda p=p, x=x: K.head_prepare(p, H, D, D, pos, half, eps, kv=(G, D, x, ploc), value_is_key=True)
                                                                    for p, x in zip(proj * 3, big * 2)]), T * (2 * H + 3 * G) * D * 2)
    pre["head_prepare (turn, columns beside)"] = _entry(_graph_us([lambda p=p, x=x: K.head_prepare(p, H, D, D, pos, full, eps, gate_cols=tail, kv=(G, D, x, ploc))
                                                                   for p, x in zip(wide * 3, big * 2)]), T * three * 4)
    kcs = [(x[:, :G * D].contiguous(), x[:, G * D:].contiguous()) for x in big]
    like_pre["rotary_embedding + store"] = _entry(_graph_us([lambda p=p, k=k, v=v: K.rotary_embedding(pos, p[:, :H * D], p[:, H * D:two], D, full, value=p[:, two:three],
                                                                                                    k_cache=k, v_cache=v, cache_loc=ploc)
                                                             for p, (k, v) in zip(wide * 3, kcs * 2)]), T * three * 4)
    blocks, w = K.QueryBlocks([0] * segs, [n] * segs, win, H // G, device), min(win, n)
    pairs = segs * (w * (w + 1) / 2 + (n - w) * w)
    kept = segs * sum(min(keep, max(0, q + 1 - win)) for q in range(n))
    pf = lambda p, x, **kw: K.grouped_prefill(p[:, :H * D], x, rr, slots, pos, seg, blocks, H, G, D, D, win, scale, **kw)
    io = T * (H * 4 + G * 4) * D
    for to, tag, pr, kw in ((pre, "grouped_prefill (sigmoid)", pairs, dict(offsets=offsets)), (pre, "grouped_prefill (kept tokens)", pairs + kept, dict(keep=keep)),
                            (like_pre, "grouped_prefill (window)", pairs, dict(sink=0.0))):
        to[tag] = _entry(_graph_us([lambda p=p, x=x: pf(p, x, **kw) for p, x in zip(wide * 2, big)]), io, bf16=4 * pr * H * D)
    del big, kcs, proj
    caches = [rnd(B * ctx + 1, row) for _ in range(3)]
    r2t = torch.zeros(B + 1, max(ctx, n), dtype=torch.int32, device=device)
    r2t[1:, :ctx] = (torch.randperm(B * ctx, device=device).int() + 1).view(B, ctx)
    loc, qd = r2t[1:, ctx - 1].long().contiguous(), rnd(B, H * D)
    backend = type("B", (), dict(max_context_len=ctx + 128))
    for tag, table, cols, cut, kw in (("head_prepare (values are keys, partials)", half, two, two, dict(value_is_key=True)),
                                      ("head_prepare (columns beside, partials)", full, three + tail, three + tail, dict(gate_cols=tail))):
        _, splits = K.choose_wstream_config(B, cols, W, True)      # a decode projection's partials, as the weight stream leaves them
        parts = [K.Partials(torch.randn(splits, B, cols, device=device), splits, B, cols, None) for _ in range(8)]
        dec[tag] = _entry(_graph_us([lambda p=p: K.head_prepare(p, H, D, D, dpos, table, eps, kv=(G, D, caches[0], loc), **kw) for p in parts * 2]),
                          B * cols * (4 * splits + 2) + (B * G * D * 2 if "value_is_key" in kw else 0))
    rows_ = [rnd(B, three) for _ in range(8)]
    kc, vc = caches[0][:, :G * D].contiguous(), caches[0][:, G * D:].contiguous()
    like_dec["rotary_embedding + store"] = _entry(_graph_us([lambda p=p: K.rotary_embedding(dpos, p[:, :H * D], p[:, H * D:two], D, full, value=p[:, two:], k_cache=kc,
                                                                                          v_cache=vc, cache_loc=loc) for p in rows_ * 2]), B * three * 4)
    keys = min(ctx, win)
    layer = type("L", (), dict(window=win, keep_first=keep, kv_heads=G, group=H // G, heads=H))
    sp = HybridAttnBackend._grouped_splits(backend, layer, B, True)
    for to, tag, ks, kw in ((dec, "grouped_attention (sigmoid)", keys, dict(offsets=offsets)), (dec, "grouped_attention (kept tokens)", min(ctx, keys + keep), dict(keep=keep)),
                            (like_dec, "grouped_attention (window)", keys, dict(sink=0.0))):
        to[tag] = _entry(_graph_us([lambda x=x: K.grouped_attention(qd, x, r2t, dslots, dpos, s0, H, G, D, D, win, scale, splits=sp, **kw) for x in caches * 2]),
                         B * ks * row * 2 + B * H * D * 4, bf16=4 * B * ks * H * D)
    del caches, parts, kc, vc
    # ---- the matrix memory beside the recurrences of the same heads, and the norm behind it
    starts = [0, MH * MD, 2 * MH * MD, 2 * MH * MD + MH * MV, 2 * MH * (MD + MV), 2 * MH * (MD + MV) + MH, beside]
    cut = lambda p: [p[:, three + a:three + b] for a, b in zip(starts, starts[1:])]
    bi, bfg = torch.zeros(MH, device=device), torch.full((MH,), 3.0, device=device)
    states = [torch.zeros(B + 1, MH, MD, MV, device=device) for _ in range(3)]
    norms = [torch.zeros(B + 1, MH, (MV + 15) // 16, MD + 1, device=device) for _ in range(3)]

    def scan(p, s, z, sl, ps, sg):
        q, k, v, _, i, f = cut(p)
        return K.memory_scan(q, k, v, i, f, bi, bfg, s, z, sl, ps, sg, mem["gate_cap"], MD ** -0.5)

    chunk = 32
    fl = T * MH * (4 * MD * MV + 1.5 * chunk * MD / 2 + 1.5 * chunk * MV / 2)
    pre["memory_chunk"] = _entry(_graph_us([lambda p=p, s=s, z=z: scan(p, s, z, slots, pos, seg) for p, s, z in zip(wide * 2, states, norms)]),
                                 T * MH * (2 * MD + 2 * MV + 2) * 2, f32=fl)
    A, dtb, Dk = torch.randn(MH, device=device) * 0.3, torch.zeros(MH, device=device) - 3, torch.ones(MH, device=device)
    xbc, dt = [rnd(T, MH * (MV + 2 * MD)) for _ in range(2)], rnd(T, 2 * MH)
    like_pre["mamba2_chunk"] = _entry(_graph_us([lambda x=x, s=s: K.mamba2_scan(x, dt[:, :MH], A, dtb, Dk, s, slots, pos, seg, MH) for x, s in zip(xbc * 2, states)]),
                                      T * MH * (2 * MD + 2 * MV + 1) * 2, f32=fl)
    like_pre["delta_chunk"] = _entry(_graph_us([lambda x=x, s=s: K.gated_delta_scan(x, dt[:, :MH], dt[:, MH:], A, dtb, s, slots, pos, seg, MH, MD ** -0.5)
                                                for x, s in zip(xbc * 2, states)]), T * MH * (2 * MD + 2 * MV + 2) * 2,
                                     f32=T * MH * (6 * MD * MV + 3 * chunk * MD + 3 * chunk * MV))
    dw = rnd(B, three + tail)
    by = B * MH * MD * MV * 8
    dec["memory_step"] = _entry(_graph_us([lambda s=s, z=z: scan(dw, s, z, dslots, dpos, s0) for s, z in zip(states * 4, norms * 4)]), by + B * MH * (MD + 1) * 8)
    like_dec["mamba2_step"] = _entry(_graph_us([lambda s=s: K.mamba2_scan(xbc[0][:B], dt[:B, :MH], A, dtb, Dk, s, dslots, dpos, s0, MH) for s in states * 4]), by)
    like_dec["delta_step"] = _entry(_graph_us([lambda s=s: K.gated_delta_scan(xbc[0][:B], dt[:B, :MH], dt[:B, MH:], A, dtb, s, dslots, dpos, s0, MH, MD ** -0.5)
                                               for s in states * 4]), by)
    hw, both = torch.ones(MH * MV, device=device), rnd(T, H * D + MH * MV)
    for to, like, rows, copies in ((pre, like_pre, T, 1), (dec, like_dec, B, 16)):
        ys = [rnd(rows, MH * MV) for _ in range(4)]
        g, o = [cut(p)[3][:rows] for p in wide], both[:rows, H * D:]
        to["gated_rmsnorm (sigmoid)"] = _entry(_graph_us([lambda y=y, z=z: K.gated_rmsnorm(y, z, hw, MH, eps, False, out=o, sigmoid_gate=True) for y, z in zip(ys * copies, g * 2 * copies)]),
                                               rows * MH * MV * 6)
        like["gated_rmsnorm (silu)"] = _entry(_graph_us([lambda y=y, z=z: K.gated_rmsnorm(y, z, hw, MH, eps, False) for y, z in zip(ys * copies, g * 2 * copies)]), rows * MH * MV * 6)
    return dict(prefill=pre, decode=dec, like_prefill=like_pre, like_decode=like_dec)
