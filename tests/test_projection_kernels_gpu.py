"""The kernels of Bulodra's mechanisms one by one against plain evaluations on the CPU: what stands between a projection and attention
(norms, rotation, biases, cache rows, latents), bigram rows, gated activations in every launch that has them, sigmoid scores within
groups, the residual launch with a norm behind the sublayer, and caps, sinks and gates of both kinds of attention."""
import math

import pytest
import torch

from oracle import bulodra as ob
from test_grouped_kernels_gpu import LENS, _Case, _rel

pytestmark = pytest.mark.gpu
F32, BF = torch.float32, torch.bfloat16


def _table(positions, dims, base=50.0):
    from sglang_amd.layers.mixers import rotary_table

    return rotary_table(positions, dims, base, torch.device("cpu"), dict(factor=3.0, original=60, fast=8.0, slow=1.0))


def _turn(x, table, pos, off, dims):
    """x [T, heads, n] float64: element off + i turns with off + i + dims / 2."""
    c, s = table[pos].double()[:, None, :].split(dims // 2, -1)
    u, v = x[..., off:off + dims // 2], x[..., off + dims // 2:off + dims]
    return torch.cat([x[..., :off], u * c - v * s, v * c + u * s, x[..., off + dims:]], -1)


def _source(K, rows, bias, form, device):
    """A projection's output as the launches take it: rows (bias included) or three partials and the bias."""
    if form == "rows":
        return (rows + (bias if bias is not None else 0)).to(device)
    T, N = rows.shape
    parts = torch.randn(3, T, N, generator=torch.Generator().manual_seed(N))
    parts[2] = rows.float() - parts[0] - parts[1]
    return K.Partials(parts.to(device), 3, T, N, bias.to(device) if bias is not None else None)


@pytest.mark.parametrize("H,G,dim,vdim,dims", [(6, 2, 40, 24, 24), (4, 4, 64, 128, 32), (3, 1, 9, 11, 6), (16, 2, 128, 128, 128), (2, 2, 20, 12, 10), (5, 5, 200, 72, 16), (1, 1, 300, 520, 300)])
@pytest.mark.parametrize("order", ["before", "after", "none"])
@pytest.mark.parametrize("dtype,form", [(BF, "rows"), (BF, "partials"), (F32, "rows")])
def test_heads_between_projection_and_attention(device, H, G, dim, vdim, dims, order, dtype, form):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(dim + dims)
    T, eps, kd, vd = 13, 1e-3, dim + -dim % 8, vdim + -vdim % 8
    pos, loc = torch.randint(0, 90, (T,), generator=g), torch.randperm(40, generator=g)[:T] + 1
    table, gates = _table(90, dims), 8 * ((H + 7) // 8)
    pad = lambda t, to: torch.cat([t, torch.zeros(*t.shape[:-1], to - t.shape[-1], dtype=t.dtype)], -1)
    make = lambda *s: torch.randn(*s, generator=g).to(dtype)
    q, k, v, gate = make(T, H, dim), make(T, G, dim), make(T, G, vdim), make(T, gates)
    bq, bk, bv = (make(n, d) if form == "partials" else None for n, d in ((H, dim), (G, dim), (G, vdim)))
    rows = torch.cat([pad(q, kd).flatten(1), pad(k, kd).flatten(1), pad(v, vd).flatten(1), gate, torch.zeros(T, 8, dtype=dtype)], 1)
    bias = torch.cat([pad(bq, kd).flatten(), pad(bk, kd).flatten(), pad(bv, vd).flatten(), torch.zeros(gates + 8, dtype=dtype)]) if bq is not None else None
    wq, wk = 1 + 0.2 * torch.randn(dim, generator=g), 1 + 0.2 * torch.randn(dim, generator=g)
    norms = tuple(pad(w, kd).to(device) for w in (wq, wk)) if order == "before" else None

    def want(x, b, w):
        x = x.double() + (b.double() if b is not None else 0)
        if order == "before":
            x = ob.unit_rms(x, eps) * w.double()
        x = _turn(x, table, pos, 0, dims)
        return ob.unit_rms(x, eps) if order == "after" else x

    wants = want(q, bq, wq), want(k, bk, wk), v.double() + (bv.double() if bv is not None else 0)
    for plain in (False, True):
        cache = torch.full((42, G * (kd + vd)), 3.0, dtype=dtype, device=device)
        got, gg = K.head_prepare(_source(K, rows, bias, form, device), H, dim, kd, pos.to(device), table.to(device), eps, norms=norms, norm_after=order == "after",
                                 gate_cols=gates, kv=(G, vd, cache, loc.to(device)), plain=plain)
        kc, vc = cache[loc.to(device)].view(T, G, kd + vd).split([kd, vd], -1)
        tol = 5e-3 if dtype == BF else 2e-6
        for out, n, ref in ((got.unflatten(1, (H, kd)), dim, wants[0]), (kc, dim, wants[1]), (vc, vdim, wants[2])):
            assert _rel(out[..., :n], ref) < tol and float(out[..., n:].abs().sum()) == 0
        assert _rel(gg[:, :H], gate[:, :H]) < tol
        untouched = torch.ones(42, dtype=torch.bool)
        untouched[loc] = False
        assert float((cache[untouched.to(device)] - 3.0).abs().max()) == 0


@pytest.mark.parametrize("H,dim,rot,dims", [(5, 24, 16, 16), (4, 64, 32, 32), (3, 7, 6, 4), (16, 128, 64, 64), (2, 40, 24, 16)])
@pytest.mark.parametrize("dtype,form", [(BF, "rows"), (BF, "partials"), (F32, "rows")])
def test_the_turned_part_behind_the_plain_one(device, H, dim, rot, dims, dtype, form):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(dim)
    T, dk = 21, dim + rot
    pos, table = torch.randint(0, 70, (T,), generator=g), _table(70, dims)
    rows = torch.randn(T, H * dk + (16 if dk % 2 == 0 else 3), generator=g).to(dtype)
    for plain in (False, True):
        got, gate = K.head_prepare(_source(K, rows, None, form, device), H, dk, dk, pos.to(device), table.to(device), 1e-6, rot_off=dim, plain=plain)
        assert gate is None and _rel(got.unflatten(1, (H, dk)), _turn(rows[:, :H * dk].double().view(T, H, dk), table, pos, dim, dims)) < (4e-3 if dtype == BF else 1e-6)


@pytest.mark.parametrize("q_rank,rank,rot,dims", [(72, 48, 16, 16), (11, 13, 6, 4), (768, 512, 64, 64), (0, 40, 8, 8), (128, 128, 32, 32)])
@pytest.mark.parametrize("dtype,form", [(BF, "rows"), (BF, "partials"), (F32, "rows")])
def test_latents_between_projection_and_cache(device, q_rank, rank, rot, dims, dtype, form):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(rank)
    T, eps = 9, 1e-3
    pos, loc, table = torch.randint(0, 70, (T,), generator=g), torch.randperm(30, generator=g)[:T] + 1, _table(70, dims)
    rows = (torch.randn(T, q_rank + rank + rot, generator=g) * 2).to(dtype)
    wq, wc = 1 + 0.2 * torch.randn(q_rank, generator=g), 1 + 0.2 * torch.randn(rank, generator=g)
    cache = torch.full((33, (rank + rot + 31) // 32 * 32), 3.0, dtype=dtype, device=device)
    cq = K.latent_down(_source(K, rows, None, form, device), wq.to(device) if q_rank else None, wc.to(device), table.to(device), pos.to(device), loc.to(device), cache, rot, eps)
    q, c, k = rows.double().split([q_rank, rank, rot], 1)
    tol = 4e-3 if dtype == BF else 1e-6
    if q_rank:
        assert _rel(cq, ob.unit_rms(q, eps) * wq.double()) < tol
    row = cache[loc.to(device)]
    assert _rel(row[:, :rank], ob.unit_rms(c, eps) * wc.double()) < tol and _rel(row[:, rank:rank + rot], _turn(k[:, None], table, pos, 0, dims)[:, 0]) < tol
    assert float((row[:, rank + rot:] - 3.0).abs().sum()) == 0 and int((cache[:, 0] == 3.0).sum()) == 33 - T


def test_bigram_rows_follow_slots(device):
    """Portions, decode batches and a shared prefix; factors beyond the number of buckets; ids large enough for 32 bits to overflow."""
    from sglang_amd import kernels as K

    toks = [[70001, 5, 99999, 7, 131071, 7, 2], [11, 12, 13]]
    mul_prev, mul_cur, buckets = 999983, 65537, 4093
    want = [ob.bigram_rows(t, mul_prev, mul_cur, buckets) for t in toks]
    d = lambda v, dt=torch.int64: torch.tensor(v, dtype=dt, device=device)
    r2t = torch.zeros(4, 8, dtype=torch.int32)
    r2t[2, :7], r2t[1, :3] = torch.tensor([9, 4, 11, 3, 8, 2, 6]), torch.tensor([5, 10, 7])
    r2t, sid = r2t.to(device), torch.zeros(12, dtype=torch.int32, device=device)
    slots, at, got = {0: [9, 4, 11, 3, 8, 2, 6], 1: [5, 10, 7]}, [0, 0], [[], []]
    for step in ([(0, 2), (1, 1)], [(1, 1), (0, 3)], [(0, 1), (1, 1)], [(0, 1)]):
        decode = all(n == 1 and at[b] for b, n in step)
        ids = [t for b, n in step for t in toks[b][at[b]:at[b] + n]]
        pos = [p for b, n in step for p in range(at[b], at[b] + n)]
        loc = [s for b, n in step for s in slots[b][at[b]:at[b] + n]]
        seg = None if decode else d([i for i, (_, n) in enumerate(step) for _ in range(n)], torch.int32)
        rows = K.bigram_rows(d(ids), d(pos), d(loc), r2t, d([2 - b for b, _ in step]), seg, sid, mul_prev, mul_cur, buckets).tolist()
        for b, n in step:
            got[b] += rows[:n]
            rows, at[b] = rows[n:], at[b] + n
    assert got == want
    # another request over the first four slots of request 0: the token in front of its fifth is found there
    r2t[3, :5] = d([9, 4, 11, 3, 1], torch.int32)
    assert K.bigram_rows(d([50]), d([4]), d([1]), r2t, d([3]), None, sid, mul_prev, mul_cur, buckets).tolist() == [(7 * mul_prev + 50 * mul_cur) % buckets]


# ---------------------------------------------------------------------------------------------- gated activations
def _acts(K):
    silu = lambda g, u: g * torch.sigmoid(g) * u
    return {"silu": (K.SILU, silu), "gelu": (K.Glu("gelu_tanh"), lambda g, u: ob.gelu_tanh(g) * u),
            "clamped": (K.Glu("clamped_swish", 0.8, 1.702), lambda g, u: ob.clamped_swiglu(g, u, 0.8))}


@pytest.mark.parametrize("name", ["silu", "gelu", "clamped"])
@pytest.mark.parametrize("T,W,ff,E,top", [(3, 288, 64, 12, 3), (70, 256, 128, 4, 2), (40, 136, 64, 9, 3), (900, 256, 64, 4, 2), (3100, 192, 128, 3, 3)])
def test_activations_of_routed_experts(device, name, T, W, ff, E, top):
    from sglang_amd import kernels as K

    act, ref = _acts(K)[name]
    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, W, generator=g).to(BF)
    w13, w2 = (torch.randn(E, 2 * ff, W, generator=g) * 1.5 / math.sqrt(W)).to(BF), (torch.randn(E, W, ff, generator=g) / math.sqrt(ff)).to(BF)
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    want = torch.zeros(T, top, W, dtype=torch.float64)
    for e in range(E):
        t, s = (ids == e).nonzero(as_tuple=True)
        want[t, s] = ref(h[t].double() @ w13[e, :ff].double().T, h[t].double() @ w13[e, ff:].double().T) @ w2[e].double().T
    args = [x.to(device) for x in (h, w13, w2)]
    assert _rel(K.routed_experts(*args, ids.to(device), act=act), want) < 8e-3
    if T < 100:
        assert _rel(K.routed_experts(*args, ids.to(device), plain=True, act=act), want) < 8e-3
        assert _rel(K.routed_experts(*(a.float() for a in args), ids.to(device), act=act), want) < 2e-6


@pytest.mark.parametrize("name", ["silu", "gelu", "clamped"])
@pytest.mark.parametrize("T,W,ff", [(5, 128, 64), (37, 256, 512), (64, 512, 1040), (100, 1024, 256), (300, 160, 72), (9, 96, 50)])
def test_activations_of_dense_parts(device, name, T, W, ff):
    from sglang_amd import kernels as K
    from sglang_amd.harness.models import Linear
    from sglang_amd.layers.feed_forward import DenseMLP

    act, ref = _acts(K)[name]
    g = torch.Generator().manual_seed(T)
    t = {"gate": torch.randn(ff, W, generator=g) * 1.5 / math.sqrt(W), "up": torch.randn(ff, W, generator=g) * 1.5 / math.sqrt(W), "down": torch.randn(W, ff, generator=g) / math.sqrt(ff)}
    h = torch.randn(T, W, generator=g)
    for dtype, tol in ((BF, 8e-3), (F32, 2e-6)):
        w = {k: v.to(BF) for k, v in t.items()}
        x = h.to(BF)
        mlp = DenseMLP(W, ff, lambda n, s, init=None: w[n].to(device, dtype), Linear, bias=False, act=act)
        want = ref(x.double() @ w["gate"].double().T, x.double() @ w["up"].double().T) @ w["down"].double().T
        y = mlp(x.to(device, dtype))
        y = y.data.flatten()[:y.splits * T * W].view(y.splits, T, W).sum(0) if isinstance(y, K.Partials) else y
        assert _rel(y, want) < tol
        if dtype == BF and ff % 16 == 0 and W % 128 == 0 and T <= 64:        # the weight stream's own epilogue, and the one behind split-K
            x, gu = x.to(device), mlp.gate_up.weight.data
            hid = ref(h.to(BF).double() @ w["gate"].double().T, h.to(BF).double() @ w["up"].double().T)
            for kw in (dict(), dict(splits=1), dict(splits=min(2, W // 128), waves_per_group=4)):
                assert _rel(K.wstream_gemm(x, gu, epilogue="silu_and_mul", act=act, **kw), hid) < 8e-3


# ---------------------------------------------------------------------------------------------- router
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("T,K,E,top,groups,keep", [(1, 64, 2, 1, 1, 1), (37, 288, 24, 3, 4, 2), (5, 102, 7, 4, 7, 5), (64, 2048, 64, 8, 8, 3), (19, 136, 20, 4, 5, 1),
                                                   (70, 256, 200, 6, 25, 4), (2100, 256, 33, 3, 3, 1), (9, 96, 256, 8, 128, 100), (40, 72, 130, 5, 2, 2)])
def test_sigmoid_scores_within_groups(device, dtype, T, K, E, top, groups, keep):
    from sglang_amd import kernels as Kn

    g = torch.Generator().manual_seed(T + E)
    h, w = torch.randn(T, K, generator=g).to(dtype), (torch.randn(E, K, generator=g) * 2 / math.sqrt(K)).to(dtype)
    c = torch.randn(E, generator=g) * 0.7 - 0.6                 # most choice scores are below zero
    scores = Kn.SigmoidScores(c.to(device), groups, keep, 2.3)
    gp, ge = Kn.moe_route(h.to(device), w.to(device), None, top, scores)
    gp, ge = gp.double().cpu(), ge.long().cpu()
    r = dict(top=top, scale=2.3, groups=dict(count=groups, keep=keep))
    clear = 0
    for t in range(T):
        ob.margins.clear()
        ref = ob.route(h[t:t + 1].double(), w.double(), c.double(), r)[0]
        if min(ob.margins, default=1.0) < 1e-5:
            continue
        clear += 1
        got = dict(zip(ge[t].tolist(), gp[t].tolist()))
        assert set(got) == {e for e, _ in ref}, t
        assert all(abs(got[e] - float(p)) < 3e-6 * 2.3 * 4 for e, p in ref)
    assert clear > 0.8 * T and all(len(set(x.tolist())) == top for x in ge)
    # what is not a number still gives every place one expert of the range
    bad = h.to(device).clone()
    bad[0] = float("nan")
    ids = Kn.moe_route(bad, w.to(device), None, top, scores)[1][0].tolist()
    assert len(set(ids)) == top and all(0 <= e < E for e in ids)
    with pytest.raises(RuntimeError, match="groups"):
        Kn.moe_route(h.to(device), w.to(device), None, top, Kn.SigmoidScores(None, E + 1, 1))


# ---------------------------------------------------------------------------------------------- residual rows
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows,W", [(3, 102), (5, 336), (64, 2048), (1100, 336), (1030, 2048), (1025, 4096), (9, 5120), (2, 6001)])
def test_a_norm_behind_the_sublayer(device, dtype, rows, W):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(W)
    rnd = lambda *s: torch.randn(*s, generator=g)
    d = lambda t: t.to(device)
    eps, m = 1e-2, 0.6
    w1, w2 = 1 + 0.2 * rnd(W), 1 + 0.2 * rnd(W)
    x, h = d(rnd(rows, W)), torch.empty(rows, W, dtype=dtype, device=device)
    y, part = rnd(rows, W).to(dtype), rnd(3, rows, W)
    data, weights = rnd(rows, 5, W).to(dtype), rnd(rows, 5)
    experts = (data.double() * weights.double()[:, :, None]).sum(1)
    for add, s in (((d(y),), y.double()), ((K.Partials(d(part), 3, rows, W, None),), part.double().sum(0)), ((K.ExpertRows(d(data), d(weights)), d(y)), experts + y.double()),
                   ((K.ExpertRows(d(data), d(weights)), K.Partials(d(part), 3, rows, W, None)), experts + part.double().sum(0)), ((d(y * 1e-3),), (y * 1e-3).double())):
        for norm in (None, w2):
            now = x.double().cpu() + m * ob.unit_rms(s, eps) * w1.double()
            K.residual_rms(x, eps, add=add, post=(d(w1), m), h=h, norm=None if norm is None else d(norm))
            assert _rel(x, now) < 1e-6
            assert _rel(h, now if norm is None else ob.unit_rms(now, eps) * w2.double()) < (4e-3 if dtype == BF else 2e-6)
    K.residual_rms(x, eps, add=(d(y),), post=(d(w1), m))
    table, ids = rnd(50, W).to(dtype), torch.randint(0, 50, (rows,), generator=g)
    K.residual_rms(x, eps, embed=(d(ids), d(table), 1.0), h=h)
    assert torch.equal(x.cpu(), table[ids].float()) and torch.equal(h.cpu(), table[ids])


# ---------------------------------------------------------------------------------------------- attention
@pytest.mark.parametrize("window", [1, 33, 64, 65, 0])
@pytest.mark.parametrize("sizes", [(6, 2, 40, 72), (3, 1, 16, 24), (4, 4, 64, 128), (20, 1, 136, 136), (2, 1, 200, 256)])
def test_caps_sinks_and_head_gates(device, sizes, window):
    from sglang_amd import kernels as K

    H, G, D, V = sizes
    sinks = torch.linspace(-3, 4, H).double()
    for dtype in (BF, F32):
        c = _Case(LENS, H, G, D, V, dtype, device, seed=window)
        forms = [("plain", 1), ("plain", 3)]
        if dtype == BF:
            forms += [("rows", 1), ("rows", 4)] + ([("prefill", 1)] if K.grouped_prefill_supported(D, V, H // G) else [])
        for sink, gated, cap in ((sinks, False, None), (None, "heads", 1.3), (sinks, "heads", 40.0)):
            want = c.want(window, 3 * D ** -0.5, sink, gated, cap)
            for form, splits in forms:
                e = _rel(c.run(form, window, 3 * D ** -0.5, sink, gated, splits, cap), want)
                assert e < (4e-3 if dtype == BF else 3e-6), (dtype, form, splits, cap, e)


def test_a_cap_bends_what_stands_out(device):
    """A key whose score is far beyond the cap takes exactly e^cap against its rivals, without overflow."""
    for form in ("rows", "prefill", "plain"):
        for distance in (0, 63, 199):
            c = _Case([(100, 100)], 2, 1, 32, 32, BF, device, seed=distance, spike=distance)
            got, want = c.run(form, 0, 1.0, None, False, 1, 3.0), c.want(0, 1.0, None, False, 3.0)
            assert _rel(got, want) < 4e-3 and _rel(got[-1], c.want(0, 1.0, None, False)[-1]) > 0.2


@pytest.mark.parametrize("heads,rank,rot,dim,vdim", [(5, 48, 16, 24, 40), (20, 72, 8, 40, 24), (4, 128, 64, 128, 128), (16, 512, 64, 128, 128), (3, 13, 6, 7, 5)])
def test_latent_sinks_in_every_form(device, heads, rank, rot, dim, vdim):
    """Absorbed (matrix and plain, split or not) and expanded: the sink a head joins every denominator once."""
    from sglang_amd import kernels as K

    lens = [(0, 100), (77, 3), (150, 1), (0, 1)]
    g = torch.Generator().manual_seed(rank)
    scale, sinks = (dim + rot) ** -0.5, torch.linspace(-2, 4, heads)
    width, row = max(p + n for p, n in lens), (rank + rot + 31) // 32 * 32
    slots, at = torch.randperm(400, generator=g) + 1, 0
    r2t, cache32 = torch.zeros(len(lens) + 1, width, dtype=torch.int32), torch.zeros(402, row)
    n = torch.tensor([m for _, m in lens], dtype=torch.int32)
    T = int(n.sum())
    rows, pos = [], torch.cat([torch.arange(p, p + m) for p, m in lens])
    for b, (p, m) in enumerate(lens):
        sl = slots[at:at + p + m]
        at += p + m
        r2t[b + 1, :p + m] = sl.int()
        cache32[sl, :rank + rot] = torch.randn(p + m, rank + rot, generator=g)
        rows.append(sl)
    seg = K.Segments(torch.repeat_interleave(torch.arange(len(lens), dtype=torch.int32), n.long()).to(device), (torch.cumsum(n, 0) - n).int().to(device), n.to(device), int(n.max()))
    wk, wv = torch.randn(heads, dim, rank, generator=g) / math.sqrt(rank), torch.randn(heads, vdim, rank, generator=g) / math.sqrt(rank)
    for dtype in (BF, F32):
        q, cache, uk, uv = (2 * torch.randn(T, heads, dim + rot, generator=torch.Generator().manual_seed(1))).to(dtype), cache32.to(dtype), wk.to(dtype), wv.to(dtype)
        qc = torch.stack([q[:, h, :dim].double() @ uk[h].double() for h in range(heads)], 1).to(dtype)       # absorbed queries, rounded once
        want_c, want_v, i = torch.zeros(T, heads, rank, dtype=torch.float64), torch.zeros(T, heads, vdim, dtype=torch.float64), 0
        for (p, m), sl in zip(lens, rows):
            c = cache[sl].double()
            keys = torch.cat([torch.stack([(c[:, :rank] @ uk[h].double().T).to(dtype).double() for h in range(heads)], 1), c[:, None, rank:rank + rot].expand(-1, heads, -1)], -1)
            vals = torch.stack([(c[:, :rank] @ uv[h].double().T).to(dtype).double() for h in range(heads)], 1)
            for j in range(m):
                see = p + j + 1
                for h in range(heads):
                    s = torch.cat([(c[:see, :rank] @ qc[i, h].double() + c[:see, rank:rank + rot] @ q[i, h, dim:].double()) * scale, sinks[h:h + 1].double()])
                    want_c[i, h] = torch.softmax(s, 0)[:-1] @ c[:see, :rank]
                    s = torch.cat([keys[:see, h] @ q[i, h].double() * scale, sinks[h:h + 1].double()])
                    want_v[i, h] = torch.softmax(s, 0)[:-1] @ vals[:see, h]
                i += 1
        dev = lambda t: t.to(device)
        args = (dev(qc), dev(q)[:, :, dim:], dev(cache), dev(r2t), torch.arange(1, len(lens) + 1, device=device), dev(pos), seg, 0, scale)
        for splits in (1, 3):
            for plain in (False, True):
                e = _rel(K.latent_attention(*args, splits, plain, sinks=dev(sinks)), want_c)
                assert e < (4e-3 if dtype == BF else 3e-6), (dtype, splits, plain, e)
        assert _rel(K.latent_attention(*args), want_c) > 0.02   # without sinks it is another answer
        if dtype == BF and rank % 8 == 0 and K.latent_prefill_supported(dim, rot, vdim):
            vis = K.VisibleKeys([p for p, _ in lens], [m for _, m in lens], 0, device)
            lat = K.latent_gather(args[2], args[3], args[4], vis)
            kv = torch.nn.functional.linear(lat[:, :rank], dev(torch.cat([uk.flatten(0, 1), uv.flatten(0, 1)], 0)))
            o = K.latent_prefill(dev(q).flatten(1), lat, kv, vis, args[5], seg, heads, dim, rot, rank, vdim, 0, scale, sinks=dev(sinks))
            assert _rel(o, want_v.flatten(1)) < 5e-3
