"""The kernels behind Mosurax one by one against plain evaluations on the CPU: grouped-query attention in every form (windows, sink,
gate, ragged segments over scattered slots, a decode batch's own keys), the router, routed experts, the residual launch and the
logits' soft cap."""
import math

import pytest
import torch

from oracle import mosurax as om

pytestmark = pytest.mark.gpu
F32, BF = torch.float32, torch.bfloat16


def _dev(t, device, dtype=None):
    return t.to(device, dtype or t.dtype)


def _rel(got, want):
    return float((got.double().cpu() - want.double()).pow(2).mean().sqrt() / want.double().pow(2).mean().sqrt().clamp(min=1e-12))


# ---------------------------------------------------------------------------------------------- attention
def _attend(q, k, v, pos, window, scale, sink, gate, cap=None):
    """q [n, H, D] at positions pos over k [L, G, D], v [L, G, V] in float64; gate [n, H, V], [n, H, 1] or None; sink a number, [H] or None."""
    per = q.shape[1] // k.shape[1]
    s = torch.einsum("nhd,lhd->hnl", q, k.repeat_interleave(per, 1)) * scale
    j = torch.arange(k.shape[0])[None, :]
    seen = (j <= pos[:, None]) & ((pos[:, None] - j < window) if window > 0 else True)
    if cap is not None:
        s = cap * torch.tanh(s / cap)
    s = s.masked_fill(~seen[None], float("-inf"))
    if sink is not None:
        s = torch.cat([torch.as_tensor(sink, dtype=s.dtype).reshape(-1, 1, 1).expand_as(s[..., :1]), s], -1)
    p = torch.softmax(s, -1)[..., (0 if sink is None else 1):]
    o = torch.einsum("hnl,lhv->nhv", p, v.repeat_interleave(per, 1))
    return o if gate is None else o * torch.sigmoid(gate)


class _Case:
    """Requests of (prefix, new) lengths over scattered cache slots; `spike` makes single far scores stand out."""

    def __init__(self, lens, H, G, D, V, dtype, device, seed=0, page=1, spike=None):
        from sglang_amd import kernels as K

        g = torch.Generator().manual_seed(seed)
        rnd = lambda *s: torch.randn(*s, generator=g).to(dtype)
        self.lens, self.H, self.G, self.D, self.V, self.dtype = lens, H, G, D, V, dtype
        total = sum(p + n for p, n in lens)
        slots = torch.randperm((total + page - 1) // page + len(lens) + 3, generator=g) + 1
        slots = (slots[:, None] * page + torch.arange(page)).flatten()
        self.ks, self.vs, self.qs, self.gates = [], [], [], []
        width = max(p + n for p, n in lens)
        r2t, rows, at = torch.zeros(len(lens) + 2, width, dtype=torch.int32), torch.zeros(int(slots.max()) + 1, G, D + V, dtype=dtype), 0
        locs = []
        for b, (p, n) in enumerate(lens):
            k, v, q = rnd(p + n, G, D), rnd(p + n, G, V), rnd(n, H, D)
            if spike is not None:
                # the last query of the request wants the key `spike` tokens before it (and finds nothing else as good)
                j = p + n - 1 - spike
                if j >= 0:
                    k[j] = 0.0
                    k[j, :, 0] = 12.0
                    q[-1, :, 0] = 12.0
            self.ks.append(k), self.vs.append(v), self.qs.append(q), self.gates.append(rnd(n, H, V))
            sl = slots[at:at + p + n]
            at += p + n
            r2t[b + 1, :p + n] = sl.int()
            rows[sl] = torch.cat([k, v], 2)
            locs.append(sl[p:])
        self.rows, self.r2t = rows.flatten(1).to(device), r2t.to(device)
        self.req = torch.arange(1, len(lens) + 1, device=device)
        self.loc = torch.cat(locs).to(device)
        self.pos_list = [torch.arange(p, p + n) for p, n in lens]
        self.pos = torch.cat(self.pos_list).to(device)
        self.q = torch.cat(self.qs).flatten(1).to(device)
        self.gate = torch.cat(self.gates).flatten(1).to(device)
        self.new_k = torch.cat([k[p:] for k, (p, _) in zip(self.ks, lens)]).flatten(1).to(device)
        self.new_v = torch.cat([v[p:] for v, (p, _) in zip(self.vs, lens)]).flatten(1).to(device)
        n = torch.tensor([n for _, n in lens], dtype=torch.int32)
        self.seg = K.Segments(torch.repeat_interleave(torch.arange(len(lens), dtype=torch.int32), n.long()).to(device),
                              (torch.cumsum(n, 0) - n).int().to(device), n.to(device), int(n.max()))

    def want(self, window, scale, sink, gated, cap=None):
        """gated: True, False, or "heads" (the first column of every head's gates is the head's)."""
        return torch.cat([_attend(q.double(), k.double(), v.double(), pos, window, scale, sink,
                                  None if not gated else g.double()[..., :1] if gated == "heads" else g.double(), cap)
                          for q, k, v, pos, g in zip(self.qs, self.ks, self.vs, self.pos_list, self.gates)]).flatten(1)

    def run(self, form, window, scale, sink, gated, splits=1, cap=None):
        from sglang_amd import kernels as K

        sizes = (self.H, self.G, self.D, self.V, window, scale)
        where = (self.rows, self.r2t, self.req, self.pos, self.seg)
        gate = self.gate.view(-1, self.H, self.V)[:, :, 0].contiguous() if gated == "heads" else self.gate if gated else None
        kw = dict(sink=sink.float().to(self.q.device) if isinstance(sink, torch.Tensor) else sink, gate=gate, cap=cap)
        if form == "prefill":
            blocks = K.QueryBlocks([p for p, _ in self.lens], [n for _, n in self.lens], window, self.H // self.G, self.q.device)
            return K.grouped_prefill(self.q, *where, blocks, *sizes, **kw)
        return K.grouped_attention(self.q, *where, *sizes, splits=splits, plain=form == "plain", **kw)


LENS = [(0, 100), (77, 3), (150, 1), (5, 70), (64, 64), (0, 1)]
SIZES = [(6, 2, 40, 72), (3, 1, 16, 24), (4, 4, 64, 128), (20, 1, 136, 136), (16, 4, 128, 64), (2, 1, 200, 256)]


@pytest.mark.parametrize("window", [1, 33, 64, 65, 0])
@pytest.mark.parametrize("sizes", SIZES)
def test_attention_forms_against_plain_rows(device, sizes, window):
    from sglang_amd import kernels as K

    H, G, D, V = sizes
    for dtype in (BF, F32):
        c = _Case(LENS, H, G, D, V, dtype, device, seed=window)
        forms = [("plain", 1), ("plain", 3)]
        if dtype == BF:
            forms += [("rows", 1), ("rows", 4)] + ([("prefill", 1)] if K.grouped_prefill_supported(D, V, H // G) else [])
        for sink, gated in ((0.0, True), (None, False), (1.5, True)):
            want = c.want(window, D ** -0.5, sink, gated)
            for form, splits in forms:
                e = _rel(c.run(form, window, D ** -0.5, sink, gated, splits), want)
                assert e < (4e-3 if dtype == BF else 3e-6), (dtype, form, splits, sink, e)


@pytest.mark.parametrize("form", ["rows", "plain", "prefill"])
@pytest.mark.parametrize("window", [31, 32, 33, 63, 64, 65, 128, 129])
def test_a_key_inside_and_outside_the_window(device, form, window):
    """The last query's best key sits just inside, just outside and at tile borders of the window: it decides the output or is gone."""
    for distance in (window - 2, window - 1, window, window + 1):
        c = _Case([(0, 200), (131, 2), (139, 70)], 4, 2, 32, 32, BF, device, seed=distance, spike=distance)
        want = c.want(window, 1.0, 0.0, False)
        got = c.run(form, window, 1.0, 0.0, False)
        assert _rel(got, want) < 4e-3
        at = c.lens[0][1] - 1                                    # request 0's last query
        hit = c.vs[0][199 - distance].double().repeat_interleave(2, 0).flatten()
        near = float((got[at].double().cpu() - hit).norm() / hit.norm())
        assert (near < 0.05) if distance < window else (near > 0.3), (distance, near)


def test_a_far_key_among_thousands(device):
    for form, splits in (("rows", 1), ("rows", 7), ("prefill", 1), ("plain", 5)):
        for distance in (1, 63, 64, 1000, 2047, 2999):
            c = _Case([(2900, 100)], 4, 1, 64, 64, BF, device, seed=distance, spike=distance, page=16)
            got = c.run(form, 0, 1.0, 0.0, False, splits)[-1].double().cpu()
            hit = c.vs[0][2999 - distance].double().repeat_interleave(4, 0).flatten()
            off = float((got - hit).norm() / hit.norm())
            assert off < 0.05, (form, distance, off)


@pytest.mark.parametrize("dtype", [BF, F32])
def test_the_sink_takes_everything_or_nothing(device, dtype):
    """Scores far below the sink's leave nothing, far above it an ordinary softmax, without overflow on either side."""
    for form in ("rows", "plain") + (("prefill",) if dtype == BF else ()):
        for sign in (-1.0, 1.0):
            c = _Case([(0, 40), (90, 17)], 2, 1, 32, 32, dtype, device, seed=3)
            for k, q in zip(c.ks, c.qs):
                k[:, :, 0], q[:, :, 0] = 20.0, 20.0 * sign
            c2 = _Case.__new__(_Case)
            c2.__dict__.update(c.__dict__)
            rows = c.rows.view(-1, 64).clone()
            rows[:, 0] = 20.0
            c2.rows, c2.q = rows, torch.cat(c.qs).flatten(1).to(device)
            got = c2.run(form, 30, 1.0, 0.0, False)
            assert torch.isfinite(got).all()
            if sign < 0:
                assert float(got.abs().max()) == 0
            else:
                assert _rel(got, c2.want(30, 1.0, 0.0, False)) < (4e-3 if dtype == BF else 3e-5)


@pytest.mark.parametrize("sizes", [(6, 2, 40, 72), (20, 1, 136, 136), (16, 16, 64, 64)])
@pytest.mark.parametrize("splits", [1, 3])
def test_a_decode_batch_brings_its_own_keys(device, sizes, splits):
    """New keys and values read from the projection and stored on the way equal stored-first ones, and land in their rows."""
    from sglang_amd import kernels as K

    H, G, D, V = sizes
    c = _Case([(0, 1), (31, 1), (32, 1), (127, 1), (200, 1)], H, G, D, V, BF, device, seed=9)
    seg, stored = K.Segments(), c.rows.clone()
    sizes = (H, G, D, V, 100, D ** -0.5)
    c.rows[c.loc] = 7.0
    got = K.grouped_attention(c.q, c.rows, c.r2t, c.req, c.pos, seg, *sizes, sink=0.0, gate=c.gate, new=(c.new_k, c.new_v, c.loc), splits=splits)
    assert torch.equal(c.rows, stored)
    assert _rel(got, c.want(100, D ** -0.5, 0.0, True)) < 4e-3
    again = K.grouped_attention(c.q, c.rows, c.r2t, c.req, c.pos, seg, *sizes, sink=0.0, gate=c.gate, splits=splits)
    assert torch.equal(got, again)
    with pytest.raises(RuntimeError, match="matrix form"):
        K.grouped_attention(c.q, c.rows, c.r2t, c.req, c.pos, seg, *sizes, new=(c.new_k, c.new_v, c.loc), plain=True)


@pytest.mark.parametrize("dtype", [BF, F32])
def test_store_writes_exactly_its_rows(device, dtype):
    from sglang_amd import kernels as K

    c = _Case(LENS, 6, 3, 24, 40, dtype, device)
    stored = c.rows.clone()
    wide = torch.full((c.loc.numel(), 504), 3.0, dtype=dtype, device=device)
    wide[:, 8:80], wide[:, 80:200] = c.new_k, c.new_v
    c.rows[c.loc] = 0
    K.grouped_kv_store(wide[:, 8:80], wide[:, 80:200], c.rows, c.loc, 3)
    assert torch.equal(c.rows, stored)


# ---------------------------------------------------------------------------------------------- router and experts
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("T,K,E,top", [(1, 64, 1, 1), (37, 288, 24, 3), (5, 102, 7, 4), (64, 2048, 64, 8), (19, 136, 20, 20), (3, 72, 200, 5),
                                       (2100, 256, 33, 3), (70, 4096, 128, 6)])
def test_router_picks_and_weighs(device, dtype, T, K, E, top):
    from sglang_amd import kernels as Kn

    g = torch.Generator().manual_seed(T + E)
    h, w = torch.randn(T, K, generator=g).to(dtype), (torch.randn(E, K, generator=g) * 3 / math.sqrt(K)).to(dtype)
    b = torch.randn(E, generator=g)
    p, e = om.route(h.double(), w.double(), b.double(), top)
    gp, ge = Kn.moe_route(h.to(device), w.to(device), b.to(device), top)
    gp, ge = gp.double().cpu(), ge.long().cpu()
    z = h.double() @ w.double().T + b.double()
    s = torch.sort(z, -1, descending=True).values
    gaps = (s[:, :-1] - s[:, 1:])[:, :top] if E > 1 else torch.ones(T, 1)
    clear = gaps.min(-1).values > 1e-4
    assert clear.float().mean() > 0.8 and torch.equal(ge[clear], e[clear])
    assert float((gp - p).abs().max()) < 1e-3 and float((gp[clear] - p[clear]).abs().max()) < 2e-5
    assert all(len(set(r.tolist())) == top for r in ge)
    # without the bias other experts win
    assert E == top or not torch.equal(Kn.moe_route(h.to(device), w.to(device), None, top)[1].long().cpu(), ge) or T == 1


@pytest.mark.parametrize("T,W,ff,E,top", [(3, 288, 64, 12, 3), (70, 256, 128, 4, 2), (40, 136, 64, 9, 3), (900, 256, 64, 4, 2), (500, 384, 128, 3, 3)])
def test_routed_experts_forms(device, T, W, ff, E, top):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(T)
    h = torch.randn(T, W, generator=g).to(BF)
    w13, w2 = (torch.randn(E, 2 * ff, W, generator=g) / math.sqrt(W)).to(BF), (torch.randn(E, W, ff, generator=g) / math.sqrt(ff)).to(BF)
    ids = torch.stack([torch.randperm(E, generator=g)[:top] for _ in range(T)]).int()
    want = torch.zeros(T, top, W, dtype=torch.float64)
    for e in range(E):
        t, s = (ids == e).nonzero(as_tuple=True)
        want[t, s] = om.gated_mlp(h[t].double(), w13[e, :ff].double(), w13[e, ff:].double(), w2[e].double())
    args = [x.to(device) for x in (h, w13, w2)]
    assert _rel(K.routed_experts(*args, ids.to(device)), want) < 8e-3
    assert _rel(K.routed_experts(*args, ids.to(device), plain=True), want) < 8e-3
    assert _rel(K.routed_experts(*(a.float() for a in args), ids.to(device)), want) < 2e-6


# ---------------------------------------------------------------------------------------------- residual rows
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows,W", [(3, 102), (5, 336), (64, 2048), (1100, 336), (1030, 2048), (1025, 4096), (9, 5120), (2, 6001)])
def test_residual_rms_sources_and_order(device, dtype, rows, W):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(W)
    rnd = lambda *s: torch.randn(*s, generator=g)
    table, ptab, ids, pos = rnd(50, W).to(dtype), rnd(40, W).to(dtype), torch.randint(0, 50, (rows,), generator=g), torch.randint(0, 40, (rows,), generator=g)
    step, extra, w = rnd(W), rnd(rows, W), 1 + 0.1 * rnd(W)
    d = lambda t: t.to(device)
    eps, tol = 1e-3, 6e-3 if dtype == BF else 2e-6

    def check(x, h, want):
        assert _rel(x, want) < 1e-6
        if h is not None:
            assert _rel(h, want / torch.sqrt((want * want).mean(-1, keepdim=True) + eps) * w.double()) < tol

    x, h, save = torch.empty(rows, W, device=device), torch.empty(rows, W, dtype=dtype, device=device), torch.empty(rows, W, device=device)
    K.residual_rms(x, eps, embed=(d(ids), d(table), 1.5), pos=(d(pos), d(ptab)), save=save, step=d(step), norm=d(w), h=h)
    x0 = table[ids].double() * 1.5 + ptab[pos].double()
    assert _rel(save, x0) < 1e-6
    check(x, h, x0 + step.double())
    now = x.double().cpu()
    y = rnd(rows, W).to(dtype)
    K.residual_rms(x, eps, add=(d(y),), extra=d(extra), step=d(step), norm=d(w), h=h)
    now = now + y.double() + extra.double() + step.double()
    check(x, h, now)
    data, weights = rnd(rows, 5, W).to(dtype), rnd(rows, 5)
    now = x.double().cpu() + (data.double() * weights.double()[:, :, None]).sum(1) + y.double()
    K.residual_rms(x, eps, add=(K.ExpertRows(d(data), d(weights)), d(y)), norm=d(w), h=h)
    check(x, h, now)
    part = rnd(3, rows, W)
    now = x.double().cpu() + part.double().sum(0)
    K.residual_rms(x, eps, add=(K.Partials(d(part), 3, rows, W, None),))
    check(x, None, now)
    now = x.double().cpu() + part.double().sum(0) + (data.double() * weights.double()[:, :, None]).sum(1)
    K.residual_rms(x, eps, add=(K.ExpertRows(d(data), d(weights)), K.Partials(d(part), 3, rows, W, None)), norm=d(w), h=h)
    check(x, h, now)
    now = x.double().cpu()
    K.residual_rms(x, eps, norm=d(w), h=h)
    check(x, h, now)


@pytest.mark.parametrize("rows,V", [(1, 97), (7, 352), (64, 32000)])
def test_soft_cap(device, rows, V):
    from sglang_amd import kernels as K

    z = torch.randn(rows, V, generator=torch.Generator().manual_seed(V)) * 40
    z[0, :3] = torch.tensor([0.0, 1e30, -1e30])
    for dtype in (BF, F32):
        x = z.to(dtype)
        got = K.soft_cap(x.to(device), 20.0)
        assert got.dtype == F32 and float((got.double().cpu() - om.soft_cap(x.double(), 20.0)).abs().max()) < 1e-5 * 20
    parts = torch.randn(3, rows, V) * 10
    assert float((K.soft_cap(K.Partials(parts.to(device), 3, rows, V, None), 20.0).double().cpu() - om.soft_cap(parts.double().sum(0), 20.0)).abs().max()) < 1e-4
