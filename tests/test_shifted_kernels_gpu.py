"""The kernels of Dugalix's mechanisms one by one against plain evaluations on the CPU: windows that keep first tokens and sigmoid weights in
every form of attention, values that are the keys as projected, both forms of the matrix memory, the token shift on its own and in the
residual launch, squared relu in every launch that has it, softmax scores within groups with identities and a gate, and the residual
launch's input rows, row factors and bias."""
import math

import pytest
import torch

from oracle import dugalix as od
from oracle import hybrid as oh
from test_grouped_kernels_gpu import LENS, SIZES, _Case, _rel
from test_hybrid_kernels_gpu import _err, _portions, _rand, _segments
from test_projection_kernels_gpu import _source, _turn

pytestmark = pytest.mark.gpu
F32, BF = torch.float32, torch.bfloat16
TOL = {F32: 2e-5, BF: 1.2e-2}


# ---------------------------------------------------------------------------------------------- attention
def _attend(q, k, v, pos, window, keep, scale, offsets):
    """q [n, H, D] at positions pos over k [L, G, D], v [L, G, V] in float64."""
    per = q.shape[1] // k.shape[1]
    s = torch.einsum("nhd,lhd->hnl", q, k.repeat_interleave(per, 1)) * scale
    j = torch.arange(k.shape[0])[None, :]
    near = (pos[:, None] - j < window) if window > 0 else torch.ones_like(j, dtype=torch.bool)
    seen = (j <= pos[:, None]) & (near | (j < keep))
    if offsets is not None:
        p = od.sigmoid(s + offsets[:, None, None]) * seen[None]
    else:
        p = torch.softmax(s.masked_fill(~seen[None], float("-inf")), -1)
    return torch.einsum("hnl,lhv->nhv", p, v.repeat_interleave(per, 1))


def _want(c, window, keep, scale, offsets):
    return torch.cat([_attend(q.double(), k.double(), v.double(), pos, window, keep, scale, offsets)
                      for q, k, v, pos in zip(c.qs, c.ks, c.vs, c.pos_list)]).flatten(1)


def _run(c, form, window, keep, scale, offsets, splits=1, out_scale=1.0, out=None):
    from sglang_amd import kernels as K

    sizes, where = (c.H, c.G, c.D, c.V, window, scale), (c.rows, c.r2t, c.req, c.pos, c.seg)
    kw = dict(keep=keep, offsets=offsets.float().to(c.q.device) if offsets is not None else None, out_scale=out_scale, out=out)
    if form == "prefill":
        blocks = K.QueryBlocks([p for p, _ in c.lens], [n for _, n in c.lens], window, c.H // c.G, c.q.device)
        return K.grouped_prefill(c.q, *where, blocks, *sizes, **kw)
    return K.grouped_attention(c.q, *where, *sizes, splits=splits, plain=form == "plain", **kw)


def _forms(K, dtype, G, H, D, V):
    forms = [("plain", 1), ("plain", 3)]
    if dtype == BF:
        forms += [("rows", 1), ("rows", 4)] + ([("prefill", 1)] if K.grouped_prefill_supported(D, V, H // G) else [])
    return forms


@pytest.mark.parametrize("window,keep", [(1, 0), (1, 1), (33, 5), (64, 64), (65, 3), (17, 100), (5, 70), (0, 4), (40, 6)])
@pytest.mark.parametrize("sizes", SIZES)
def test_kept_tokens_and_sigmoid_weights_in_every_form(device, sizes, window, keep):
    from sglang_amd import kernels as K

    H, G, D, V = sizes
    for dtype in (BF, F32):
        c = _Case(LENS, H, G, D, V, dtype, device, seed=window + keep)
        g = torch.Generator().manual_seed(1)
        for offsets in (None, torch.randn(H, generator=g).double()):
            want = _want(c, window, keep, D ** -0.5, offsets)
            for form, splits in _forms(K, dtype, G, H, D, V):
                wide = torch.full((c.q.shape[0], H * V + 24), 9.0, dtype=dtype, device=device)
                got = _run(c, form, window, keep, D ** -0.5, offsets, splits, out_scale=-1.7, out=wide[:, 8:8 + H * V])
                assert _rel(got, -1.7 * want) < (6e-3 if dtype == BF else 3e-6), (form, splits, offsets is not None, dtype)
                assert float((wide[:, :8] - 9).abs().max()) == 0 and float((wide[:, 8 + H * V:] - 9).abs().max()) == 0


@pytest.mark.parametrize("form,splits", [("plain", 1), ("plain", 3), ("rows", 1), ("rows", 4), ("prefill", 1)])
@pytest.mark.parametrize("at,inside", [(0, True), (5, True), (6, False), (7, False), (110, False), (111, True), (149, True)])
@pytest.mark.parametrize("sigmoid", [False, True])
def test_one_key_at_every_edge(device, form, splits, at, inside, sigmoid):
    """The last query of 150 looks for one key that outweighs all others, through a window of 39 beside 6 kept tokens."""
    c = _Case([(20, 130)], 4, 2, 40, 24, BF, device, seed=3, spike=149 - at)
    offsets = torch.full((4,), -9.0).double() if sigmoid else None
    want, got = _want(c, 39, 6, 0.2, offsets)[-1], _run(c, form, 39, 6, 0.2, offsets, splits)[-1].double().cpu()
    spike = c.vs[0][at].double().repeat_interleave(2, 0).flatten()
    assert float((got - want).abs().max()) < 2e-2
    near = lambda x: float((x - spike).pow(2).mean().sqrt()) < 0.2                # (the other keys' sigmoids add a little)
    assert near(got) == inside and near(want) == inside


@pytest.mark.parametrize("keep,window", [(4, 64), (700, 5), (64, 64)])
def test_decoding_far_behind_the_kept_tokens(device, keep, window):
    """Single queries thousands of tokens in, many splits, most of the kept range and of the window in different ones."""
    c = _Case([(3000, 1), (63, 1), (64, 1), (700, 1), (5, 1)], 8, 2, 64, 64, BF, device, seed=keep)
    for offsets in (None, torch.linspace(-3, 1, 8).double()):
        want = _want(c, window, keep, 0.3, offsets)
        for form, splits in (("plain", 5), ("rows", 1), ("rows", 7), ("rows", 32)):
            assert _rel(_run(c, form, window, keep, 0.3, offsets, splits), want) < 6e-3, (form, splits)


def test_sigmoid_weights_refuse_sinks_and_caps(device):
    from sglang_amd import kernels as K

    c = _Case([(0, 20)], 2, 1, 16, 16, BF, device)
    off = torch.zeros(2, device=device)
    for kw in (dict(sink=0.0), dict(cap=3.0), dict(sink=torch.zeros(2, device=device))):
        with pytest.raises(RuntimeError, match="no cap and no sink"):
            K.grouped_attention(c.q, c.rows, c.r2t, c.req, c.pos, c.seg, 2, 1, 16, 16, 0, 1.0, offsets=off, **kw)


@pytest.mark.parametrize("H,G,dim,dims,tail", [(6, 2, 40, 24, 48), (3, 1, 9, 6, 13), (16, 4, 128, 32, 1040), (2, 2, 20, 0, 7), (5, 5, 200, 16, 0)])
@pytest.mark.parametrize("dtype,form", [(BF, "rows"), (BF, "partials"), (F32, "rows")])
def test_values_that_are_keys_and_columns_beside(device, H, G, dim, dims, tail, dtype, form):
    """Cache rows [turned key | key as projected], and the columns of another mixer behind them as rows."""
    from sglang_amd import kernels as K
    from sglang_amd.layers.mixers import rotary_table

    g = torch.Generator().manual_seed(dim + tail)
    T, kd, cols = 11, dim + -dim % 8, (tail + 7) // 8 * 8
    pos, loc = torch.randint(0, 90, (T,), generator=g), torch.randperm(40, generator=g)[:T] + 1
    table = rotary_table(90, dims, 60.0, torch.device("cpu"), dict(factor=2.5)) if dims else None
    pad = lambda t: torch.cat([t, torch.zeros(*t.shape[:-1], kd - dim, dtype=t.dtype)], -1)
    q, k, rest = (torch.randn(*s, generator=g).to(dtype) for s in ((T, H, dim), (T, G, dim), (T, cols)))
    rows = torch.cat([pad(q).flatten(1), pad(k).flatten(1), rest, torch.zeros(T, 8, dtype=dtype)], 1)
    turn = lambda x: _turn(x.double(), table, pos, 0, dims) if dims else x.double()
    tol = 5e-3 if dtype == BF else 2e-6
    for plain in (False, True):
        cache = torch.full((42, 2 * G * kd), 3.0, dtype=dtype, device=device)
        got, beside = K.head_prepare(_source(K, rows, None, form, device), H, dim, kd, pos.to(device), table.to(device) if dims else None, 1e-6,
                                     gate_cols=cols, kv=(G, kd, cache, loc.to(device)), value_is_key=True, plain=plain)
        kc, vc = cache[loc.to(device)].view(T, G, 2 * kd).split(kd, -1)
        for out, ref in ((got.unflatten(1, (H, kd)), turn(q)), (kc, turn(k)), (vc, k)):
            assert _rel(out[..., :dim], ref) < tol and float(out[..., dim:].abs().sum()) == 0
        assert (beside is None) == (tail == 0) and (beside is None or _rel(beside, rest) < tol)


# ---------------------------------------------------------------------------------------------- matrix memory
class _Memory:
    """Requests of one head layout over dirty slots, advanced portion by portion."""

    def __init__(self, lens, H, D, V, dtype, device, cap=3.0, loud=1.0, seed=0):
        g = torch.Generator().manual_seed(seed)
        self.H, self.D, self.V, self.cap, self.dtype, self.device, self.scale = H, D, V, cap, dtype, device, D ** -0.5
        self.cols = [0, H * D, 2 * H * D, 2 * H * D + H * V, 2 * H * D + H * V + H, 2 * H * D + H * V + 2 * H]
        self.rows = []
        for n in lens:
            r = torch.randn(n, self.cols[-1] + (-self.cols[-1]) % 4 + 4, generator=g)
            r[:, self.cols[3]:] *= loud
            self.rows.append(r.to(dtype))
        self.bi, self.bf = torch.randn(H, generator=g) * 0.5, torch.randn(H, generator=g) + 2.0
        self.state = torch.full((len(lens) + 3, H, D, V), 7.0, device=device)
        self.norm = torch.full((len(lens) + 3, H, (V + 15) // 16, D + 1), -5.0, device=device)
        self.slots = (torch.randperm(len(lens) + 2, generator=g)[:len(lens)] + 1).to(device)
        self.at = [0] * len(lens)

    def want(self):
        out = []
        for r in self.rows:
            q, k, v, i, f = (r[:, a:b].double() for a, b in zip(self.cols, self.cols[1:]))
            T, cap = len(r), self.cap
            gi, gf = cap * torch.tanh((i + self.bi.double()) / cap), od.log_sigmoid(cap * torch.tanh((f + self.bf.double()) / cap))
            out.append(od.memory_recurrence(q.view(T, self.H, self.D) * self.scale, k.view(T, self.H, self.D), v.view(T, self.H, self.V), gi, gf).flatten(1))
        return out

    def step(self, counts, form):
        """Advance request b by counts[b] tokens (those with none are left out) -> their outputs, packed."""
        from sglang_amd import kernels as K

        who = [b for b, n in enumerate(counts) if n]
        x = torch.cat([self.rows[b][self.at[b]:self.at[b] + counts[b]] for b in who]).to(self.device)
        pos = torch.cat([torch.arange(self.at[b], self.at[b] + counts[b]) for b in who]).to(self.device)
        seg = K.Segments() if form == "single" else _segments([counts[b] for b in who], self.device)
        parts = [x[:, a:b] for a, b in zip(self.cols, self.cols[1:])]
        o = K.memory_scan(*parts, self.bi.to(self.device), self.bf.to(self.device), self.state, self.norm, self.slots[who].contiguous(), pos, seg, self.cap,
                          self.scale, form=None if form == "single" else form)
        for b in who:
            self.at[b] += counts[b]
        return o


def _close(got, want, dtype):
    """Keys of random signs make denominators that cancel now and then: single elements may be further off than all together."""
    return _err(got, want) < (2e-3 if dtype == F32 else 5e-2) and _rel(got, want) < (3e-5 if dtype == F32 else 4e-3)


@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("form", ["step", "chunk"])
@pytest.mark.parametrize("H,D,V,cap,loud", [(4, 64, 64, 3.0, 1.0), (2, 128, 128, 15.0, 4.0), (3, 20, 28, 9.0, 3.0), (1, 7, 3, 2.0, 1.0), (2, 192, 80, 12.0, 6.0), (5, 16, 200, 0.5, 1.0),
                                            (2, 33, 17, 30.0, 12.0)])
def test_memory_forms_match_the_recurrence(device, dtype, form, H, D, V, cap, loud):
    m = _Memory([150], H, D, V, dtype, device, cap, loud, seed=D)
    want = m.want()[0]
    for sizes in ([150], [1], [2], [7, 1, 33, 64], [31, 32, 1, 2], [90, 1, 1, 45]):
        m.at = [0]                                         # from position 0 over whatever the slot holds
        got = torch.cat([m.step([b - a], form) for a, b in _portions(150, sizes)])
        assert _close(got, want, dtype), sizes


@pytest.mark.parametrize("dtype", [F32, BF])
def test_memories_of_a_ragged_batch_and_both_forms_in_turn(device, dtype):
    """Requests advance by unequal portions, one left out now and then, step, chunk and single tokens in any order."""
    m = _Memory([120, 77, 33, 1], 3, 40, 72, dtype, device, 6.0, 2.0)
    want, left, got = m.want(), [120, 77, 33, 1], [[], [], [], []]
    plan = [("chunk", [40, 1, 2, 0]), ("step", [1, 30, 2, 1]), ("single", [1, 1, 1, 0]), ("chunk", [33, 32, 0, 0]), ("single", [1, 0, 1, 0]), ("step", [2, 13, 0, 0]),
            ("chunk", [42, 0, 27, 0])]
    for form, counts in plan:
        before = list(m.at)
        pieces = m.step(counts, form).cpu().split([n for n in counts if n])
        for b, piece in zip([b for b, n in enumerate(counts) if n], pieces):
            got[b].append(piece)
            assert m.at[b] == before[b] + len(piece)
    for b, rows in enumerate(got):
        assert _close(torch.cat(rows), want[b], dtype), b
    assert m.at == left
    untouched = [s for s in range(m.state.shape[0]) if s not in m.slots.tolist()]
    assert float((m.state[untouched] - 7).abs().max()) == 0 and float((m.norm[untouched] + 5).abs().max()) == 0


@pytest.mark.parametrize("form", ["step", "chunk"])
def test_memory_denominators_on_both_sides(device, form):
    """Input gates far below one keep |n.q| under e^-m, large ones lift it far above: the read-out is what the recurrence says, not what a plain
    normalization would.  (Positive keys and queries: no denominator cancels.)"""
    for shift, cap in ((-4.0, 6.0), (11.0, 12.0)):
        m = _Memory([70], 2, 16, 24, F32, device, cap)
        m.bi += shift
        m.rows[0][:, :m.cols[2]] = m.rows[0][:, :m.cols[2]].abs()
        want = m.want()[0]
        got = torch.cat([m.step([n], form) for n in (40, 30)])
        assert _close(got, want, F32), shift


# ---------------------------------------------------------------------------------------------- token shift
@pytest.mark.parametrize("dtype", [F32, BF])
@pytest.mark.parametrize("width", [64, 250, 1032, 4096])
def test_token_shift_portions_and_single_tokens(device, dtype, width):
    """Portions (the shift alone) and single tokens (the residual launch) of two requests in turn, over dirty state, twice."""
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(width)
    mu, norm, eps = _rand(g, width) * 0.4 + 0.5, _rand(g, width) * 0.3 + 1.0, 1e-5
    state, slots = torch.full((4, width), 7.0, dtype=dtype, device=device), torch.tensor([3, 1], device=device)
    for sizes in ([(5, 11), (1, 1), (2, 3), (1, 1), (1, 1), (6, 2)], [(1, 1), (1, 7), (9, 2), (1, 1)]):
        xs = [_rand(g, sum(s[i] for s in sizes), width) for i in (0, 1)]
        hs = [oh.rms_norm(x.double(), norm.double(), eps).to(dtype).double() for x in xs]
        want, at = [od.token_shift(h, mu.double()) for h in hs], [0, 0]
        for n in sizes:
            cut = lambda t: torch.cat([t[i][at[i]:at[i] + n[i]] for i in (0, 1)]).to(device)
            pos, h = cut([torch.arange(1000), torch.arange(1000)]), torch.empty((sum(n), width), dtype=dtype, device=device)
            if n == (1, 1):
                shift = K.TokenShift(mu.to(device), state, slots, pos)
                K.residual_rms(cut(xs).contiguous(), eps, add=(torch.zeros_like(h),), norm=norm.to(device), h=h, shift=shift)
            else:
                K.token_shift(cut(hs).to(dtype), mu.to(device), state, slots, pos, _segments(list(n), device), h)
            assert _err(h, cut(want).cpu()) < TOL[dtype] * 2, (sizes, n)
            at = [at[0] + n[0], at[1] + n[1]]
            for i in (0, 1):
                assert _err(state[slots[i]], hs[i][at[i] - 1]) < TOL[dtype]
        assert float((state[0] - 7).abs().max()) == 0 and float((state[2] - 7).abs().max()) == 0


# ---------------------------------------------------------------------------------------------- squared relu
@pytest.mark.parametrize("T,W,ff,E,top", [(5, 256, 128, 4, 2), (64, 256, 64, 6, 1), (300, 256, 128, 2, 2), (2100, 256, 256, 2, 2), (40, 102, 64, 5, 3), (33, 136, 96, 3, 2)])
@pytest.mark.parametrize("dtype", [BF, F32])
def test_experts_of_squared_relu_skip_identities(device, T, W, ff, E, top, dtype):
    from sglang_amd import kernels as K

    if dtype == F32 and T > 300:
        pytest.skip("the plain form is slow")
    g = torch.Generator().manual_seed(T)
    h, up, down = (torch.randn(*s, generator=g).to(dtype) for s in ((T, W), (E, ff, W), (E, W, ff)))
    up, down = up / W ** 0.5, down / ff ** 0.5
    ids = torch.stack([torch.randperm(E + 2, generator=g)[:top] for _ in range(T)])
    ids = torch.where(ids < E, ids, -1).int()
    act, rows = K.Pointwise(), torch.arange(T) if T <= 300 else torch.arange(0, T, 13)
    for plain in (False, True) if dtype == BF and T <= 300 else (False,):
        got = K.routed_experts(h.to(device), up.to(device), down.to(device), ids.to(device), plain, act).cpu()
        for t in rows.tolist():
            for k, e in enumerate(ids[t].tolist()):
                if e >= 0:
                    mid = (torch.clamp(h[t].double() @ up[e].double().T, min=0) ** 2).to(dtype).double()
                    assert _rel(got[t, k], mid @ down[e].double().T) < (1.5e-2 if dtype == BF else 1e-5), (t, k)


@pytest.mark.parametrize("M,N,Kd,splits", [(1, 256, 128, None), (17, 512, 256, 1), (64, 96, 1024, 4), (33, 4096, 2048, None), (100, 128, 256, 2)])
@pytest.mark.parametrize("bias", [False, True])
def test_squared_relu_behind_a_projection(device, M, N, Kd, splits, bias):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(N)
    x, w = torch.randn(M, Kd, generator=g).to(BF), (torch.randn(N, Kd, generator=g) / Kd ** 0.5).to(BF)
    b = torch.randn(N, generator=g).to(BF) if bias else None
    want = torch.clamp(x.double() @ w.double().T + (b.double() if bias else 0), min=0) ** 2
    got = K.wstream_gemm(x.to(device), w.to(device), b.to(device) if bias else None, splits=splits, act=K.Pointwise())
    assert _rel(got, want) < 5e-3
    with pytest.raises(Exception, match="does not fit"):
        K.wstream_gemm(x.to(device), w.to(device), epilogue="silu_and_mul", act=K.Pointwise())


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows,d", [(3, 8), (5, 37), (70, 4104), (2, 9000)])
def test_squared_relu_of_rows(device, rows, d, dtype):
    from sglang_amd import kernels as K

    wide = torch.randn(rows, d + 8, generator=torch.Generator().manual_seed(d)).to(dtype)
    x = wide.to(device)
    K.squared_relu_(x[:, :d])
    assert _rel(x[:, :d], torch.clamp(wide[:, :d].double(), min=0) ** 2) < (4e-3 if dtype == BF else 1e-6)
    assert torch.equal(x[:, d:].cpu(), wide[:, d:])


# ---------------------------------------------------------------------------------------------- router and residual launch
@pytest.mark.parametrize("T,width,E,identities,top,groups,keep", [(7, 64, 14, 2, 2, 2, 1), (40, 256, 8, 8, 3, 4, 2), (200, 100, 250, 3, 9, 5, 2), (33, 128, 64, 1, 4, 64, 9),
                                                                 (100, 512, 40, 0, 40, 1, 1), (5, 72, 1, 0, 1, 1, 1)])
@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("gate", [False, True])
def test_softmax_scores_within_groups_identities_and_a_gate(device, dtype, T, width, E, identities, top, groups, keep, gate):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(E + T)
    h, w = torch.randn(T, width, generator=g).to(dtype), (torch.randn(E + gate, width, generator=g) / width ** 0.5 * 2).to(dtype)
    c = torch.randn(E, generator=g) * 0.3 - 0.5                # choice scores of both signs
    weights, ids, *rest = K.moe_route(h.to(device), w.to(device), None, top, K.SoftmaxScores(c.to(device), groups, keep), identities, gate)
    od.margins.clear()
    want = od.route(h.double(), w[:E].double(), c.double(), dict(top=top, groups=dict(count=groups, keep=keep)))
    weights, ids = weights.cpu(), ids.cpu()
    s = torch.softmax(h.double() @ w[:E].double().T, -1)
    for t in range(T):
        chosen = [(e if e < E - identities else -1, float(p)) for e, p in want[t]]
        got = sorted(zip(ids[t].tolist(), weights[t].tolist()))
        assert [e for e, _ in got] == sorted(e for e, _ in chosen) and torch.allclose(torch.tensor([p for _, p in got]), torch.tensor(sorted(chosen))[:, 1].float(), rtol=1e-4, atol=1e-7) \
            or min(od.margins) < 1e-5, t
    assert (len(rest) == 1) == gate
    if gate:
        assert _rel(rest[0], od.sigmoid(h.double() @ w[E].double())) < 1e-5


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("rows,W", [(3, 64), (9, 250), (1100, 512), (1030, 2048), (1025, 4096), (5, 6144)])
def test_input_rows_row_factors_and_bias_of_the_residual(device, dtype, rows, W):
    """x + m * norm(sum of expert rows, input rows and a scaled part + bias), and the norm of that in the place of the input rows."""
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(rows)
    eps, top, m, n = 1e-4, 3, 0.3, min(rows, 40)
    x, h = _rand(g, rows, W), _rand(g, rows, W).to(dtype)
    data, wide = _rand(g, rows, top, W).to(dtype), torch.rand(rows, top + 1, generator=g)
    ids = torch.randint(-1, 3, (rows, top), generator=g).int()
    data[ids < 0] = float("nan")                               # never read
    shared, post, norm, bias = _rand(g, rows, W).to(dtype), _rand(g, W) * 0.2 + 1, _rand(g, W) * 0.2 + 1, _rand(g, W)
    items = torch.where((ids < 0)[..., None], h[:, None].double(), data.double())
    y = (items * wide[:, :top, None].double()).sum(1) + shared.double() * wide[:, top:].double() + bias.double()
    want = x.double() + m * oh.rms_norm(y, post.double(), eps)
    xd, hd, wd = x.to(device), h.to(device), wide.to(device)
    a = K.ExpertRows(data.to(device), wd[:, :top], ids.to(device), hd)
    K.residual_rms(xd, eps, add=(a, K.Scaled(shared.to(device), wd[:, top])), bias=bias.to(device), post=(post.to(device), m), norm=norm.to(device), h=hd)
    assert _err(xd, want) < 1e-4 and _err(hd, oh.rms_norm(want, norm.double(), eps)) < TOL[dtype] * 2
    # the scaled part as split-K partials
    parts = torch.randn(4, rows, W, generator=g)
    x2 = x.to(device)
    K.residual_rms(x2, eps, add=(shared.to(device), K.Scaled(K.Partials(parts.to(device), 4, rows, W, None), wd[:, top])), bias=bias.to(device))
    assert _err(x2, x.double() + shared.double() + parts.double().sum(0) * wide[:, top:].double() + bias.double()) < 1e-5


@pytest.mark.parametrize("dtype", [BF, F32])
@pytest.mark.parametrize("groups,size", [(1, 192), (3, 20), (4, 7), (32, 128), (2, 1000)])
def test_a_sigmoid_gate_behind_the_heads_norm(device, dtype, groups, size):
    from sglang_amd import kernels as K

    g = torch.Generator().manual_seed(groups * 1000 + size)
    n, rows, eps = groups * size, 9, 1e-5
    y, z, w = _rand(g, rows, n).to(dtype), _rand(g, rows, n + 12, scale=2.0).to(dtype)[:, 4:4 + n], _rand(g, n) + 1.0
    out = torch.zeros((rows, n + 16), dtype=dtype, device=device)
    K.gated_rmsnorm(y.to(device), z.to(device), w.to(device), groups, eps, gate_first=False, out=out[:, 8:8 + n], sigmoid_gate=True)
    assert _err(out[:, 8:8 + n], oh.grouped_rms_norm(y.double(), w.double(), groups, eps) * od.sigmoid(z.double())) < TOL[dtype] * 4
    assert float(out[:, :8].abs().sum()) == 0 and float(out[:, 8 + n:].abs().sum()) == 0
