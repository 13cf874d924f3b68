"""Dugalix through the framework's engine on the GPU, against the plain evaluation of whole sequences (oracle/dugalix.py): whole
prompts, portions down to two tokens, token-by-token and long decoding (graph and eager), mixed batches of unequal requests,
pages, rows and states freed and used again, and greedy generation through Engine.generate and the command line."""
import json
import random
import subprocess
import sys
from pathlib import Path

import pytest
import torch

from dugalix_cases import CASES, attention, config, dense, memory, moe, parallel
from oracle import dugalix as od
from oracle import hybrid as oh

pytestmark = pytest.mark.gpu
ROOT = Path(__file__).resolve().parent.parent
# rms error of a logits row over the rms of the logits: fp32 rounding, and bf16 projections / activations over the layers.  A
# 16-bit position may go up to three times as far as the oracle itself moves when it rounds what the product rounds (the
# largest of four draws).
BAR = {torch.float32: 5e-5, torch.bfloat16: 3e-2}
FORMS = [(torch.float32, None), (torch.bfloat16, None), (torch.bfloat16, "rows"), (torch.bfloat16, "prefill"), (torch.bfloat16, "plain")]
LENS = [170, 1, 33]
_ORACLE, _SLACK = {}, {}


def _row_error(got, want):
    d = got - want
    return (d - d.mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.pow(2).mean().sqrt()


def _evaluate(cfg, w, s):
    od.margins.clear()
    rows, _ = od.forward(cfg, w, s)
    assert not od.margins or min(od.margins) > 2e-3            # no expert is chosen by a hair
    draws = []
    for grid in (1.0, 1.19, 1.41, 1.68):
        with oh.rounding(torch.bfloat16, grid):
            draws.append(_row_error(od.forward(cfg, w, s)[0], rows))
    _SLACK[rows.data_ptr()] = 3 * torch.stack(draws).max(0).values
    return rows


def _case(name, lens, seed=7):
    """(config, weights, token lists, oracle logits per sequence), evaluated once per session."""
    key = (name, tuple(lens), seed)
    if key not in _ORACLE:
        cfg = CASES[name]
        w = od.random_weights(cfg, seed)
        rnd = random.Random(seed)
        seqs = [[rnd.randrange(cfg["vocab"]) for _ in range(n)] for n in lens]
        _ORACLE[key] = (cfg, w, seqs, [_evaluate(cfg, w, s) for s in seqs])
    return _ORACLE[key]


def _engine(cfg, w, device, dtype, *, tokens=1024, reqs=4, page=64, graph=False, form=None, ctx=512):
    from sglang_amd.harness.dugalix import DugalixConfig
    from sglang_amd.harness.engine import Engine, ModelRunner
    from sglang_amd.harness.weights import TensorWeights

    r = ModelRunner(DugalixConfig.from_dict(cfg), max_total_tokens=tokens, max_running_requests=reqs, max_context_len=ctx, page_size=page,
                    device=device, use_graph=graph, weights=TensorWeights(w, device, dtype), dtype=dtype)
    r.attn_backend.grouped_form = form
    return Engine(r)


def _check(got, want, dtype, what, slack):
    bar = torch.clamp(slack, min=BAR[dtype]) if dtype == torch.bfloat16 else BAR[dtype]
    e = _row_error(got.double().cpu(), want.double()) / bar
    assert float(e.max()) < 1, (what, float(e.max()), int(e.argmax()))


def _req(i):
    from sglang_amd.harness.engine import Req

    return Req(i, [], 0)


def _drive(eng, seqs, plan, want_rows, dtype, what):
    """plan: steps of [(sequence, count)]; every position's logits are compared.  Requests end with their last token."""
    live, at, zero = {}, {}, torch.zeros(1)
    for n, step in enumerate(plan):
        reqs, toks = [], []
        for i, c in step:
            lo = at.get(i, 0)
            live[i] = live.get(i) or _req(i)
            reqs.append(live[i])
            toks.append(seqs[i][lo:lo + c])
            at[i] = lo + len(toks[-1])
        got = eng.advance(reqs, toks, [list(range(len(t))) for t in toks])
        ref = torch.cat([want_rows[i][at[i] - len(t):at[i]] for (i, _), t in zip(step, toks)])
        slack = torch.cat([_SLACK.get(want_rows[i].data_ptr(), zero.expand(len(seqs[i])))[at[i] - len(t):at[i]] for (i, _), t in zip(step, toks)])
        _check(got, ref, dtype, (what, n, step), slack)
        done = [i for i, _ in step if at[i] == len(seqs[i])]
        eng.release([live.pop(i) for i in done])
        for i in done:
            at.pop(i)


@pytest.mark.parametrize("dtype,form", FORMS)
@pytest.mark.parametrize("name", sorted(CASES))
def test_layers_and_whole_prompts(device, name, dtype, form):
    cfg, w, seqs, want = _case(name, LENS)
    eng = _engine(cfg, w, device, dtype, form=form)
    eng.r.model.layer_trace = []
    _drive(eng, seqs, [[(0, 170)]], want, dtype, name)
    _, trace = od.forward(cfg, w, seqs[0])
    assert len(trace) == len(eng.r.model.layer_trace)
    for k, (got, ref) in enumerate(zip(eng.r.model.layer_trace, trace)):
        e = (got.double().cpu() - ref).pow(2).mean().sqrt() / ref.pow(2).mean().sqrt()
        assert float(e) < BAR[dtype], (k, float(e))
    eng.r.model.layer_trace = None
    _drive(eng, seqs, [[(1, 1), (2, 33)]], want, dtype, name)


@pytest.mark.parametrize("name", ["mixed", "tiles"])
def test_experts_without_matrix_instructions(device, name):
    cfg, w, seqs, want = _case(name, LENS)
    eng = _engine(cfg, w, device, torch.bfloat16)
    for layer in eng.r.model.layers:
        if hasattr(layer.mlp, "plain_experts"):
            layer.mlp.plain_experts = True
    _drive(eng, seqs, [[(0, 169)], [(0, 1)]], want, torch.bfloat16, name)


@pytest.mark.parametrize("dtype,form", FORMS)
@pytest.mark.parametrize("name", sorted(CASES))
@pytest.mark.parametrize("sizes", [[2], [3, 64, 2, 1], [50, 49, 51], [17, 1, 1, 90]])
def test_portions_equal_the_whole(device, name, dtype, form, sizes):
    cfg, w, seqs, want = _case(name, LENS)
    eng = _engine(cfg, w, device, dtype, form=form)
    plan, at, k = [], 0, 0
    while at < 170:
        plan.append([(0, min(sizes[k % len(sizes)], 170 - at))])
        at, k = at + plan[-1][0][1], k + 1
    _drive(eng, seqs, plan, want, dtype, (name, sizes))


@pytest.mark.parametrize("dtype", list(BAR))
@pytest.mark.parametrize("name,graph", [("mixed", True), ("odd", True), ("tiles", True), ("flat", False)])
def test_long_decoding_from_the_first_token(device, name, dtype, graph):
    """Every position decoded alone behind a one-token prompt, past every small window and several pages."""
    cfg, w, seqs, want = _case(name, LENS)
    _drive(_engine(cfg, w, device, dtype, graph=graph), seqs, [[(0, 1)]] * 170, want, dtype, name)


@pytest.mark.parametrize("dtype", list(BAR))
@pytest.mark.parametrize("name,page", [("mixed", 64), ("odd", 1), ("tiles", 16)])
def test_mixed_batches_reuse_pages_and_rows(device, name, dtype, page):
    """Four live requests over a pool that the whole trace would not fit in: portions beside single tokens, requests left out of
    steps, ended and replaced; each position equals its request's alone."""
    lens = [130, 70, 9, 1, 101, 66, 40, 2, 88, 120, 95]
    cfg, w, seqs, want = _case(name, lens)
    rnd = random.Random(5)
    plan, left, live, queue = [], dict(enumerate(lens)), [], list(range(len(lens)))
    while queue or live:
        while queue and len(live) < 4:
            live.append(queue.pop(0))
        picked = [i for i in live if rnd.random() < 0.8] or live[:1]
        step = []
        for i in picked:
            c = min(left[i], 1 if left[i] < lens[i] and rnd.random() < 0.5 else rnd.choice([2, 5, 17, 40, 64]))
            step.append((i, c))
            left[i] -= c
        live = [i for i in live if left[i]]
        plan.append(step)
    eng = _engine(cfg, w, device, dtype, tokens=10 * 64, page=page, graph=True)
    assert eng.r.token_to_kv_pool.size < sum(lens)
    for _ in range(2):
        _drive(eng, seqs, plan, want, dtype, (name, page))
    assert eng.r.req_to_token_pool.available_size() == 4
    assert eng.r.token_to_kv_pool_allocator.available_size() == eng.r.token_to_kv_pool.size


def _moves(cfg, w, ids, dtype, change, rows, least=5):
    """The oracle's rows, after making sure that `change`, applied to a copy of the configuration and weights, moves at least `least` of
    the logits rows `rows` by more than twice the bar."""
    want = _evaluate(cfg, w, ids)
    c2, w2 = json.loads(json.dumps(cfg)), dict(w)
    change(c2, w2)
    moved = _row_error(od.forward(c2, w2, ids)[0], want)
    bar = torch.clamp(_SLACK[want.data_ptr()], min=BAR[dtype]) if dtype == torch.bfloat16 else torch.full_like(moved, BAR[dtype])
    assert int((moved[rows] > 2 * bar[rows]).sum()) >= least, float((moved / bar)[rows].max())
    return want


def _set(*path):
    *path, value = path

    def change(cfg, w):
        at = cfg["layers"][0]
        for p in path[:-1]:
            at = at[p]
        at[path[-1]] = value
    return change


LOUD = dict(right=memory(2, 12, 12), scales=(1.0, 0.3), factor=1.0)


@pytest.mark.parametrize("dtype", list(BAR))
@pytest.mark.parametrize("lay,change,first", [
    (attention(window=37, scale=3.0, mlp=dense(64)), _set("mixer", "mask", "size", 38), 37),
    (attention(window=64, scale=3.0, mlp=dense(64)), _set("mixer", "mask", "size", 63), 63),
    (parallel(window=37, first=3, scale=4.0, mlp=dense(64), **LOUD), _set("mixer", "left", "mask", "size", 38), 40),
    (parallel(window=5, first=11, scale=4.0, mlp=dense(64), **LOUD), _set("mixer", "left", "mask", "keep_first", 10), 16),
    (parallel(window=5, first=11, scale=4.0, mlp=dense(64), **LOUD), _set("mixer", "left", "mask", "keep_first", 12), 17),
    (parallel(window=9, first=64, scale=4.0, mlp=dense(64), **LOUD), _set("mixer", "left", "mask", "keep_first", 65), 74),
], ids=["sigmoid-37", "sigmoid-64", "softmax-37", "first-11-out", "first-11-in", "first-64-in"])
def test_every_edge_shows_in_the_logits(device, lay, change, first, dtype):
    """One layer whose scale makes single scores stand out: moving a window or the number of kept tokens by one changes the oracle's logits
    by far more than the bar, and the product agrees with the right one, in prompts, in portions and in decoding."""
    cfg = config([lay], width=128)
    w = od.random_weights(cfg, 3)
    ids = [(i * 37 + 11) % cfg["vocab"] for i in range(120)]
    want = _moves(cfg, w, ids, dtype, change, slice(first, None))
    for plan in ([[(0, 120)]], [[(0, 12)]] + [[(0, 1)]] * 54 + [[(0, 2)]] * 3 + [[(0, 48)]], [[(0, 1)]] * 120):
        _drive(_engine(cfg, w, device, dtype), [ids], plan, [want], dtype, "edge")


def _zero(*names):
    return lambda c, w: w.update({"l0." + n: torch.zeros_like(w["l0." + n]) for n in names})


@pytest.mark.parametrize("dtype", list(BAR))
@pytest.mark.parametrize("lay,change", [
    (attention(mlp=dense(64)), lambda c, w: w.update({"l0.mix.pb": w["l0.mix.pb"].flip(0)})),
    (attention(mlp=dense(64)), _zero("shift")),
    (attention(), lambda c, w: c.update(residual_mult=0.7)),
    (parallel(mlp=dense(64)), lambda c, w: w.update({"l0.mix.left.k.b": -w["l0.mix.left.k.b"]})),
    (parallel(mlp=dense(64)), _zero("mix.left.v.b")),
    (parallel(mlp=dense(64)), _zero("mix.left.o.b")),
    (parallel(scale=0.8, mlp=dense(64)), _set("mixer", "left", "rot", "scaling", "factor", 5.0)),
    (parallel(mlp=dense(64)), _set("mixer", "left_scale", 0.9)),
    (parallel(mlp=dense(64)), _set("mixer", "right_scale", 0.9)),
    (parallel(mlp=dense(64)), _set("mixer", "right", "gate_cap", 1.2)),
    (parallel(mlp=dense(64)), _zero("mix.right.f.b")),
    (parallel(mlp=dense(64)), _zero("mix.right.i")),
    (parallel(mlp=dense(64)), _zero("mix.right.g")),
    (parallel(mlp=moe(6, 2, 2, 40, (2, 1), 48)), _zero("mlp.shared.sg")),
    (parallel(mlp=moe(6, 2, 3, 40, (4, 2), 48)), _set("mlp", "router", "groups", "keep", 3)),
    (parallel(mlp=moe(5, 3, 2, 40)), lambda c, w: w.update({"l0.mlp.correction": w["l0.mlp.correction"].flip(0) * 8})),
], ids=["offset", "shift", "residual", "key-bias", "value-bias", "output-bias", "factor", "left", "right", "cap", "forget-bias", "input-gate", "gate",
        "shared-gate", "groups", "correction"])
def test_every_constant_shows_in_the_logits(device, lay, change, dtype):
    cfg = config([lay], width=128)
    w = od.random_weights(cfg, 5)
    ids = [(i * 29 + 5) % cfg["vocab"] for i in range(90)]
    want = _moves(cfg, w, ids, dtype, change, slice(1, None))
    for plan in ([[(0, 90)]], [[(0, 2)], [(0, 30)]] + [[(0, 1)]] * 10 + [[(0, 3)], [(0, 45)]]):
        _drive(_engine(cfg, w, device, dtype), [ids], plan, [want], dtype, "constants")


@pytest.mark.parametrize("dtype", list(BAR))
def test_states_survive_every_cut_and_belong_to_one_request(device, dtype):
    """Portions that begin behind a page's last token, rows and states that belonged to others, a request left out of steps: the token in
    front and the memory are the sequence's own.  Shifts near one, forget gates that stay open and a loud right side make others show."""
    cfg = config([parallel(right=memory(3, 16, 24, 8.0), scales=(0.3, 1.5), mlp=dense(64)), attention(mlp=None)], width=128)
    w = od.random_weights(cfg, 6)
    w["l0.shift"], w["l1.shift"] = torch.full_like(w["l0.shift"], 0.9), torch.full_like(w["l1.shift"], 1.1)
    w["l0.mix.right.f.b"] = torch.full_like(w["l0.mix.right.f.b"], 5.0)
    seqs = [[(i * k + 3) % cfg["vocab"] for i in range(n)] for n, k in ((100, 31), (70, 17), (3, 5), (66, 7))]
    want = [_evaluate(cfg, w, s) for s in seqs]
    plan = [[(0, 64), (1, 1)], [(0, 1), (1, 2)], [(1, 61)], [(0, 2), (1, 1), (2, 1)], [(1, 5), (2, 2)], [(3, 2), (0, 1)], [(3, 64), (0, 32)]]
    eng = _engine(cfg, w, device, dtype, tokens=5 * 64, reqs=3, graph=True)
    for _ in range(3):
        _drive(eng, seqs, plan, want, dtype, "states")
        for _ in range(2):
            eng.advance([q := _req("x")], [[7] * 90])          # somebody else's tokens in the freed pages, rows and states
            eng.release([q])


@pytest.mark.parametrize("dtype", list(BAR))
@pytest.mark.parametrize("graph,page,chunk", [(True, 1, 0), (False, 1, 0), (True, 64, 0), (True, 1, 24)])
def test_greedy_generation_through_the_scheduler(device, dtype, graph, page, chunk):
    """Engine.generate on three unequal prompts: every generated token is the oracle's arg-max over the same context, or a near
    tie of it; everything is given back at the end, and nothing is taken from the prefix tree (a state cannot be rewound)."""
    from sglang_amd.harness.engine import Req

    cfg, w, seqs, _ = _case("mixed", [61, 5, 33], seed=9)
    eng = _engine(cfg, w, device, dtype, graph=graph, page=page)
    for _ in range(2):
        reqs = [Req(i, list(s), 20 - 3 * i) for i, s in enumerate(seqs)]
        eng.generate(reqs, chunked_prefill_size=chunk)
        for q, s in zip(reqs, seqs):
            assert len(q.output_ids) == q.max_new_tokens and q.cached_tokens == 0
            rows, _ = od.forward(cfg, w, s + q.output_ids[:-1])
            rows = rows[len(s) - 1:]
            gap = rows.max(-1).values - rows[torch.arange(len(rows)), torch.tensor(q.output_ids)]
            assert float(gap.max()) < BAR[dtype] * 12 * float(rows.pow(2).mean().sqrt()), gap
        assert eng.r.req_to_token_pool.available_size() == 4
        assert eng.r.token_to_kv_pool_allocator.available_size() == eng.r.token_to_kv_pool.size


def test_mixed_step_and_retraction_keep_the_outputs(device):
    """A request that joins a running batch (mixed step) and one that a full pool pushes out and prefills again generate what they
    generate alone."""
    from sglang_amd.harness.engine import Req

    cfg, w, seqs, _ = _case("mixed", [61, 5, 33], seed=9)
    alone = []
    eng = _engine(cfg, w, device, torch.float32)
    for i, s in enumerate(seqs):
        q = Req(i, list(s), 24)
        eng.generate([q])
        alone.append(q.all_output_ids)
    eng = _engine(cfg, w, device, torch.float32, page=1)
    a, b = Req(0, list(seqs[0]), 24), Req(1, list(seqs[1]), 24)
    eng.prefill([a])
    for _ in range(3):
        eng.decode_step()
    eng.mixed_step([b])
    while eng.running:
        eng.flush_decode_outputs()
        done = [q for q in eng.running if q.finished()]
        if done:
            eng.finish(done)
        else:
            eng.decode_step()
    assert a.output_ids == alone[0] and b.output_ids == alone[1]
    eng = _engine(cfg, w, device, torch.float32, tokens=130, page=1)
    reqs = [Req(i, list(s), 24) for i, s in enumerate(seqs)]
    eng.generate(reqs)
    assert eng.stats.get("retracted", 0) > 0 and [q.all_output_ids for q in reqs] == alone


def test_graph_replays_equal_eager_steps(device):
    """The same decode steps replayed (with eager work between them) and run eagerly, padded batches included."""
    cfg, w, seqs, _ = _case("tiles", [40, 25, 60], seed=4)
    runs = []
    for graph in (True, False):
        eng = _engine(cfg, w, device, torch.bfloat16, graph=graph)
        reqs = [_req(i) for i in range(3)]
        out = [eng.advance(reqs, [s[:20] for s in seqs])]
        for k in range(20, 25):
            out.append(eng.advance(reqs, [[s[k]] for s in seqs]).clone())
            out.append(eng.advance(reqs[:1], [[seqs[0][k + 5]]]).clone() if k == 22 else torch.randn(64, device=device)[:0])
        runs.append([o for o in out if o.numel()])
    for x, y in zip(*runs):
        assert float((x.double() - y.double()).pow(2).mean().sqrt() / y.double().pow(2).mean().sqrt()) < 1e-2


def test_sampling_follows_its_seeds(device):
    from sglang_amd.harness.engine import Req
    from sglang_amd.layers.sampler import SamplingBatchInfo

    cfg, w, seqs, _ = _case("mixed", [61, 5, 33], seed=9)
    eng = _engine(cfg, w, device, torch.bfloat16, graph=True, page=1)

    def run(seed):
        f = lambda v, dt=torch.float32: torch.full((3,), v, dtype=dt, device=device)
        info = SamplingBatchInfo(f(1.0)[:, None], f(0.9), f(40, torch.int32), f(0.0), False, True, True, False, torch.arange(seed, seed + 3, device=device))
        reqs = [Req(i, list(s), 12) for i, s in enumerate(seqs)]
        eng.generate(reqs, info)
        return [q.all_output_ids for q in reqs]

    a, b = run(5), run(1000)
    assert a != b and all(0 <= t < cfg["vocab"] for ids in a for t in ids)


def test_command_line_generates_from_a_model_folder(device, tmp_path):
    from safetensors.torch import save_file

    cfg, w, seqs, _ = _case("mixed", [61, 5, 33], seed=9)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    cmd = [sys.executable, "-m", "sglang_amd.harness.cli", "--model", str(tmp_path), "--dtype", "float32", "--max-new-tokens", "6", "--no-graph"]
    for s in seqs[:2]:
        cmd += ["--prompt-ids", ",".join(map(str, s))]
    out = subprocess.run(cmd, cwd=ROOT, capture_output=True, text=True, timeout=100)
    assert out.returncode == 0, out.stderr[-800:]
    lines = [[int(t) for t in x.split(",")] for x in out.stdout.strip().splitlines()[-2:]]
    for s, ids in zip(seqs, lines):
        rows, _ = od.forward(cfg, w, s + ids[:-1])
        assert rows[len(s) - 1:].argmax(-1).tolist() == ids
