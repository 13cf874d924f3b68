"""Dugalix without a GPU: configuration and registry, weight loading and padding, cache and state bookkeeping, rotation tables, the small
library's build list, and the plain oracle against closed forms and itself."""
import json
import math

import pytest
import torch
from safetensors.torch import save_file

from dugalix_cases import CASES, attention, config, dense, memory, moe, parallel
from oracle import dugalix as od
from sglang_amd import build, kernels
from sglang_amd.harness import registry
from sglang_amd.harness.dugalix import DugalixConfig, DugalixForCausalLM
from sglang_amd.harness.weights import SyntheticWeights, TensorWeights
from sglang_amd.layers.mixers import rotary_table
from sglang_amd.mem_cache.memory_pool import GroupedTokenToKVPool, HybridReqToTokenPool

CPU = torch.device("cpu")
F64 = torch.float64


@pytest.fixture(autouse=True)
def no_library_calls(monkeypatch):
    """Modules ask the library which forms exist for their sizes when they are built."""
    for name in ("grouped_attention_matrix_form", "grouped_prefill_supported"):
        monkeypatch.setattr(kernels, name, lambda *a: True)


@pytest.mark.parametrize("name", sorted(CASES))
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_registry_reads_a_model_folder(tmp_path, name, dtype):
    cfg, w = CASES[name], od.random_weights(CASES[name], 1)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    c = registry.load_config(tmp_path)
    assert isinstance(c, DugalixConfig) and registry.model_class(c) is DugalixForCausalLM and registry.unit_group(c) == "shifted"
    assert c.num_hidden_layers == len(cfg["layers"]) and c.residual_mult == cfg["residual_mult"] and c.eps == cfg["norm"]["eps"]
    m = DugalixForCausalLM(c, CPU, weights=TensorWeights.from_dir(tmp_path, CPU, dtype), dtype=dtype, max_context_len=64)
    assert torch.equal(m.norm, 1 + w["final.norm"].float()) and torch.equal(m.layers[0].norm1b, 1 + w["l0.norm1b"].float())
    up = lambda n: (n + 7) // 8 * 8
    pool, rows = m.create_kv_pool(128, 64, "auto", CPU, False), m.create_req_to_token_pool(3, 64, CPU)
    assert isinstance(pool, GroupedTokenToKVPool) and isinstance(rows, HybridReqToTokenPool) and not m.supports_prefix_cache
    states = iter(range(99))
    for i, ((layer, run), lay) in enumerate(zip(m.runs, cfg["layers"])):
        mx = lay["mixer"]
        a = mx if lay["type"] == "attention" else mx["left"]
        assert pool.get_kv_rows(i).shape == (192, a["kv_heads"] * (up(a["dim"]) + up(a["vdim"]))) and pool.get_kv_rows(i).dtype == dtype
        assert rows.state_pool.shift[i].shape == (4, cfg["width"]) and rows.state_pool.shift[i].dtype == dtype
        if lay["type"] == "attention":
            assert run == i
            continue
        r, k = mx["right"], next(states)
        assert run == (i, k) and rows.state_pool.state[k].shape == (4, r["heads"], r["dim"], r["vdim"])
        assert rows.state_pool.norm[k].shape == (4, r["heads"], (r["vdim"] + 15) // 16, r["dim"] + 1) and rows.state_pool.state[k].dtype == torch.float32
    assert len(rows.state_pool.state) == next(states) and rows.state_pool.size_bytes() > 0


def test_a_folder_that_does_not_fit_is_refused():
    cfg, w = CASES["mixed"], od.random_weights(CASES["mixed"], 2)
    c = DugalixConfig.from_dict(cfg)
    for gone in ("l0.shift", "l0.norm1b", "l0.mix.left.k.b", "l0.mix.left.o.b", "l0.mix.right.f.b", "l0.mlp.e6.down", "l0.mlp.shared.sg", "l0.mlp.correction", "l1.mix.pb", "l1.mlp.up"):
        with pytest.raises(KeyError, match=gone):
            DugalixForCausalLM(c, CPU, weights=TensorWeights({k: v for k, v in w.items() if k != gone}, CPU))
    with pytest.raises(ValueError, match="l0.mlp.router"):
        DugalixForCausalLM(c, CPU, weights=TensorWeights({**w, "l0.mlp.router": torch.ones(7, 160)}, CPU))
    for extra in ("l1.mix.v", "l1.mlp.gate", "l0.mlp.e7.up", "l2.norm2"):
        with pytest.raises(ValueError, match=extra):
            DugalixForCausalLM(c, CPU, weights=TensorWeights({**w, extra: torch.ones(3)}, CPU))
    with pytest.raises(ValueError, match="unknown mixer"):
        DugalixConfig.from_dict(config([dict(attention(), type="delta")]))
    with pytest.raises(ValueError, match="unknown feed-forward"):
        DugalixConfig.from_dict(config([attention(mlp=dict(kind="sparse"))]))
    wrong = attention()
    wrong["mixer"]["vdim"] = 32
    for bad in (wrong, attention(heads=5, kv_heads=2), attention(dims=7), parallel(dims=26), attention(mlp=moe(4, 1, 6, 8)), attention(mlp=moe(6, 2, 3, 8, (4, 1))),
                attention(mlp=moe(6, 1, 3, 8, (2, 1))), attention(mlp=moe(6, 2, 2, 8, (2, 3))), attention(mlp=moe(255, 1, 2, 8, shared=8))):
        with pytest.raises(ValueError):
            DugalixForCausalLM(DugalixConfig.from_dict(config([bad])), CPU, weights=SyntheticWeights(CPU))
    with pytest.raises(NotImplementedError):
        DugalixForCausalLM(c, CPU, tp_size=2)
    with pytest.raises(NotImplementedError):
        DugalixForCausalLM(c, CPU, weights=TensorWeights(w, CPU)).create_kv_pool(128, 64, "fp8_e4m3", CPU, False)


def test_named_models_and_synthetic_weights():
    assert isinstance(registry.named_config("dugalix-1b"), DugalixConfig) and "dugalix-8b" in registry.config_names()
    m = DugalixForCausalLM(DugalixConfig.from_dict(CASES["odd"]), CPU)
    assert float(m.layers[0].norm1.min()) == float(m.layers[0].norm1.max()) == 1.0 and float(m.layers[0].shift.abs().sum()) == 0.0


def test_projections_merge_and_pad():
    """Heads of 12 and 5 become 16 and 8; the memory's rows follow the attention's; one output projection over both."""
    cfg = CASES["odd"]
    w = od.random_weights(cfg, 3)
    m = DugalixForCausalLM(DugalixConfig.from_dict(cfg), CPU, weights=TensorWeights(w, CPU)).layers[1].mixer
    W, a = m.left.in_proj.weight.data, 2 * 16 + 16 + 8
    r = cfg["layers"][1]["mixer"]["right"]
    total = a + 2 * 3 * 7 + 2 * 3 * 11 + 2 * 3
    assert W.shape == (total + -total % 16, 102) and m.right.parts is None
    assert torch.equal(W[:12], w["l1.mix.left.q"][:12]) and float(W[12:16].abs().sum()) == 0 and torch.equal(W[48:53], w["l1.mix.left.v"])
    for name, at in (("q", 0), ("k", 21), ("v", 42), ("g", 75), ("i", 108), ("f", 111)):
        rows = w[f"l1.mix.right.{name}"]
        assert torch.equal(W[a + at:a + at + rows.shape[0]], rows) and m.right.starts[("q", "k", "v", "g", "i", "f").index(name)] == at
    assert torch.equal(m.left.in_proj.bias.data[48:53], w["l1.mix.left.v.b"]) and float(m.left.in_proj.bias.data[a:].abs().sum()) == 0
    o = m.o_proj.weight.data
    assert o.shape[1] == 2 * 8 + 33 + 7 and torch.equal(o[:, 16:49], w["l1.mix.right.o"]) and torch.equal(o[:, 8:13], w["l1.mix.left.o"][:, 5:]) and float(o[:, 49:].abs().sum()) == 0
    assert torch.allclose(m.out_bias, -0.7 * w["l1.mix.left.o.b"].float()) and torch.allclose(m.right.norm_weight, 0.4 * w["l1.mix.right.norm"].float())
    s = DugalixForCausalLM(DugalixConfig.from_dict(cfg), CPU, weights=TensorWeights(w, CPU)).layers[0].mixer
    assert s.in_proj.weight.shape == (3 * 16 + 16, 102) and s.value_is_key and s.cache_spec == (1, 16, 16) and torch.equal(s.offsets, w["l0.mix.pb"].float())


@pytest.mark.parametrize("dims,base", [(2, 10.0), (16, 1000.0), (64, 500000.0)])
@pytest.mark.parametrize("factor", [1.0, 8.0])
def test_rotation_tables_under_a_linear_scaling(dims, base, factor):
    t = rotary_table(300, dims, base, CPU, dict(factor=factor))
    x = torch.zeros(300, 1, dims, dtype=F64)
    x[..., :dims // 2] = 1.0                                   # the pair (1, 0) turns into (cos, sin)
    assert float((t.double() - od.rotate(x, dict(dims=dims, base=base, scaling=dict(factor=factor)))[:, 0]).abs().max()) < 1e-6


def test_unit_group_lists_existing_sources_and_not_the_rest():
    assert all(p.exists() for p in build.sources("shifted")) and len(build.sources("shifted")) < len(build.sources())


# ---------------------------------------------------------------------------------------------- the oracle
def test_oracle_visible_keys():
    assert od.visible(9, 3, 2) == [0, 1, 7, 8, 9] and od.visible(3, 3, 2) == [0, 1, 2, 3] and od.visible(1, 1, 5) == [0, 1] and od.visible(4, 1) == [4]


def test_oracle_sigmoid_weights_are_not_normalized():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(12, h, 4, generator=g, dtype=F64) for h in (4, 2, 2))
    off = torch.tensor([0.5, -1.0, 2.0, 0.0], dtype=F64)
    a = od.attend(q, k, v, 0.7, window=5, offsets=off)
    p = 1 / (1 + torch.exp(-(k[7:, 1] @ q[11, 2] * 0.7 + 2.0)))
    assert torch.allclose(a[11, 2], p @ v[7:, 1])


def test_oracle_memory_against_a_closed_form():
    """With the sums written out: S and n over all tokens, each weighted by its input gate and every forget gate behind it."""
    g = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn(9, 1, n, generator=g, dtype=F64) for n in (3, 3, 5))
    i, f = torch.randn(9, 1, generator=g, dtype=F64), od.log_sigmoid(torch.randn(9, 1, generator=g, dtype=F64))
    o = od.memory_recurrence(q, k, v, i, f)
    t, logs = 8, [float(i[j, 0] + f[j + 1:9, 0].sum()) for j in range(9)]
    m = max(logs + [float(f.sum())])                       # the running maximum starts at 0
    y = sum(math.exp(logs[j] - m) * (k[j, 0] @ q[t, 0]) * v[j, 0] for j in range(9))
    d = sum(math.exp(logs[j] - m) * (k[j, 0] @ q[t, 0]) for j in range(9))
    assert torch.allclose(o[t, 0], y / (max(abs(float(d)), math.exp(-m)) + 1e-6))


def test_oracle_token_shift_and_feed_forward():
    h = torch.tensor([[1.0, 2.0], [3.0, 5.0]], dtype=F64)
    assert od.token_shift(h, torch.tensor([0.5, 0.0], dtype=F64)).tolist() == [[0.5, 2.0], [2.0, 5.0]]
    w = {"up": torch.eye(2, dtype=F64), "down": torch.eye(2, dtype=F64)}
    assert od.feed_forward(torch.tensor([[-3.0, 2.0]], dtype=F64), w).tolist() == [[0.0, 4.0]]


def test_oracle_router_groups_identities_and_negative_scores():
    # groups {0 1} {2 3} {4 5}; 5 is an identity; the best member decides a group, closed members lose to negative ones
    z, eye = torch.tensor([[2.0, -8.0, 1.0, 0.9, -1.0, -1.5]], dtype=F64), torch.eye(6, dtype=F64)
    s = torch.softmax(z[0], 0)
    c = torch.full((6,), -2.0, dtype=F64)
    got = od.route(z, eye, c, dict(top=3, groups=dict(count=3, keep=2)))[0]
    assert [e for e, _ in got] == [0, 2, 3] and math.isclose(float(got[1][1]), float(s[2]))
    c[5] = 1.0
    got = od.route(z, eye, c, dict(top=2, groups=dict(count=3, keep=1)))[0]
    assert [e for e, _ in got] == [5, 4] and math.isclose(float(got[0][1]), float(s[5]))
    w = {"router": eye, "correction": c, **{f"e{e}.{n}": torch.full((6, 6), float(e + 1), dtype=F64) for e in range(5) for n in ("up", "down")}}
    y = od.moe(z, w, dict(router=dict(experts=5, identity=1, top=1, groups=dict(count=3, keep=1))))
    assert torch.allclose(y, s[5] * z)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_oracle_is_causal_and_the_token_in_front_matters(name):
    cfg = CASES[name]
    w = od.random_weights(cfg, 3)
    g = torch.Generator().manual_seed(0)
    ids = torch.randint(0, cfg["vocab"], (30,), generator=g).tolist()
    full, tr = od.forward(cfg, w, ids)
    part, _ = od.forward(cfg, w, ids[:17])
    assert torch.allclose(full[:17], part, atol=1e-9) and len(tr) == len(cfg["layers"])
    changed = list(ids)
    changed[3] = (changed[3] + 1) % cfg["vocab"]
    other, _ = od.forward(cfg, w, changed)
    assert torch.equal(other[:3], full[:3]) and float((other[3:] - full[3:]).abs().max()) > 1e-3
    # one layer whose window is the token itself: what reaches the next one comes through the shift
    one = config([attention(window=1, mlp=dense(16))])
    w = od.random_weights(one, 1)
    a, b = (od.forward(one, w, s)[0] for s in ([3, 5, 8], [4, 5, 8]))
    assert float((a[1] - b[1]).abs().max()) > 1e-3 and torch.equal(a[2], b[2])


@pytest.mark.parametrize("name", sorted(CASES))
def test_routers_of_the_test_models_have_clear_choices(name):
    cfg = CASES[name]
    od.margins.clear()
    od.forward(cfg, od.random_weights(cfg, 7), [(i * 31 + 7) % cfg["vocab"] for i in range(60)])
    assert not od.margins or min(od.margins) > 2e-3
