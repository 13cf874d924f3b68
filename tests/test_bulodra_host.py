"""Bulodra without a GPU: configuration and registry, weight loading and padding, cache bookkeeping, rotation tables, the small library's
build list, and the plain oracle against closed forms and itself."""
import json
import math

import pytest
import torch
from safetensors.torch import save_file

from bulodra_cases import CASES, YARN, attention, capped, config, dense, latent, moe
from oracle import bulodra as ob
from oracle import hybrid as oh
from sglang_amd import build, kernels
from sglang_amd.harness import registry
from sglang_amd.harness.bulodra import BulodraConfig, BulodraForCausalLM
from sglang_amd.harness.weights import SyntheticWeights, TensorWeights
from sglang_amd.layers.mixers import rotary_table
from sglang_amd.mem_cache.memory_pool import LayeredTokenToKVPool

CPU = torch.device("cpu")
F64 = torch.float64


@pytest.fixture(autouse=True)
def no_library_calls(monkeypatch):
    """Modules ask the library which forms exist for their sizes when they are built."""
    for name in ("grouped_attention_matrix_form", "grouped_prefill_supported", "latent_prefill_supported"):
        monkeypatch.setattr(kernels, name, lambda *a: True)


@pytest.mark.parametrize("name", sorted(CASES))
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_registry_reads_a_model_folder(tmp_path, name, dtype):
    cfg, w = CASES[name], ob.random_weights(CASES[name], 1)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    c = registry.load_config(tmp_path)
    assert isinstance(c, BulodraConfig) and registry.model_class(c) is BulodraForCausalLM and registry.unit_group(c) == "layered"
    assert c.num_hidden_layers == len(cfg["layers"]) and (c.residual_mult, c.logit_scale) == (cfg["residual_mult"], cfg["logit_scale"])
    m = BulodraForCausalLM(c, CPU, weights=TensorWeights.from_dir(tmp_path, CPU, dtype), dtype=dtype, max_context_len=64)
    assert torch.equal(m.norm, w["final.norm"].float() * cfg["logit_scale"])
    pool = m.create_kv_pool(128, 64, "auto", CPU, False)
    assert isinstance(pool, LayeredTokenToKVPool) and pool.slot_ids.numel() == 192 and pool.get_kv_size_bytes()[0] > 0
    up = lambda n, k: (n + k - 1) // k * k
    seen = {True: 0, False: 0}
    for (layer, run_id), lay in zip(m.runs, cfg["layers"]):
        mx, lat = lay["mixer"], lay["type"] == "latent_attention"
        assert run_id == seen[lat]
        seen[lat] += 1
        rows = pool.get_latent_buffer(run_id) if lat else pool.get_kv_rows(run_id)
        width = up(mx["kv_rank"] + mx["rot_dim"], 32) if lat else mx["kv_heads"] * (up(mx["dim"], 8) + up(mx["vdim"], 8))
        assert rows.shape == (192, width) and rows.dtype == dtype and float(rows.abs().sum()) == 0


def test_a_folder_that_does_not_fit_is_refused():
    cfg, w = CASES["mixed"], ob.random_weights(CASES["mixed"], 2)
    c = BulodraConfig.from_dict(cfg)
    for gone in ("bigram", "l0.mix.g", "l1.mix.q.b", "l1.mix.k.norm", "l1.mix.sink", "l1.mlp.correction", "l1.mlp.e11.down", "l1.mlp.shared.up", "l2.mix.dq.norm"):
        with pytest.raises(KeyError, match=gone):
            BulodraForCausalLM(c, CPU, weights=TensorWeights({k: v for k, v in w.items() if k != gone}, CPU))
    with pytest.raises(ValueError, match="bigram"):
        BulodraForCausalLM(c, CPU, weights=TensorWeights({**w, "bigram": torch.ones(53, 160)}, CPU))
    with pytest.raises(ValueError, match="l0.mix.sink"):
        BulodraForCausalLM(c, CPU, weights=TensorWeights({**w, "l0.mix.sink": torch.ones(6)}, CPU))
    with pytest.raises(ValueError, match="unknown mixer"):
        BulodraConfig.from_dict(config([dict(capped(), type="delta")]))
    with pytest.raises(ValueError, match="unknown feed-forward"):
        BulodraConfig.from_dict(config([capped(mlp=dict(kind="sparse"))]))
    for bad in (capped(heads=5, kv_heads=2), capped(mlp=moe(4, 5, 8)), capped(mlp=moe(8, 3, 8, (3, 1))), capped(mlp=moe(8, 3, 8, (4, 1))),
                capped(mlp=moe(8, 3, 8, (4, 5))), capped(dims=7), capped(dims=26), latent(rot_dim=7)):
        with pytest.raises(ValueError):
            BulodraForCausalLM(BulodraConfig.from_dict(config([bad])), CPU, weights=SyntheticWeights(CPU))
    with pytest.raises(NotImplementedError):
        BulodraForCausalLM(c, CPU, tp_size=2)
    with pytest.raises(NotImplementedError):
        BulodraForCausalLM(c, CPU, weights=TensorWeights(w, CPU)).create_kv_pool(128, 64, "fp8_e4m3", CPU, False)


def test_named_models_and_synthetic_weights():
    assert isinstance(registry.named_config("bulodra-1b"), BulodraConfig) and "bulodra-8b" in registry.config_names()
    m = BulodraForCausalLM(BulodraConfig.from_dict(CASES["odd"]), CPU)
    assert float(m.layers[0].norm1.min()) == 1.0 and float(m.layers[0].mlp.scores.correction.abs().sum()) == 0.0


def test_projections_are_padded_with_zeros():
    """Heads of 9 and 11 become 16 and 16 everywhere: rows, biases, norms and the output projection's columns."""
    cfg = CASES["odd"]
    w = ob.random_weights(cfg, 3)
    m = BulodraForCausalLM(BulodraConfig.from_dict(cfg), CPU, weights=TensorWeights(w, CPU)).layers[0].mixer
    W = m.in_proj.weight.data
    assert W.shape == (80, 102) and m.in_proj.bias.shape == (80,) and m.o_proj.weight.shape == (102, 48)
    assert torch.equal(W[16:25], w["l0.mix.q"][9:18]) and float(W[25:32].abs().sum()) == 0 and torch.equal(W[48:57], w["l0.mix.k"])
    assert torch.equal(m.in_proj.bias.data[48:57], w["l0.mix.k.b"]) and float(m.in_proj.bias.data[57:64].abs().sum()) == 0
    assert m.norms[0].tolist() == w["l0.mix.q.norm"].float().tolist() + [0.0] * 7
    g = BulodraForCausalLM(BulodraConfig.from_dict(cfg), CPU, weights=TensorWeights(w, CPU)).layers[1].mixer
    assert torch.equal(g.in_proj.weight.data[2 * 16 + 16 + 8:][:2], w["l1.mix.g"]) and g.gate_cols == 2


@pytest.mark.parametrize("scaling", [None, YARN, dict(factor=1.0, original=100, fast=4.0, slow=1.0), dict(factor=3.0, original=7, fast=64.0, slow=0.5),
                                     dict(factor=16.0, original=4096, fast=32.0, slow=1.0)])
@pytest.mark.parametrize("dims,base", [(2, 10.0), (16, 1000.0), (64, 500000.0)])
def test_rotation_tables(dims, base, scaling):
    t = rotary_table(300, dims, base, CPU, scaling)
    f, factor = ob.frequencies(dims, base, scaling)
    a = torch.arange(300, dtype=F64)[:, None] * torch.tensor(f, dtype=F64)
    assert float((t.double() - factor * torch.cat([a.cos(), a.sin()], 1)).abs().max()) < 1e-6


def test_unit_group_lists_existing_sources_and_not_the_rest():
    assert all(p.exists() for p in build.sources("layered")) and len(build.sources("layered")) < len(build.sources())
    assert len({build.lib_path(g) for g in build.UNIT_GROUPS} | {build.lib_path()}) == len(build.UNIT_GROUPS) + 1


# ---------------------------------------------------------------------------------------------- the oracle
def test_oracle_bigram_rows():
    assert ob.bigram_rows([3, 5, 5, 0], 10, 1, 7) == [7, 35 % 7, 55 % 7, 50 % 7]


def test_oracle_frequencies_fast_pairs_stay_and_slow_ones_stretch():
    f, factor = ob.frequencies(32, 10000.0, dict(factor=8.0, original=4096, fast=32.0, slow=1.0))
    plain, one = ob.frequencies(32, 10000.0)
    assert f[0] == plain[0] and math.isclose(f[-1], plain[-1] / 8) and one == 1.0 and math.isclose(factor, 0.1 * math.log(8) + 1)
    assert all(p / 8 <= x <= p for x, p in zip(f, plain)) and any(p / 8 < x < p for x, p in zip(f, plain))


def test_oracle_rotation_depends_on_distance_alone():
    g = torch.Generator().manual_seed(0)
    q, k = torch.randn(1, 1, 12, generator=g, dtype=F64).expand(30, 1, 12), torch.randn(1, 1, 12, generator=g, dtype=F64).expand(30, 1, 12)
    r = dict(dims=8, base=100.0)
    a, b = ob.rotate_halves(q, r)[:, 0], ob.rotate_halves(k, r)[:, 0]
    assert torch.allclose(a[9] @ b[4], a[25] @ b[20]) and not torch.allclose(a[9] @ b[4], a[9] @ b[5])
    assert torch.equal(a[:, 8:], q[:, 0, 8:]) and torch.allclose(a.norm(dim=-1), q[:, 0].norm(dim=-1))


def test_oracle_attention_window_cap_and_sink():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(12, h, 4, generator=g, dtype=F64) for h in (4, 2, 2))
    a = ob.attend(q, k, v, 1.0, window=5, cap=2.0)
    for at, moved in ((7, True), (6, False)):                   # position 11 sees 7 .. 11
        k2 = k.clone()
        k2[at] += 3
        assert (float((a[11] - ob.attend(q, k2, v, 1.0, window=5, cap=2.0)[11]).abs().max()) > 1e-3) == moved
    s = 2.0 * torch.tanh(k[7:, 1] @ q[11, 3] / 2.0)
    assert torch.allclose(a[11, 3], torch.softmax(s, 0) @ v[7:, 1])
    sink = torch.tensor([0.5, -1.0, 2.0, 60.0], dtype=F64)
    b = ob.attend(q, k, v, 1.0, sink=sink)
    z = torch.exp(k[:, 0] @ q[11, 1])
    assert torch.allclose(b[11, 1], (z / (z.sum() + math.exp(-1.0))) @ v[:, 0]) and float(b[:, 3].abs().max()) < 1e-12


def test_oracle_activations_and_router():
    assert torch.allclose(ob.gelu_tanh(torch.tensor([0.5, -2.0, 30.0], dtype=F64)), torch.nn.functional.gelu(torch.tensor([0.5, -2.0, 30.0], dtype=F64), approximate="tanh"))
    y = ob.clamped_swiglu(torch.tensor([3.0, -4.0], dtype=F64), torch.tensor([9.0, -9.0], dtype=F64), 2.0)
    assert torch.allclose(y, torch.tensor([2 / (1 + math.exp(-3.404)) * 3, -4 / (1 + math.exp(6.808)) * -1], dtype=F64))
    # groups {0 1} {2 3} {4 5}: corrected scores decide groups and experts, plain scores the weights; the best single score sits in a group that loses
    z = torch.tensor([[2.0, -8.0, 0.5, 0.4, -1.0, -1.0]], dtype=F64)
    c = torch.tensor([0.0, 0.0, 0.0, 0.1, -0.6, -3.0], dtype=F64)
    got = ob.route(z, torch.eye(6, dtype=F64), c, dict(top=2, scale=3.0, groups=dict(count=3, keep=1)))[0]
    s = ob.sigmoid(z[0])
    assert [e for e, _ in got] == [3, 2] and math.isclose(float(got[0][1]), 3 * float(s[3])) and math.isclose(float(got[1][1]), 3 * float(s[2]))
    # an expert with a negative choice score still beats one of a closed group
    got = ob.route(z, torch.eye(6, dtype=F64), c - 2.0, dict(top=3, scale=1.0, groups=dict(count=3, keep=2)))[0]
    assert [e for e, _ in got] == [0, 3, 2]


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_oracle_is_causal_and_the_token_in_front_matters(name):
    cfg = CASES[name]
    w = ob.random_weights(cfg, 3)
    g = torch.Generator().manual_seed(0)
    ids = torch.randint(0, cfg["vocab"], (30,), generator=g).tolist()
    full, tr = ob.forward(cfg, w, ids)
    part, _ = ob.forward(cfg, w, ids[:17])
    assert torch.allclose(full[:17], part, atol=1e-9) and len(tr) == len(cfg["layers"])
    changed = list(ids)
    changed[3] = (changed[3] + 1) % cfg["vocab"]
    other, _ = ob.forward(cfg, w, changed)
    assert torch.equal(other[:3], full[:3]) and float((other[3:] - full[3:]).abs().max()) > 1e-3
    # one layer whose sublayers write nothing: the stream is the two embeddings
    flat = config([capped()])
    w = ob.random_weights(flat, 1)
    w["l0.norm1"] = torch.zeros_like(w["l0.norm1"])
    _, tr = ob.forward(flat, w, [3, 5, 5])
    rows = ob.bigram_rows([3, 5, 5], 29, 7, 53)
    assert torch.equal(tr[0], w["embed"][[3, 5, 5]].double() + w["bigram"][rows].double())


@pytest.mark.parametrize("name", sorted(CASES))
def test_routers_of_the_test_models_have_clear_choices(name):
    cfg = CASES[name]
    ob.margins.clear()
    ob.forward(cfg, ob.random_weights(cfg, 7), [(i * 31 + 7) % cfg["vocab"] for i in range(60)])
    assert not ob.margins or min(ob.margins) > 2e-3
