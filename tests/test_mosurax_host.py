"""Mosurax without a GPU: configuration and registry, weight loading and padding, run order, cache bookkeeping, prefill blocks, the
small library's build list, and the plain oracle against closed forms and itself."""
import json
import math
from pathlib import Path

import pytest
import torch
from safetensors.torch import save_file

from mosurax_cases import CASES, attention, config, dense, moe
from oracle import hybrid as oh
from oracle import mosurax as om
from sglang_amd import build, kernels
from sglang_amd.harness import registry
from sglang_amd.harness.genusun import GenusunConfig
from sglang_amd.harness.layered import LayeredConfig
from sglang_amd.harness.mosurax import MosuraxConfig, MosuraxForCausalLM
from sglang_amd.harness.weights import SyntheticWeights, TensorWeights
from sglang_amd.layers.mixers import padded_heads
from sglang_amd.mem_cache.memory_pool import GroupedTokenToKVPool

CPU = torch.device("cpu")
F64 = torch.float64


@pytest.fixture(autouse=True)
def no_library_calls(monkeypatch):
    """Modules ask the library which forms exist for their sizes when they are built."""
    monkeypatch.setattr(kernels, "grouped_attention_matrix_form", lambda *a: True)
    monkeypatch.setattr(kernels, "grouped_prefill_supported", lambda *a: True)


@pytest.mark.parametrize("name", sorted(CASES))
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_registry_reads_a_model_folder(tmp_path, name, dtype):
    cfg, w = CASES[name], om.random_weights(CASES[name], 1)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file(w, str(tmp_path / "model.safetensors"))
    c = registry.load_config(tmp_path)
    assert isinstance(c, MosuraxConfig) and registry.model_class(c) is MosuraxForCausalLM and registry.unit_group(c) == "grouped"
    assert c.runs() == oh.run_order(cfg) and c.num_hidden_layers == len(c.runs()) and c.logit_softcap == cfg["logit_softcap"]
    m = MosuraxForCausalLM(c, CPU, weights=TensorWeights.from_dir(tmp_path, CPU, dtype), dtype=dtype, max_context_len=64)
    # every pass of a looped layer has its own cache, the weights are the same objects
    assert [r for _, r, _ in m.runs] == list(range(len(c.runs()))) and [layer for layer, _, _ in m.runs] == [m.layers[i] for i, _ in c.runs()]
    pool = m.create_kv_pool(128, 64, "auto", CPU, False)
    assert isinstance(pool, GroupedTokenToKVPool) and len(pool.kv_rows) == len(c.runs()) and pool.dtype == dtype
    for (i, _), rows in zip(c.runs(), pool.kv_rows):
        mx = cfg["layers"][i]["mixer"]
        up = lambda n: (n + 7) // 8 * 8
        assert rows.shape == (192, mx["kv_heads"] * (up(mx["dim"]) + up(mx["vdim"]))) and float(rows.abs().sum()) == 0
    # no request can be longer than the table of positions
    assert m.create_req_to_token_pool(4, 4096, CPU).req_to_token.shape == (5, cfg["max_positions"])


def test_a_folder_that_does_not_fit_is_refused():
    cfg, w = CASES["mixed"], om.random_weights(CASES["mixed"], 2)
    c = MosuraxConfig.from_dict(cfg)
    for gone in ("pos", "loop.step", "l1.mlp.router.b", "l1.mlp.e11.down", "l1.mlp.shared.up", "l2.mix.g"):
        with pytest.raises(KeyError, match=gone):
            MosuraxForCausalLM(c, CPU, weights=TensorWeights({k: v for k, v in w.items() if k != gone}, CPU))
    with pytest.raises(ValueError, match="pos"):
        MosuraxForCausalLM(c, CPU, weights=TensorWeights({**w, "pos": torch.ones(3, 160)}, CPU))
    with pytest.raises(ValueError, match="l0.mix.q.b"):
        MosuraxForCausalLM(c, CPU, weights=TensorWeights({**w, "l0.mix.q.b": torch.ones(3)}, CPU))
    with pytest.raises(ValueError, match="unknown mixer"):
        MosuraxConfig.from_dict(config([dict(attention(), type="delta")]))
    with pytest.raises(ValueError, match="unknown feed-forward"):
        MosuraxConfig.from_dict(config([attention(mlp=dict(kind="sparse"))]))
    with pytest.raises(ValueError, match="unknown feed-forward"):
        GenusunConfig.from_dict(dict(vocab=8, width=8, norm=dict(eps=1e-5), embedding=dict(scale=1.0),
                                     layers=[dict(type="mamba2", mixer={}, mlp=moe(2, 1, 8))]))
    with pytest.raises(ValueError, match="loop"):
        MosuraxConfig.from_dict(config([attention()], loop=(0, 2, 1)))
    for bad in (attention(heads=5, kv_heads=2), attention(mlp=moe(4, 5, 8)), attention(mlp=moe(300, 2, 8))):
        with pytest.raises(ValueError):
            MosuraxForCausalLM(MosuraxConfig.from_dict(config([bad])), CPU, weights=SyntheticWeights(CPU))
    with pytest.raises(NotImplementedError):
        MosuraxForCausalLM(c, CPU, tp_size=2)
    with pytest.raises(NotImplementedError):
        MosuraxForCausalLM(c, CPU, weights=TensorWeights(w, CPU)).create_kv_pool(128, 64, "fp8_e4m3", CPU, False)


def test_named_models_and_synthetic_weights():
    assert isinstance(registry.named_config("mosurax-1b"), MosuraxConfig) and "mosurax-8b" in registry.config_names()
    m = MosuraxForCausalLM(MosuraxConfig.from_dict(CASES["odd"]), CPU)
    assert float(m.layers[0].norm1.min()) == 1.0 and float(m.layers[0].mlp.router_bias.abs().sum()) == 0.0


def test_heads_are_padded_with_zeros():
    w = torch.arange(1, 25, dtype=torch.float32).view(6, 4)
    p = padded_heads(w, 2, 3, 8, 0)
    assert p.shape == (16, 4) and torch.equal(p[:3], w[:3]) and torch.equal(p[8:11], w[3:]) and float(p.sum()) == float(w.sum())
    p = padded_heads(w, 2, 2, 8, 1)
    assert p.shape == (6, 16) and torch.equal(p[:, 8:10], w[:, 2:]) and float(p.sum()) == float(w.sum())
    assert padded_heads(w, 2, 3, 3, 0) is w


def test_runs_of_every_loop_placement():
    lay = [attention()] * 3

    def runs(loop):
        return LayeredConfig("x", 8, 8, lay, 1e-5, None if loop is None else dict(zip(("start", "stop", "times"), loop))).runs()

    assert runs(None) == [(0, None), (1, None), (2, None)]
    assert runs((0, 2, 2)) == [(0, 0), (1, None), (0, 1), (1, None), (2, None)]
    assert runs((2, 3, 3)) == [(0, None), (1, None), (2, 0), (2, 1), (2, 2)]
    assert runs((0, 3, 1)) == [(0, 0), (1, None), (2, None)]


def test_prefill_blocks_cover_every_token_once():
    for group, lens in ((1, [600, 2]), (3, [85, 86, 1]), (16, [40, 16])):
        q = kernels.QueryBlocks([0] * len(lens), lens, 32, group, CPU, rows=256)
        per = 256 // group
        got = sorted((b, f + i) for b, f in q.blocks.tolist() for i in range(min(per, lens[b] - f)))
        assert got == [(b, i) for b, n in enumerate(lens) for i in range(n)]
    # the block with the most visible keys comes first
    assert kernels.QueryBlocks([0, 1000], [300, 5], 0, 1, CPU, rows=256).blocks.tolist() == [[1, 0], [0, 256], [0, 0]]
    assert kernels.QueryBlocks([0], [], 0, 1, CPU, rows=256).blocks.shape == (0, 2)


def test_unit_group_lists_existing_sources_and_not_the_rest():
    assert all(p.exists() for p in build.sources("grouped")) and len(build.sources("grouped")) < len(build.sources())
    assert len({build.lib_path(g) for g in ("all", "hybrid", "grouped")}) == 3


# ---------------------------------------------------------------------------------------------- the oracle
def test_oracle_softmax_with_a_sink():
    g = torch.Generator().manual_seed(0)
    s = torch.randn(5, 7, generator=g, dtype=F64) * 4
    assert torch.allclose(om.sink_softmax(s), torch.softmax(torch.cat([torch.zeros(5, 1, dtype=F64), s], 1), -1)[:, 1:])
    assert torch.equal(om.sink_softmax(torch.full((1, 3), -1e4, dtype=F64)), torch.zeros(1, 3, dtype=F64))
    assert torch.allclose(om.sink_softmax(torch.full((1, 4), 1e4, dtype=F64)), torch.full((1, 4), 0.25, dtype=F64))


def test_oracle_window_edges_and_groups():
    g = torch.Generator().manual_seed(1)
    q, k, v = (torch.randn(12, h, 4, generator=g, dtype=F64) for h in (4, 2, 2))
    a = om.windowed_attention(q, k, v, 5, 1.0)
    for at, moved in ((7, True), (6, False)):                   # position 11 sees 7 .. 11
        k2 = k.clone()
        k2[at] += 3
        b = om.windowed_attention(q, k2, v, 5, 1.0)
        assert (float((a[11] - b[11]).abs().max()) > 1e-3) == moved
    k2 = k.clone()
    k2[11, 1] += 3                                              # key head 1 belongs to query heads 2 and 3
    d = (om.windowed_attention(q, k2, v, 5, 1.0) - a)[11].abs().amax(-1)
    assert float(d[:2].max()) == 0 and float(d[2:].min()) > 1e-3


def test_oracle_router_and_experts():
    h = torch.eye(3, dtype=F64)
    w = torch.tensor([[1.0, 0, 0], [0, 5, 0], [3, 0, 0], [0, 0, 2]], dtype=F64)
    p, e = om.route(h, w, torch.tensor([0.0, 0, 0, 0.5], dtype=F64), 2)
    assert e.tolist() == [[2, 0], [1, 3], [3, 0]]
    assert torch.allclose(p[0], torch.softmax(torch.tensor([3.0, 1.0], dtype=F64), 0)) and math.isclose(float(p[2, 0]), 1 / (1 + math.exp(-2.5)))
    assert om.soft_cap(torch.tensor([0.0, 1e9]), 7.0).tolist() == [0.0, 7.0]
    f = moe(3, 2, 4, 5)
    cfg = config([attention(mlp=f)], width=16)
    sub = {k: v.double() for k, v in oh._sub(om.random_weights(cfg, 3), "l0.mlp.").items()}
    x = torch.randn(4, 16, dtype=F64)
    p, e = om.route(x, sub["router"], sub["router.b"], 2)
    full = torch.stack([om.gated_mlp(x, sub[f"e{i}.gate"], sub[f"e{i}.up"], sub[f"e{i}.down"]) for i in range(3)], 1)
    want = (full.gather(1, e[:, :, None].expand(-1, -1, 16)) * p[:, :, None]).sum(1) + om.gated_mlp(x, sub["shared.gate"], sub["shared.up"], sub["shared.down"])
    assert torch.allclose(om.moe_mlp(x, sub, f), want)


@pytest.mark.parametrize("name", ["mixed", "odd"])
def test_oracle_is_causal_and_positions_matter(name):
    cfg = CASES[name]
    w = om.random_weights(cfg, 3)
    g = torch.Generator().manual_seed(0)
    ids = torch.randint(0, cfg["vocab"], (30,), generator=g).tolist()
    full, tr = om.forward(cfg, w, ids)
    part, _ = om.forward(cfg, w, ids[:17])
    assert torch.allclose(full[:17], part, atol=1e-9) and len(tr) == len(oh.run_order(cfg))
    changed = list(ids)
    changed[3] = (changed[3] + 1) % cfg["vocab"]
    other, _ = om.forward(cfg, w, changed)
    assert torch.equal(other[:3], full[:3]) and float((other[3:] - full[3:]).abs().max()) > 1e-3
    same, _ = om.forward(cfg, w, [ids[0]] * 2)
    assert float((same[0] - same[1]).abs().max()) > 1e-3


def test_oracle_loop_adds_the_embedding_output_and_a_step_per_pass():
    """A looped layer whose sublayers write nothing leaves x0 + step[0], then 2 x0 + step[0] + step[1]."""
    cfg = config([attention()], loop=(0, 1, 2))
    w = om.random_weights(cfg, 1)
    w["l0.mix.o"] = torch.zeros_like(w["l0.mix.o"])
    _, tr = om.forward(cfg, w, [3, 5])
    x0 = w["embed"][[3, 5]].double() + w["pos"][:2].double()
    s = w["loop.step"].double()
    assert torch.allclose(tr[0], x0 + s[0]) and torch.allclose(tr[1], 2 * x0 + s[0] + s[1])


@pytest.mark.parametrize("name", sorted(CASES))
def test_routers_of_the_test_models_have_clear_choices(name):
    cfg = CASES[name]
    om.margins.clear()
    om.forward(cfg, om.random_weights(cfg, 7), [(i * 31 + 7) % cfg["vocab"] for i in range(60)])
    assert not om.margins or min(om.margins) > 0.05
