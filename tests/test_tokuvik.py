"""Tokuvik without a GPU: its configuration, plan, checkpoint names and caches, and the plain implementation held against
itself (what chunks, sinks, gates per head, layer norms, state spaces and the tokens' own inputs do)."""

import copy
import math

import pytest
import torch

from tests import plain_tokuvik as plain
from tests.tokuvik_cases import CASES, random_weights

F = torch.float64


def parts_of(raw):
    from atomserve_amd.config.registry import architecture_for
    from atomserve_amd.models.decoder import DecoderModel

    arch = architecture_for(raw)
    config = arch.parse_config(raw)
    return arch, config, DecoderModel(arch.build_plan(config), torch.float32, "cpu")


@pytest.mark.parametrize("case", sorted(CASES))
def test_configuration_plan_and_names(case):
    raw = CASES[case]
    arch, config, model = parts_of(raw)
    assert arch.name == "Tokuvik" and arch.parse_config(config.to_dict()) == config
    plan = model.plan
    assert [r.layer for r in plan.run] == list(range(len(raw["layers"])))
    assert [(r.cache, r.writes) for r in plan.run] == [(layer["mixer"].get("kv_from"), layer["mixer"].get("kv_from") is None)
                                                       for layer in raw["layers"]]  # fmt: skip
    assert plan.tied_head and plan.final_norm.kind == "layernorm" and plan.embed_norm is None
    assert all(block.arrangement == "sandwich" and (block.token_input is not None) == ("token_side" in raw) for block in plan.layers)
    weights = random_weights(raw, seed=1)
    shapes = arch.checkpoint_shapes(config)
    assert set(shapes) == set(weights) and all(tuple(weights[k].shape) == tuple(v[0]) for k, v in shapes.items())
    from atomserve_amd.weights.loader import as_stack

    takes = [t for target in model.weight_decls() for t in as_stack(arch.checkpoint_map(config)[target]).parts]
    used = [(t.name, t.cols) for t in takes]
    assert len(used) == len(set(used)) and {t.name for t in takes} == set(weights), "every tensor is read, and nothing twice"
    assert model.capturable


def test_tables_of_token_inputs_are_columns_of_the_stored_one(tmp_path):
    """Each layer's table holds its own columns, from memory and from a file (of which only those columns are read)."""
    from safetensors.torch import save_file

    from atomserve_amd.weights.loader import DictSource, WeightsError, bind_checkpoint, load_weights

    raw = CASES["odd_sizes"]
    arch, config, model = parts_of(raw)
    weights = random_weights(raw, seed=2)
    save_file({k: v.bfloat16().contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    for tensors in (bind_checkpoint(model, arch, config, DictSource(weights)), load_weights(str(tmp_path), parts_of(raw)[2], arch, config)):
        for i in range(len(raw["layers"])):
            assert torch.equal(tensors[f"layers.{i}.token_input.table"], weights["side.embed"][:, 9 * i : 9 * i + 9])
    with pytest.raises(WeightsError, match="side.embed"):
        bind_checkpoint(model, arch, config, DictSource(dict(weights, **{"side.embed": weights["side.embed"][:, :-1]})))


def test_what_the_layers_keep():
    from atomserve_amd.parts.base import PagedCacheRequest, StateCacheRequest

    _, _, model = parts_of(CASES["all_kinds"])
    requests = model.cache_requests()
    paged = {k: v for k, v in requests.items() if isinstance(v, PagedCacheRequest)}
    states = {k: v for k, v in requests.items() if isinstance(v, StateCacheRequest)}
    assert sorted(paged, key=str) == [(0, "0.pages"), 2]
    mine = paged[(0, "0.pages")]  # chunks of 13, 7 and 30
    assert (mine.num_kv_heads, mine.head_dim, mine.window, mine.keep_first) == (2, 32, 30, 0)
    assert (paged[2].num_kv_heads, paged[2].head_dim, paged[2].window) == (1, 64, 0)
    assert {k: v.shape for k, v in states.items()} == {(1, "state"): (6, 24, 16), (1, "conv"): (3, 96 + 2 * 3 * 24)}
    cores = [block.mixer.cores[0] for block in model.plan.layers if block.mixer.kind == "joined"]
    assert [(c.chunk, c.window, c.own_kv) for c in cores] == [(13, 0, True), (7, 0, False), (30, 0, False)]
    # a reader without chunks keeps everything; a convolution of one tap keeps no inputs
    _, _, model = parts_of(CASES["odd_sizes"])
    requests = model.cache_requests()
    assert requests[(1, "0.pages")].window == 0 and (3, "conv") not in requests and requests[(0, "conv")].shape == (2, 31)


def test_pages_behind_a_chunk_are_given_back_and_those_of_the_chunk_are_not():
    from atomserve_amd.cache.manager import CacheManager

    _, _, model = parts_of(CASES["all_kinds"])
    manager = CacheManager(model.cache_requests(), 4, 60, 2)
    assert not manager.prefix_reuse_possible
    group = next(g for g, p in enumerate(manager.paged_groups) if p.request.window == 30)
    rc = manager.new_request()
    assert manager.reserve(rc, 0, 100)
    for computed in range(1, 101):
        manager.release_behind_window(rc, computed)
        first = computed // 30 * 30  # the oldest key that the next query sees in the longest chunk
        assert all(p >= 0 for p in rc.tables[group][first // 4 :]), computed
    assert sum(p >= 0 for p in rc.tables[group]) <= (30 + 4) // 4 + 1
    manager.release(rc)


def test_what_the_configuration_refuses():
    from atomserve_amd.config.model_config import ConfigError, TokuvikConfig

    raw = CASES["all_kinds"]
    for change, needle in (
        (lambda r: r["layers"][0].update(type="delta"), "type"),
        (lambda r: r["layers"][0]["mlp"].update(kind="moe"), "kind"),
        (lambda r: r["layers"][0]["mlp"].update(ff=0), "ff"),
        (lambda r: r["layers"][0]["mixer"].pop("scale"), "scale"),
        (lambda r: r["layers"][0]["mixer"].update(heads=3), "kv_heads"),
        (lambda r: r["layers"][0]["mixer"]["mask"].update(size=-2), "mask"),
        (lambda r: r["layers"][1]["mixer"].pop("state"), "state"),
        (lambda r: r["layers"][1]["mixer"].update(groups=4), "groups"),
        (lambda r: r["layers"][1]["mixer"].update(norm_groups=5), "norm_groups"),
        (lambda r: r["layers"][2]["mixer"].update(q_rank=0), "positive"),
        (lambda r: r["layers"][3]["mixer"].update(kv_from=3), "kv_from"),
        (lambda r: r["layers"][3]["mixer"].update(kv_from=2), "kv_from"),
        (lambda r: r["layers"][4]["mixer"].update(kv_from=3), "kv_from"),
        (lambda r: r["layers"][3]["mixer"].update(vdim=16), "kv_from"),
        (lambda r: r["norm"].pop("eps"), "eps"),
        (lambda r: r["norm"].update(eps=0.0), "eps"),
        (lambda r: r["token_side"].pop("dim"), "dim"),
    ):
        broken = copy.deepcopy(raw)
        change(broken)
        with pytest.raises(ConfigError, match=needle):
            TokuvikConfig.from_dict(broken)


def test_parts_refuse_what_they_do_not_compute():
    from atomserve_amd.parts.base import BuildEnv, build
    from atomserve_amd.parts.plan import (
        BlockSpec, GatedMLPSpec, JoinedMixerSpec, NormSpec, ShortConvSpec, SoftmaxCoreSpec, StateSpaceSpec, TokenInputSpec,
    )  # fmt: skip

    env = BuildEnv(torch.float32, torch.device("cpu"))
    for bad, needle in (
        (JoinedMixerSpec("joined", 64, (SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25, out_gate=True, head_gate=True),), (1.0,)), "not both"),
        (JoinedMixerSpec("joined", 64, (SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25, window=3, chunk=4),), (1.0,)), "not both"),
        (StateSpaceSpec("state_space", 64, 3, 8, 8, 2, ShortConvSpec(4), 1, 1e-5), "groups of B"),
        (StateSpaceSpec("state_space", 64, 4, 8, 8, 2, ShortConvSpec(4), 3, 1e-5), "norm"),
        (StateSpaceSpec("state_space", 64, 4, 8, 8, 2, ShortConvSpec(40), 1, 1e-5), "taps"),
        (StateSpaceSpec("state_space", 64, 4, 8, 4096, 2, ShortConvSpec(4), 1, 1e-5), "exceeds"),
    ):  # fmt: skip
        with pytest.raises(ValueError, match=needle):
            build("mixer", bad, env)
    core = SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25)
    norm, grouped = NormSpec("layernorm", 64, 1e-5), NormSpec("grouped_rmsnorm", 64, 1e-5, 2)
    with pytest.raises(ValueError, match="grouped_rmsnorm"):
        build("arrangement", BlockSpec("sandwich", JoinedMixerSpec("joined", 64, (core,), (1.0,)), norm, GatedMLPSpec("gated_mlp", 64, 32, "silu"),
                                       norm, mixer_post_norm=norm, ffn_post_norm=norm,
                                       token_input=TokenInputSpec("gated_table", 64, 8, 100, grouped)), env)  # fmt: skip


# ---- the plain implementation against itself ----------------------------------------------------------------------


def test_which_keys_a_position_sees():
    seen = plain.visible(12, 5)
    assert [row.nonzero().flatten().tolist() for row in seen[[0, 4, 5, 9, 10]]] == [[0], [0, 1, 2, 3, 4], [5], [5, 6, 7, 8, 9], [10]]
    assert torch.equal(plain.visible(9, 1), torch.eye(9, dtype=torch.bool))
    assert torch.equal(plain.visible(9), torch.ones(9, 9, dtype=torch.bool).tril())
    assert torch.equal(plain.visible(9, 40), plain.visible(9))


def test_a_sink_takes_a_share_and_is_not_scaled():
    s = torch.tensor([[-3.0, 2.0], [-50.0, -50.0]], dtype=F)
    w = plain.softmax_weights(s, torch.tensor(1.5, dtype=F))
    assert torch.allclose(w[0], torch.exp(s[0]) / (math.exp(1.5) + torch.exp(s[0]).sum())) and float(w[1].sum()) < 1e-20
    assert torch.allclose(plain.softmax_weights(s).sum(-1), torch.ones(2, dtype=F))
    q, k, v = (torch.randn(4, 2, n, dtype=F) for n in (3, 3, 5))
    sinks = torch.tensor([0.7, -40.0], dtype=F)
    o, bare = plain.attention(q, k, v, 0.5, sinks=sinks), plain.attention(q, k, v, 0.5)
    assert torch.allclose(o[:, 1], bare[:, 1]) and not torch.allclose(o[:, 0], bare[:, 0], atol=1e-3)
    first = torch.exp(0.5 * (q[0, 0] * k[0, 0]).sum())
    assert torch.allclose(o[0, 0], v[0, 0] * first / (first + math.exp(0.7)))


def test_norms():
    x = torch.randn(3, 12, dtype=F) * 4 + 7
    w = torch.rand(12, dtype=F) + 0.5
    assert torch.allclose(plain.layer_norm(x, w, 1e-5), torch.nn.functional.layer_norm(x, (12,), w, None, 1e-5))
    assert torch.allclose(plain.rms_norm(x, w, 1e-5), torch.nn.functional.rms_norm(x, (12,), w, 1e-5))
    parts = torch.cat([plain.rms_norm(p, torch.ones(4, dtype=F), 1e-5) for p in x.split(4, dim=1)], dim=1)
    assert torch.allclose(plain.grouped_rms_norm(x, w, 1e-5, 3), parts * w)
    assert torch.allclose(plain.grouped_rms_norm(x, w, 1e-5, 1), plain.rms_norm(x, w, 1e-5))


def test_a_gate_per_head_and_gelu():
    heads, g = torch.randn(2, 3, 4, dtype=F), torch.randn(2, 3, dtype=F)
    assert torch.allclose(plain.head_gates(g, heads)[1, 2], heads[1, 2] / (1 + math.exp(-float(g[1, 2]))))
    z = torch.linspace(-5, 5, 21, dtype=F)
    assert torch.allclose(plain.gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    z = torch.tensor([-800.0, 0.0, 800.0], dtype=F)
    assert plain.softplus(z).tolist() == [0.0, math.log(2.0), 800.0]


def test_the_convolution_sees_the_last_taps_only():
    gen = torch.Generator().manual_seed(3)
    x, w, b = torch.randn(7, 3, generator=gen, dtype=F), torch.randn(3, 4, generator=gen, dtype=F), torch.randn(3, generator=gen, dtype=F)
    y = plain.causal_conv(x, w, b)
    assert torch.allclose(y[0], w[:, 3] * x[0] + b) and torch.allclose(y[5], (w * x[2:6].t()).sum(1) + b)
    assert torch.allclose(plain.causal_conv(x, w[:, :1], b), x * w[:, 0] + b)


def test_a_state_space_is_a_sum_over_the_past():
    """y_t = sum_j (C_t . B_j) exp(-rate (dt_(j+1) + .. + dt_t)) dt_j x_j + D x_t, each head with its group's B and C."""
    gen = torch.Generator().manual_seed(1)
    T, H, G, N, E = 6, 4, 2, 3, 5
    x, B, C = (torch.randn(T, n, m, generator=gen, dtype=F) for n, m in ((H, E), (G, N), (G, N)))
    dt, rate, D = torch.rand(T, H, generator=gen, dtype=F), torch.randn(H, generator=gen, dtype=F), torch.randn(H, generator=gen, dtype=F)
    got = plain.state_space_scan(x, B, C, dt, rate, D)
    for t in range(T):
        for h in range(H):
            want = D[h] * x[t, h]
            for j in range(t + 1):
                decay = torch.exp(-torch.exp(rate[h]) * dt[j + 1 : t + 1, h].sum())
                want = want + (C[t, h // 2] * B[j, h // 2]).sum() * decay * dt[j, h] * x[j, h]
            assert torch.allclose(got[t, h], want)


def test_token_inputs_depend_on_the_stream_and_the_token():
    gen = torch.Generator().manual_seed(2)
    W = {"l0.side.gate": torch.randn(3, 6, generator=gen, dtype=F), "l0.side.proj": torch.randn(6, 3, generator=gen, dtype=F),
         "l0.side.norm": torch.ones(6, dtype=F)}  # fmt: skip
    x, e = torch.randn(2, 6, generator=gen, dtype=F), torch.randn(2, 3, generator=gen, dtype=F)
    y = plain.token_input(x, W, "l0.", e, 1e-9, False)
    assert torch.allclose((y * y).mean(-1), torch.ones(2, dtype=F), atol=1e-6)
    z = torch.nn.functional.gelu(x @ W["l0.side.gate"].t(), approximate="tanh") * e
    assert torch.allclose(y, plain.rms_norm(z @ W["l0.side.proj"].t(), W["l0.side.norm"], 1e-9))
    assert not torch.allclose(plain.token_input(x, W, "l0.", e.flip(0), 1e-9, False), y, atol=0.1)


@pytest.mark.parametrize("case", sorted(CASES))
def test_later_tokens_change_nothing_before_them(case):
    raw = CASES[case]
    weights = random_weights(raw, seed=3)
    ids = torch.randint(0, raw["vocab"], (40,), generator=torch.Generator().manual_seed(4)).tolist()
    full, part = plain.logits(raw, weights, ids), plain.logits(raw, weights, ids[:23])
    assert torch.allclose(full[:23], part, atol=1e-6) and float(full.std()) > 0.05


def test_a_reader_uses_the_other_layers_keys_and_its_own_chunks():
    raw = copy.deepcopy(CASES["all_kinds"])
    weights = random_weights(raw, seed=5)
    ids = list(range(3, 53))
    want = plain.logits(raw, weights, ids)
    for change in (lambda r: r["layers"][4]["mixer"]["mask"].update(size=29), lambda r: r["layers"][3]["mixer"]["mask"].update(size=8)):
        other = copy.deepcopy(raw)
        change(other)
        assert float((plain.logits(other, weights, ids) - want).abs().max()) > 1e-4
    outs = []
    two = dict(raw, layers=raw["layers"][:1] + raw["layers"][3:4], token_side=None)
    two["layers"][1] = dict(two["layers"][1], mlp=None)
    plain.forward(two, {k.replace("l3.", "l1."): v for k, v in dict(weights, **{"l0.mix.v": weights["l0.mix.v"] * 1.5}).items()}, ids, layers_out=outs)
    assert len(outs) == 2 and float((outs[1] - outs[0]).abs().max()) > 0.1
