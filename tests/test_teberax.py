"""Teberax without a GPU: its configuration, plan, checkpoint names and caches, and the plain implementation held
against itself (what the masks, the sink, the cap, the two maps, the decays per channel, the polynomial of normed powers
and the corrected router do)."""

import copy
import math

import pytest
import torch

from tests import plain_teberax as plain
from tests.teberax_cases import CASES, random_weights

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
    assert arch.name == "Teberax" and arch.parse_config(config.to_dict()) == config
    plan = model.plan
    assert [r.layer for r in plan.run] == list(range(len(raw["layers"])))
    assert [(r.cache, r.writes) for r in plan.run] == [(layer["mixer"].get("kv_from"), layer["mixer"].get("kv_from") is None)
                                                       for layer in raw["layers"]]  # fmt: skip
    assert not plan.tied_head and plan.logit_softcap == raw.get("logit_softcap", 0.0)
    assert plan.final_norm.one_gain and plan.embed_norm.one_gain
    assert all(block.arrangement == "sandwich" for block in plan.layers)
    weights = random_weights(raw, seed=1)
    shapes = arch.checkpoint_shapes(config)
    assert set(shapes) == set(weights) and all(tuple(weights[k].shape) == tuple(v[0]) for k, v in shapes.items())
    from atomserve_amd.weights.loader import as_stack

    used = [t.name for target in model.weight_decls() for t in as_stack(arch.checkpoint_map(config)[target]).parts]
    assert len(used) == len(set(used)) and set(used) == set(weights), "every tensor of the checkpoint is read exactly once"
    assert model.capturable


def test_pages_keep_what_the_widest_of_their_readers_sees():
    from atomserve_amd.cache.manager import CacheManager
    from atomserve_amd.parts.base import PagedCacheRequest, StateCacheRequest

    _, _, model = parts_of(CASES["all_kinds"])
    requests = model.cache_requests()
    paged = {k: v for k, v in requests.items() if isinstance(v, PagedCacheRequest)}
    states = {k: v for k, v in requests.items() if isinstance(v, StateCacheRequest)}
    assert sorted(paged, key=str) == [(0, "0.pages"), (1, "0.pages"), 2]
    mine = paged[(0, "0.pages")]  # windows of 13, 7 and 30 that keep 3, 9 and 2 first tokens; two keys of 16 beside a value of 24
    assert (mine.num_kv_heads, mine.head_dim, mine.window, mine.keep_first) == (2, 32, 30, 9)
    assert (paged[(1, "0.pages")].window, paged[2].window, paged[2].keep_first) == (0, 17, 0)
    assert list(states) == [(1, "1.state")] and states[(1, "1.state")].shape == (3, 16, 8)
    cores = [block.mixer.cores[0] for block in model.plan.layers if block.mixer.kind == "joined"]
    assert [(c.window, c.keep_first, c.own_kv) for c in cores] == [(13, 3, True), (0, 0, True), (7, 9, False), (30, 2, False)]
    manager = CacheManager(requests, 4, 60, 2)
    assert not manager.prefix_reuse_possible
    rc = manager.new_request()
    assert manager.reserve(rc, 0, 50)
    manager.release_behind_window(rc, 50)
    group = next(g for g, p in enumerate(manager.paged_groups) if p.request == mine)
    assert [p >= 0 for p in rc.tables[group]] == [True] * 3 + [False] * 2 + [True] * 8  # 9 first tokens; the next sees 21 ..
    manager.release(rc)
    # a reader without a window keeps everything
    _, _, model = parts_of(CASES["odd_sizes"])
    assert model.cache_requests()[(1, "0.pages")].window == 0


def test_what_the_configuration_refuses_and_completes():
    from atomserve_amd.config.model_config import ConfigError, TeberaxConfig

    raw = CASES["all_kinds"]
    for change, needle in (
        (lambda r: r["layers"][0].update(type="delta"), "type"),
        (lambda r: r["layers"][0]["mlp"].update(kind="gated"), "kind"),
        (lambda r: r["layers"][0]["mixer"].pop("diff"), "diff"),
        (lambda r: r["layers"][0]["mixer"].update(heads=3), "kv_heads"),
        (lambda r: r["layers"][0]["mixer"]["mask"].update(keep_first=-1), "keep_first"),
        (lambda r: r["layers"][1]["mixer"]["left"]["rot"].update(dims=26), "rot"),
        (lambda r: r["layers"][1]["mixer"]["left"]["rot"]["scaling"].update(factor=0.0), "factor"),
        (lambda r: r["layers"][1]["mixer"]["right"].update(tau=0.0), "tau"),
        (lambda r: r["layers"][2]["mixer"]["rot"].update(dims=6), "rot_dim"),
        (lambda r: r["layers"][2]["mlp"]["router"].update(top=6), "top"),
        (lambda r: r["layers"][3]["mixer"].update(kv_from=3), "kv_from"),
        (lambda r: r["layers"][3]["mixer"].update(kv_from=2), "kv_from"),
        (lambda r: r["layers"][4]["mixer"].update(kv_from=3), "kv_from"),
        (lambda r: r["layers"][3]["mixer"].update(vdim=16), "kv_from"),
        (lambda r: r["norm"].pop("eps"), "eps"),
        (lambda r: r.update(logit_softcap=-1.0), "logit_softcap"),
    ):
        broken = copy.deepcopy(raw)
        change(broken)
        with pytest.raises(ConfigError, match=needle):
            TeberaxConfig.from_dict(broken)
    # the rank that config.json does not name comes from a tensor's shape; without either there is no plan
    bare = copy.deepcopy(raw)
    bare["layers"][1]["mixer"]["right"].pop("rank")
    arch, _, _ = parts_of(raw)
    config = arch.parse_config(bare)
    with pytest.raises(ConfigError, match="rank"):
        arch.build_plan(config)
    assert arch.complete(config, {"l1.mix.right.a1": (5, 96)}.get) == arch.parse_config(raw)


def test_parts_refuse_what_they_do_not_compute():
    from atomserve_amd.parts.base import BuildEnv, build
    from atomserve_amd.parts.plan import (
        BlockSpec, ChannelDecaySpec, GatedRoutedExpertsSpec, JoinedMixerSpec, NeighbourRotarySpec, NormSpec, PolyNormMLPSpec, SoftmaxCoreSpec,
    )  # fmt: skip

    env = BuildEnv(torch.float32, torch.device("cpu"))
    two = dict(maps=2, difference=0.3, difference_eps=1e-5)
    core = SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25)
    for bad, needle in (
        (JoinedMixerSpec("joined", 64, (SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25, maps=3),), (1.0,)), "maps|map"),
        (JoinedMixerSpec("joined", 64, (SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25, position=NeighbourRotarySpec("rope_neighbours", 8, 100.0), **two),), (1.0,)), "rotation"),
        (JoinedMixerSpec("joined", 64, (SoftmaxCoreSpec("softmax_core", 4, 2, 16, 16, 0.25, own_kv=False, value_mix="first"),), (1.0,)), "another layer"),
        (JoinedMixerSpec("joined", 64, (core,), (1.0,), out_norm_eps=1e-5), "two"),
        (JoinedMixerSpec("joined", 64, (core,), (1.0,), out_bias=(True,)), "biases"),
        (JoinedMixerSpec("joined", 64, (ChannelDecaySpec("channel_decay", 2, 8, 8, 0, 1.0, 1e-5),), (1.0,)), "first step"),
    ):  # fmt: skip
        with pytest.raises(ValueError, match=needle):
            build("mixer", bad, env)
    with pytest.raises(ValueError, match="corrected"):
        build("feed_forward", GatedRoutedExpertsSpec("gated_routed_experts", 64, 8, 4, 2, "silu", 0.0, score="softmax", groups=2,
                                                     keep_groups=1, correction=True), env)  # fmt: skip
    with pytest.raises(ValueError, match="cannot be chosen"):
        build("feed_forward", GatedRoutedExpertsSpec("gated_routed_experts", 64, 8, 2, 5, "silu", 0.0, score="softmax", identity=2), env)
    grouped = NormSpec("grouped_rmsnorm", 64, 1e-5, 2)
    with pytest.raises(ValueError, match="grouped_rmsnorm"):
        build("arrangement", BlockSpec("sandwich", JoinedMixerSpec("joined", 64, (core,), (1.0,)), grouped, PolyNormMLPSpec("poly_norm_mlp", 64, 32, 1e-5),
                                       grouped, mixer_post_norm=grouped, ffn_post_norm=grouped), env)  # fmt: skip


# ---- the plain implementation against itself ----------------------------------------------------------------------


def test_which_keys_a_position_sees():
    seen = plain.visible(12, {"size": 4, "keep_first": 2})
    assert seen[9].nonzero().flatten().tolist() == [0, 1, 6, 7, 8, 9] and seen[3].nonzero().flatten().tolist() == [0, 1, 2, 3]
    assert seen[5].nonzero().flatten().tolist() == [0, 1, 2, 3, 4, 5] and seen[6].nonzero().flatten().tolist() == [0, 1, 3, 4, 5, 6]
    assert torch.equal(plain.visible(9, {"size": 1}), torch.eye(9, dtype=torch.bool))
    assert torch.equal(plain.visible(9, None), torch.ones(9, 9, dtype=torch.bool).tril())
    assert torch.equal(plain.visible(9, {"size": 2, "keep_first": 9}), torch.ones(9, 9, dtype=torch.bool).tril())


def test_a_sink_takes_a_share_and_a_cap_bounds_scores():
    s = torch.tensor([[-3.0, 2.0], [-50.0, -50.0]], dtype=F)
    w = plain.softmax_weights(s, True)
    assert torch.allclose(w[0], torch.exp(s[0]) / (1 + torch.exp(s[0]).sum())) and float(w[1].sum()) < 1e-20
    assert torch.allclose(plain.softmax_weights(s, False).sum(-1), torch.ones(2, dtype=F))
    z = torch.tensor([1e-3, 1.0, 1e3, -1e3], dtype=F)
    assert torch.allclose(plain.softcap(z, 5.0), torch.tensor([1e-3, 5 * math.tanh(0.2), 5.0, -5.0], dtype=F), atol=1e-9)
    assert torch.equal(plain.softcap(z, 0.0), z)


def test_equal_maps_cancel_by_one_minus_lambda_and_the_norm_hides_it():
    """With both maps equal the difference is (1 - lambda) times the map: its norm is the map's own, times the sign."""
    a = torch.randn(5, 2, 8, dtype=F)
    same = plain.differential_combine(a, a, 0.25, 0.3, 1e-12)
    assert torch.allclose(same, plain.rms(a, 0.0) * 0.7, atol=1e-9)
    assert torch.allclose(plain.differential_combine(a, a, 1.75, 0.3, 1e-12), -same, atol=1e-9)
    w = {"x.lq1": torch.zeros(4), "x.lk1": torch.ones(4), "x.lq2": torch.tensor([1.0, 0, 0, 0]), "x.lk2": torch.tensor([0.5, 9, 9, 9])}
    assert abs(float(plain.differential_lambda(w, "x.", 0.2)) - (1.0 - math.exp(0.5) + 0.2)) < 1e-12


def test_the_rotation_is_a_function_of_the_distance_and_scaling_slows_it():
    gen = torch.Generator().manual_seed(0)
    q, k = torch.randn(1, 1, 12, generator=gen, dtype=F), torch.randn(1, 1, 12, generator=gen, dtype=F)

    def score(i, j, rot):
        return float((plain.rotate_neighbours(q, torch.tensor([i]), rot) * plain.rotate_neighbours(k, torch.tensor([j]), rot)).sum())

    rot = {"dims": 8, "base": 50.0}
    slow = {"dims": 8, "base": 50.0, "scaling": {"factor": 4.0}}
    assert abs(score(9, 4, rot) - score(25, 20, rot)) < 1e-9 and abs(score(9, 4, rot) - score(9, 5, rot)) > 1e-3
    assert abs(score(36, 16, slow) - score(9, 4, rot)) < 1e-9
    turned = plain.rotate_neighbours(q, torch.tensor([1]), {"dims": 2, "base": 7.0})
    assert torch.equal(turned[..., 2:], q[..., 2:])
    a = torch.tensor([math.cos(1.0), math.sin(1.0)], dtype=F)
    assert torch.allclose(turned[0, 0, :2], torch.stack([q[0, 0, 0] * a[0] - q[0, 0, 1] * a[1], q[0, 0, 1] * a[0] + q[0, 0, 0] * a[1]]))


def test_decays_per_channel_forget_channel_by_channel():
    gen = torch.Generator().manual_seed(1)
    T, H, D, E = 6, 2, 3, 4
    q, k, v = (torch.randn(T, H, n, generator=gen, dtype=F) for n in (D, D, E))
    alpha = torch.ones(T, H, D, dtype=F)
    want = torch.einsum("thd,jhd,jhe,tj->the", q, k, v, torch.ones(T, T, dtype=F).tril())
    assert torch.allclose(plain.channel_decay_scan(q, k, v, alpha), want)
    alpha[:, :, 1] = 0.0  # this channel remembers nothing but the token itself
    got = plain.channel_decay_scan(q, k, v, alpha)
    lost = torch.einsum("th,jh,jhe,tj->the", q[:, :, 1], k[:, :, 1], v, torch.ones(T, T, dtype=F).tril(-1))
    assert torch.allclose(got, want - lost)
    z = torch.tensor([0.0, 30.0, -4.0], dtype=F)
    assert torch.allclose(plain.channel_decays(z, 2.0), torch.sigmoid(z) ** 0.5)


def test_the_polynomial_of_normed_powers():
    z = torch.tensor([[1.0, -2.0, 3.0]], dtype=F)
    a = torch.tensor([2.0, 0.0, 0.0, 0.5], dtype=F)
    assert torch.allclose(plain.poly_norm(z, a, 0.0), 2 * z / math.sqrt(14 / 3) + 0.5)
    only = plain.poly_norm(z, torch.tensor([0.0, 1.0, 0.0, 0.0], dtype=F), 0.0)
    assert torch.allclose(only, z**2 / math.sqrt((1 + 16 + 81) / 3))
    cube = plain.poly_norm(z, torch.tensor([0.0, 0.0, 1.0, 0.0], dtype=F), 0.0)
    assert torch.allclose(cube, z**3 / math.sqrt((1 + 64 + 729) / 3))


def test_corrections_choose_and_do_not_weigh_and_identity_experts_return_the_input():
    gen = torch.Generator().manual_seed(2)
    h = torch.randn(4, 6, generator=gen, dtype=F)
    f = {"router": {"experts": 2, "top": 1, "identity": 1}, "expert": {"ff": 3}}
    W = {"x.router": torch.randn(3, 6, generator=gen, dtype=F), "x.correction": torch.tensor([-5.0, -5.0, 0.0], dtype=F)}
    for e in range(2):
        for name, shape in (("gate", (3, 6)), ("up", (3, 6)), ("down", (6, 3))):
            W[f"x.e{e}.{name}"] = torch.randn(*shape, generator=gen, dtype=F)
    s = torch.softmax(h @ W["x.router"].t(), dim=-1)
    assert torch.allclose(plain.experts(h, W, "x.", f, False), s[:, 2:] * h)
    W["x.correction"] = torch.tensor([0.0, 3.0, 0.0], dtype=F)
    y = torch.nn.functional.silu(h @ W["x.e1.gate"].t()) * (h @ W["x.e1.up"].t()) @ W["x.e1.down"].t()
    assert torch.allclose(plain.experts(h, W, "x.", f, False), s[:, 1:2] * y)
    assert plain.corrected_choice(torch.full((1, 4), 0.25), torch.zeros(4), 2).tolist() == [[0, 1]]


@pytest.mark.parametrize("case", sorted(CASES))
def test_later_tokens_change_nothing_before_them(case):
    raw = CASES[case]
    weights = random_weights(raw, seed=3)
    ids = torch.randint(0, raw["vocab"], (40,), generator=torch.Generator().manual_seed(4)).tolist()
    full, part = plain.logits(raw, weights, ids), plain.logits(raw, weights, ids[:23])
    assert torch.allclose(full[:23], part, atol=1e-6) and float(full.std()) > 0.05


def test_a_reader_uses_the_other_layers_keys_and_its_own_mask():
    raw = copy.deepcopy(CASES["all_kinds"])
    weights = random_weights(raw, seed=5)
    ids = list(range(3, 53))
    want = plain.logits(raw, weights, ids)
    for change in (lambda r: r["layers"][4]["mixer"]["mask"].update(size=29), lambda r: r["layers"][3]["mixer"]["mask"].update(keep_first=8)):
        other = copy.deepcopy(raw)
        change(other)
        assert float((plain.logits(other, weights, ids) - want).abs().max()) > 1e-4
    w2 = dict(weights)
    w2["l0.mix.v"] = weights["l0.mix.v"] * 1.5
    raw["layers"] = raw["layers"][:1] + [dict(raw["layers"][3], mlp=None)]
    outs = []
    plain.forward(raw, {k.replace("l3.", "l1."): v for k, v in w2.items()}, ids, layers_out=outs)
    assert len(outs) == 2 and float((outs[1] - outs[0]).abs().max()) > 0.1
