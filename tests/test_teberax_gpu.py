"""Teberax on the GPU against the plain implementation (tests/plain_teberax.py): each mechanism alone, and whole models
of several shapes stepped whole, token by token, in portions down to two tokens, in mixed batches with pages and state
slots used again, and through the engine's scheduler.  Configurations and weights are made here; where random weights
would hide a fault (a far key among hundreds, a window's edge, the first tokens, a sink, a decay near zero) the inputs
are made so that it shows."""

import json
import os

import pytest
import torch

from tests import plain_teberax as plain
from tests import replay_cases as rc
from tests.teberax_cases import CASES, random_weights

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
I32 = torch.int32


def build_model(raw, weights, dtype):
    from atomserve_amd.config.registry import architecture_for
    from atomserve_amd.models.decoder import DecoderModel
    from atomserve_amd.weights.loader import DictSource, bind_checkpoint

    arch = architecture_for(raw)
    config = arch.parse_config(raw)
    model = DecoderModel(arch.build_plan(config), DTYPES[dtype], DEV)
    bind_checkpoint(model, arch, config, DictSource(weights))
    return model


def make_replay(raw, weights, dtype, max_tokens, block_size=16, max_live=4):
    from atomserve_amd.engine.replay import Replay

    return Replay("", dtype, max_tokens, device=DEV, block_size=block_size, max_live=max_live, model=build_model(raw, weights, dtype))


class Against:
    """Engine - plain, row by row, beside what rounding to bfloat16 alone does to the plain model at the same rows."""

    def __init__(self):
        self.err, self.noise, self.scale = [], [], 1.0

    def add(self, got, exact, rounded=None):
        got, exact = got.reshape(-1, exact.shape[-1]), exact.reshape(-1, exact.shape[-1])
        self.err += (got - exact).pow(2).mean(-1).sqrt().tolist()
        if rounded is not None:
            self.noise += (rounded.reshape(exact.shape) - exact).pow(2).mean(-1).sqrt().tolist()
        self.scale = max(self.scale, float(exact.abs().max()))

    def take(self, other):
        self.err += other.err
        self.noise += other.noise
        self.scale = max(self.scale, other.scale)

    def check(self, dtype, what=""):
        """32-bit: rounding of float32 only, at every row.  bfloat16: the rows' errors as a distribution against what
        rounding the stored activations moves the plain model itself at the same rows (a token whose router scores lie
        within rounding of each other may take another expert in either model; such rows stand out in both)."""
        assert self.err
        err = torch.tensor(self.err)
        if dtype == "float32":
            assert float(err.max()) <= 3e-5 * self.scale, f"{what}: {float(err.max()):.3e} against |logits| {self.scale:.3e}"
            return
        noise = torch.tensor(self.noise)
        mid, high = (float(err.median()), float(noise.median())), (float(err.quantile(0.9)), float(noise.quantile(0.9)))
        assert mid[0] <= 1.5 * mid[1] and high[0] <= 2.0 * high[1], (
            f"{what}: row errors' median {mid[0]:.3e} and ninth decile {high[0]:.3e}; rounding alone moves the plain model "
            f"by {mid[1]:.3e} and {high[1]:.3e}; |logits| {self.scale:.3e}; {len(self.err)} rows")  # fmt: skip


def reference(raw, weights, ids, refs, key, dtype):
    if key not in refs:
        refs[key] = (plain.logits(raw, weights, ids), plain.logits(raw, weights, ids, rounded=True) if dtype == "bfloat16" else None)
    return refs[key]


def compare(replay, steps, requests, raw, weights, refs, dtype):
    at = {rid: 0 for rid in requests}
    result = Against()
    for s in steps:
        logits = replay.step(s["entries"], s["end"])
        k = 0
        for e in s["entries"]:
            rid = e["id"]
            exact, rounded = reference(raw, weights, requests[rid], refs, rid, dtype)
            for w in e["want"]:
                place = at[rid] + w
                result.add(logits[k], exact[place], None if rounded is None else rounded[place])
                k += 1
            at[rid] += len(e["tokens"])
    return result


# ---- whole models -------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", sorted(CASES))
def test_whole_decoded_in_portions_and_mixed(case, dtype):
    """One model, several ways of cutting the same requests: all must give the plain model's logits at every place.
    Every way starts on pages and state slots that the way before used."""
    raw = CASES[case]
    weights = random_weights(raw, seed=len(case))
    vocab = raw["vocab"]
    requests = {"a": rc.random_ids(vocab, 131, 1), "b": rc.random_ids(vocab, 37, 2), "c": rc.random_ids(vocab, 2, 3),
                "d": rc.random_ids(vocab, 1, 4), "e": rc.random_ids(vocab, 50, 5)}  # fmt: skip
    refs = {}
    replay = make_replay(raw, weights, dtype, max_tokens=4 * 192)
    manager = replay.manager
    free_pages = manager.num_free
    ways = [(rid + " whole", rc.whole(rid, ids)) for rid, ids in requests.items()]
    ways.append(("a decoded", rc.prefill_then_decode("a", requests["a"], tail=90)))
    ways.append(("b token by token", rc.prefill_then_decode("b", requests["b"], tail=36)))
    ways.append(("a portions", rc.portions("a", requests["a"])))
    ways.append(("e portions of two", rc.portions("e", requests["e"], sizes=(2,))))
    ways.append(("mixed", rc.mixed(requests, seed=7, max_live=3)))
    ways.append(("mixed again", rc.mixed(requests, seed=8, max_live=4, sizes=(2, 3, 16, 17, 5))))
    total = Against()
    for name, steps in ways:
        result = compare(replay, steps, requests, raw, weights, refs, dtype)
        if dtype == "float32":
            result.check(dtype, f"{case} {name}")
        total.take(result)
        assert manager.num_free == free_pages, name
    total.check(dtype, case)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("block_size", [4, 8, 64])
def test_pages_of_other_sizes(block_size, dtype):
    raw = CASES["all_kinds"]
    weights = random_weights(raw, seed=9)
    requests = {"a": rc.random_ids(raw["vocab"], 90, 6), "b": rc.random_ids(raw["vocab"], 33, 7), "c": rc.random_ids(raw["vocab"], 70, 8)}
    replay = make_replay(raw, weights, dtype, max_tokens=3 * 128, block_size=block_size, max_live=3)
    refs, total = {}, Against()
    for steps in (rc.portions("a", requests["a"], sizes=(5, 2, 30, 3, 9)), rc.mixed(requests, seed=3, max_live=3),
                  rc.prefill_then_decode("c", requests["c"], tail=45)):  # fmt: skip
        total.take(compare(replay, steps, requests, raw, weights, refs, dtype))
    total.check(dtype, f"pages of {block_size}")
    assert replay.manager.num_free == replay.manager.num_blocks


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding_past_many_pages(dtype):
    """A short prompt and 150 tokens decoded one by one (captured steps) over pages of 8 tokens, past every window; a
    second request starts beside it later, decodes from another position and ends first."""
    raw = CASES["matrix_cores"] if dtype == "bfloat16" else CASES["all_kinds"]
    weights = random_weights(raw, seed=21)
    a, b = rc.random_ids(raw["vocab"], 160, 11), rc.random_ids(raw["vocab"], 90, 12)
    refs = {}
    replay = make_replay(raw, weights, dtype, max_tokens=320, block_size=8 if dtype == "float32" else 16)
    got = {"a": [replay.step([{"id": "a", "tokens": a[:10], "want": list(range(10))}], [])], "b": []}
    for i in range(10, 160):
        entries = [{"id": "a", "tokens": [a[i]], "want": [0]}]
        j = i - 40
        if j == 0:
            entries.append({"id": "b", "tokens": b[:3], "want": [0, 1, 2]})
        elif 3 <= j < 90:
            entries.append({"id": "b", "tokens": [b[j]], "want": [0]})
        out = replay.step(entries, [e["id"] for e in entries if (e["id"] == "a" and i == 159) or (e["id"] == "b" and j == 89)])
        got["a"].append(out[:1])
        if len(entries) > 1:
            got["b"].append(out[1:])
    for rid, ids in (("a", a), ("b", b)):
        result = Against()
        result.add(torch.cat(got[rid]), *reference(raw, weights, ids, refs, rid, dtype))
        result.check(dtype, rid)
    assert replay.manager.num_free == replay.manager.num_blocks
    if dtype == "float32":
        assert replay.runner.decode_graphs.graphs, "decode steps were not captured"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_greedy_generation_through_the_scheduler(dtype):
    """The engine's own entry point: prompts of unequal lengths under a small token budget (so prompts are cut) and a
    pool small enough that pages and slots are used again; greedy tokens are the plain model's."""
    from atomserve_amd.config import EngineConfig
    from atomserve_amd.engine.engine import create_engine
    from atomserve_amd.engine.sequence import SamplingParams

    raw = CASES["all_kinds"]
    weights = random_weights(raw, seed=33)
    model = build_model(raw, weights, dtype)
    engine = create_engine(model, EngineConfig(block_size=16, num_blocks=24, max_model_len=128, max_num_seqs=2,
                                               max_num_batched_tokens=12))  # fmt: skip
    assert not engine.scheduler.manager.prefix_reuse_possible
    prompts = [rc.random_ids(raw["vocab"], n, 40 + n) for n in (5, 29, 1, 44)]
    outs = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=7, ignore_eos=True))
    assert engine.scheduler.manager.num_free == 24
    for prompt, out in zip(prompts, outs):
        assert len(out) == 7
        seq = list(prompt)
        for t in out:
            ref = plain.logits(raw, weights, seq)[-1]
            if dtype == "float32":
                assert t == int(ref.argmax())
            else:  # as good as the best token but for what rounding moves the plain model's own logits here
                moved = float((plain.logits(raw, weights, seq, rounded=True)[-1] - ref).abs().max())
                assert ref[t] >= ref.max() - 2e-2 * float(ref.abs().max()) - 2.0 * moved, (seq, t, float(ref[t]), float(ref.max()), moved)
            seq.append(t)


def test_the_replay_tool_on_a_folder(tmp_path):
    """The replay tool's own main on a model folder written here: config.json names the architecture, and the rank of
    the decays' two-step projection, which this config.json does not name, is read from the tensors' shapes."""
    import io

    import numpy as np
    from safetensors.torch import save_file

    from atomserve_amd.engine import replay

    raw = json.loads(json.dumps(CASES["odd_sizes"]))
    weights = random_weights(raw, seed=17)
    raw["layers"][2]["mixer"]["right"].pop("rank")
    folder = tmp_path / "model"
    os.makedirs(folder)
    save_file({k: v.bfloat16().contiguous() for k, v in weights.items()}, str(folder / "model.safetensors"))
    (folder / "config.json").write_text(json.dumps(raw))
    ids = rc.random_ids(raw["vocab"], 30, 2)
    lines = [json.dumps({"step": 0, "entries": [{"id": "x", "tokens": ids[:21], "want": [3, 20]}], "end": []}),
             json.dumps({"step": 1, "entries": [{"id": "x", "tokens": ids[21:], "want": [8]}], "end": ["x"]})]  # fmt: skip
    out = tmp_path / "out"
    assert replay.main(["--model", str(folder), "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                       stdin=io.StringIO("\n".join(lines) + "\n")) == 0  # fmt: skip
    ref = plain.logits(CASES["odd_sizes"], weights, ids)
    got0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1))
    got1 = torch.from_numpy(np.fromfile(out / "1.f32", dtype="<f4").reshape(1, -1))
    assert (got0 - ref[[3, 20]]).abs().max() <= 3e-5 * float(ref.abs().max())
    assert (got1 - ref[[29]]).abs().max() <= 3e-5 * float(ref.abs().max())


def test_the_command_line_generates_from_a_folder_and_from_random_weights(tmp_path, capsys):
    from safetensors.torch import save_file

    from atomserve_amd.engine import cli

    raw = CASES["all_kinds"]
    weights = random_weights(raw, seed=17)
    (tmp_path / "config.json").write_text(json.dumps(raw))
    save_file({k: v.bfloat16().contiguous() for k, v in weights.items()}, str(tmp_path / "model.safetensors"))
    prompt = rc.random_ids(raw["vocab"], 21, 3)
    common = ["--dtype", "fp32", "--prompt-ids", " ".join(map(str, prompt)), "--max-tokens", "5", "--temperature", "0",
              "--ignore-eos", "--kv-mem-gb", "0.05", "--max-num-seqs", "2", "--max-batched-tokens", "16"]  # fmt: skip
    assert cli.main([str(tmp_path), *common]) == 0
    lines = [json.loads(line) for line in capsys.readouterr().out.splitlines() if line.startswith("{")]
    want, seq = [], list(prompt)
    for _ in range(5):
        want.append(int(plain.logits(raw, weights, seq)[-1].argmax()))
        seq.append(want[-1])
    assert lines[-1]["output_ids"] == want
    assert cli.main([str(tmp_path), "--random-weights", "3", *common]) == 0
    lines = [json.loads(line) for line in capsys.readouterr().out.splitlines() if line.startswith("{")]
    assert len(lines[-1]["output_ids"]) == 5


def normed_sum(y):
    """What a `NormedSum` stands for, in float64."""
    total = 0.0
    for t, bias, gain in zip(y.ys, y.biases, y.gains):
        t = t.double() if bias is None else t.double() + bias.double()
        total = total + plain.rms(t, y.eps) * gain.double()
    return total


def settled(delta):
    """What a pending output adds to the stream, in float64."""
    from atomserve_amd.parts.base import NormedSum

    y = normed_sum(delta.y) if isinstance(delta.y, NormedSum) else delta.y.double()
    return plain.rms(y, delta.norm.spec.eps) * delta.norm.gain_f32.double()


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", ["all_kinds", "odd_sizes", "wide"])
def test_the_stream_after_every_layer(case, dtype):
    """The stream after every layer against the plain model's: a fault shows at the first layer it touches."""
    raw = CASES[case]
    weights = random_weights(raw, seed=4)
    ids = rc.random_ids(raw["vocab"], 45, 3)
    want, rounded = [], []
    plain.forward(raw, weights, ids, layers_out=want)
    if dtype == "bfloat16":
        plain.forward(raw, weights, ids, bf16=True, layers_out=rounded)
    replay = make_replay(raw, weights, dtype, max_tokens=64)
    seen = []
    for block in replay.model.blocks:
        inner = block.forward

        def watched(x, delta, step, *a, inner=inner, **k):
            d = inner(x, delta, step, *a, **k)
            seen.append((x.double() + settled(d)).cpu())  # the layer's last sum is still pending
            return d

        block.forward = watched
    replay.step([{"id": "a", "tokens": ids, "want": [44]}], ["a"])
    assert len(seen) == len(want) == len(raw["layers"])
    for i, (got, ref) in enumerate(zip(seen, want)):
        rows = (got - ref).abs().max(-1).values
        if dtype == "float32":
            assert float(rows.max()) <= 2e-5 * float(ref.abs().max()), f"layer {i}: {float(rows.max()):.3e} of {float(ref.abs().max()):.3e}"
            continue
        noise = (rounded[i] - ref).abs().max(-1).values
        assert float(rows.median()) <= 2.0 * float(noise.median()) and float(rows.quantile(0.9)) <= 2.0 * float(noise.quantile(0.9)), (
            f"layer {i}: rows' median {float(rows.median()):.3e} and ninth decile {float(rows.quantile(0.9)):.3e}; the plain "
            f"model's {float(noise.median()):.3e} and {float(noise.quantile(0.9)):.3e}")  # fmt: skip


# ---- what a query sees: the attention kernels alone -----------------------------------------------------------------


def paged(k, v, bs, gen, dtype, width):
    """Pages in a shuffled order that hold k [L, G, D] and v [L, G, E], heads laid out `width` wide; the rest of the pool is
    filled with large numbers that nobody may see."""
    L, G, D = k.shape
    pages = -(-L // bs)
    pool = pages + 3
    kp, vp = torch.full((pool, G, bs, width), 7.0), torch.full((pool, G, width, bs), 1e3)
    order = torch.randperm(pool, generator=gen)[:pages]
    for i in range(L):
        p, o = int(order[i // bs]), i % bs
        kp[p, :, o, :], vp[p, :, :, o] = 0.0, 0.0
        kp[p, :, o, :D] = k[i]
        vp[p, :, : v.shape[2], o] = v[i]
    table = order.to(I32).view(1, -1)
    return kp.to(DEV).to(dtype), vp.to(DEV).to(dtype), table.to(DEV)


SIGHTS = [  # window, first tokens that stay visible, cap of the scores, sink
    (0, 0, 0.0, True), (0, 0, 3.0, False), (1, 0, 0.0, False), (1, 1, 2.0, True), (2, 70, 0.0, True), (31, 5, 0.0, False), (32, 33, 5.0, True),
    (33, 64, 0.0, False), (64, 20, 4.0, True), (65, 1, 0.0, False), (100, 130, 6.0, True), (250, 30, 0.0, False), (500, 7, 0.0, True),
]  # fmt: skip


@pytest.mark.parametrize("sight", SIGHTS)
@pytest.mark.parametrize("sizes", [(4, 2, 64, 16), (2, 1, 96, 16), (20, 1, 32, 32), (3, 3, 40, 8), (2, 2, 272, 16)])
def test_attention_kernels_under_every_mask_cap_and_sink(sizes, sight):
    """Windows with kept first tokens, capped scores and the sink in every attention kernel: single queries in 32 bits
    and on the matrix cores (several partitions and one, groups of more heads than a tile), prompts (both tilings, cut
    into pieces and whole), and heads of any width; scores large enough that the cap bites, some heads' scores all far
    below zero so that the sink takes nearly everything."""
    from atomserve_amd.kernels import ops

    H, G, D, bs = sizes
    window, keep, cap, sink = sight
    L = 331
    gen = torch.Generator().manual_seed(H * 1000 + D + window)
    q, k, v = torch.randn(L, H, D, generator=gen), torch.randn(L, G, D, generator=gen), torch.randn(L, G, D, generator=gen)
    q[:, H - 1] *= 3.0
    k[:, :, 0], q[:, 0, 0] = 2.0, -6.0  # the first head's scores lie below zero
    q, k, v = (t.bfloat16().float() for t in (q, k, v))
    scale = 3.0 * D**-0.5
    mask = {"size": window, "keep_first": keep} if window else None
    want = plain.attention(q.double(), k.double(), v.double(), scale, mask, cap, sink).float()
    how = dict(keep_first=keep, softcap=cap, sink=sink)
    pos = torch.arange(L, dtype=I32, device=DEV)
    row = torch.zeros(L, dtype=I32, device=DEV)
    checks = 0
    for dtype in (torch.float32, torch.bfloat16):
        tol = (2e-5 if dtype == torch.float32 else 2e-2) * float(v.abs().max())
        kp, vp, table = paged(k, v, bs, gen, dtype, D)
        qd = q.to(DEV).to(dtype)

        def check(out, what):
            nonlocal checks
            err = (out.float().cpu() - want).abs().amax(dim=(1, 2))
            worst = int(err.argmax())
            assert float(err.max()) <= tol, f"{what} {dtype} {sizes} {sight}: {float(err.max()):.3e} at {worst}"
            checks += 1

        for out_dtype in {dtype, torch.float32}:
            out = torch.empty(L, H, D, dtype=out_dtype, device=DEV)
            ops.wide_attend(qd, kp, vp, pos, row, table, out, scale, L, window, **how)
            check(out, "any width")
        if D > ops.SINGLE_QUERY_MAX_HEAD_DIM:
            continue
        for part in (None, 64, 32 * -(-(L + 64) // 32)):
            for generic in (False, True):  # (and the results of bfloat16 heads in fp32)
                out = torch.full((L, H, D), float("nan"), dtype=torch.float32 if part == 64 else dtype, device=DEV)
                ops.attn_single_query(qd, kp, vp, None, pos, row, table, out, scale, window, L, part, force_generic=generic, **how)
                check(out, f"single queries, partitions of {part}, general {generic}")
        if ops.attn_prefill_supported(dtype, D, bs):
            for first in (0, 77):  # a whole prompt, and portions behind a cached prefix
                tiles = [[t, min(64, L - t), 0, t] for t in range(first, L, 64)]
                for kind in (1, 2):
                    for pieces in (1, 3):
                        before, ops.PREFILL_PIECES = ops.PREFILL_PIECES, pieces
                        out = want.to(DEV).to(torch.float32 if kind == 1 else dtype).clone()
                        out[first:] = float("nan")
                        try:
                            ops.attn_prefill(qd, kp, vp, torch.tensor(tiles[::-1], dtype=I32, device=DEV), table, out, scale, window, L, kind, **how)
                        finally:
                            ops.PREFILL_PIECES = before
                        check(out, f"prompt from {first}, {kind} query tiles, {pieces} pieces")
    assert checks >= 2


# ---- each mechanism alone -------------------------------------------------------------------------------------


def env_for(dtype):
    from atomserve_amd.kernels import ops
    from atomserve_amd.parts.base import BuildEnv

    return BuildEnv(DTYPES[dtype], torch.device(DEV), products=ops.ProductChoices(fixed=True))


def bf(x):
    return x.bfloat16().float()


def run_mixers(mixers, inputs, cuts, dtype, block_size=16, slots=3, warm=None, reads=None):
    """Mixers alone (one after the other in every step, sharing the step's results) over one request cut into rows of `cuts`
    tokens; reads: mixer -> the mixer whose caches it reads (it writes none); warm: how many tokens another request
    first runs on the same slot and pages before it ends, so that what it left must not show.  Returns each mixer's outputs."""
    from atomserve_amd.cache.manager import CacheManager
    from atomserve_amd.cache.pools import CachePools
    from atomserve_amd.engine.batch import Row, StepBatch
    from atomserve_amd.parts.base import NormedSum

    reads = reads or {}
    asked = {}
    for i, mixer in enumerate(mixers):
        if i not in reads:
            req = mixer.cache_request()
            asked.update({(i, name): r for name, r in req.items()} if isinstance(req, dict) else {i: req})
    manager = CacheManager(asked, block_size, 64, slots)
    pools = CachePools(manager, DTYPES[dtype], DEV)
    splits = sorted({s for s in [m.row_split() for m in mixers] if s is not None})

    def feed(xs, pieces):
        req, at, outs = manager.new_request(), 0, [[] for _ in mixers]
        for n in pieces:
            assert manager.reserve(req, at, n)
            batch = StepBatch([Row([0] * n, at, req.tables, [], req.state_slot)], block_size, len(manager.paged_groups), 10,
                              DEV, pools=pools, row_splits=splits)  # fmt: skip
            for i, (mixer, x) in enumerate(zip(mixers, xs)):
                y = mixer.forward(x[at : at + n].to(DEV).to(DTYPES[dtype]).contiguous(), batch, batch.cache_view(reads.get(i, i), i not in reads))
                outs[i].append((normed_sum(y) if isinstance(y, NormedSum) else y).float().cpu())
            at += n
            manager.release_behind_window(req, at)
        manager.release(req)
        return [torch.cat(o) for o in outs]

    if warm:
        gen = torch.Generator().manual_seed(warm)
        feed([bf(torch.randn(warm, x.shape[1], generator=gen) * 3) for x in inputs], [warm])
    return feed(inputs, cuts)


def give(part, tensors, dtype):
    part.bind({k: v.to(DEV).to(DTYPES[dtype]).contiguous() for k, v in tensors.items()})
    return part


def mask_of(window, keep):
    return {"size": window, "keep_first": keep} if window else None


def differential_weights(hidden, m, gen, std=0.3):
    def mat(*s, sd=std):
        return bf(torch.randn(*s, generator=gen) * sd)

    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    w = {"q": mat(2 * H * D, hidden), "k": mat(2 * G * D, hidden), "v": mat(G * E, hidden), "o": mat(hidden, H * E)}
    w.update({name: mat(D, sd=0.8 * D**-0.25) for name in ("lq1", "lk1", "lq2", "lk2")})
    return w


def bind_differential(w, hidden, m, dtype, own=True, cache=(None, None)):
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import JoinedMixerSpec, SoftmaxCoreSpec

    mask = m.get("mask") or {"size": 0, "keep_first": 0}
    core = SoftmaxCoreSpec("softmax_core", m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], window=mask["size"],
                           keep_first=mask["keep_first"], maps=2, difference=m["diff"], difference_eps=1e-5, own_kv=own,
                           cache_window=cache[0], cache_keep_first=cache[1])  # fmt: skip
    part = build("mixer", JoinedMixerSpec("joined", hidden, (core,), (1.0,)), env_for(dtype))
    t = {"in.weight": torch.cat([w[k] for k in (("q", "k", "v") if own else ("q",))]), "out_t.weight": w["o"].t()}
    t.update({"c0." + name: w[name] for name in ("lq1", "lk1", "lq2", "lk2")})
    return give(part, t, dtype)


def plain_differential(h, w, m, kept=None, index=0, rounded=False):
    return plain.differential_attention(h.double(), {"x." + k: v.double() for k, v in w.items()}, "x.", m, 1e-5, rounded,
                                        {} if kept is None else kept, index).float()  # fmt: skip


def close(got, ref, rounded, dtype, what):
    """32-bit: every number.  bfloat16: the rows' largest errors as a distribution against the plain mixer's own when its
    activations are rounded (two maps that nearly cancel make what is left of them, and of every rounding, larger)."""
    rows = (got - ref).abs().amax(-1)
    if dtype == "float32":
        assert float(rows.max()) <= 3e-5 * max(1.0, float(ref.abs().max())), f"{what}: {float(rows.max()):.3e} of {float(ref.abs().max()):.3e}"
        return
    noise = (rounded - ref).abs().amax(-1)
    for q in (0.5, 0.9):
        assert float(rows.quantile(q)) <= 2.0 * float(noise.quantile(q)), f"{what}: {float(rows.quantile(q)):.3e}, rounding alone {float(noise.quantile(q)):.3e}"
    assert float(rows.max()) <= 4.0 * float(noise.max()), f"{what}: {float(rows.max()):.3e}, rounding alone {float(noise.max()):.3e}"


DIFFERENTIALS = [  # heads, kv heads, keys, values, window, kept first tokens, diff
    (4, 2, 16, 32, 13, 3, 0.2), (3, 3, 5, 14, 0, 0, 0.7), (8, 2, 32, 64, 9, 12, 0.3), (4, 1, 64, 128, 1, 1, 0.5), (2, 2, 24, 96, 20, 0, 0.0),
    (2, 1, 140, 24, 10, 4, 0.4), (6, 2, 8, 8, 5, 40, 0.8),
]  # fmt: skip


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", DIFFERENTIALS)
def test_differential_attention_alone(shape, dtype):
    H, G, D, E, window, keep, diff = shape
    hidden, T = 64, 45
    gen = torch.Generator().manual_seed(H * 100 + D)
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": D**-0.5, "diff": diff, "mask": mask_of(window, keep)}
    w = differential_weights(hidden, m, gen)
    h = bf(torch.randn(T, hidden, generator=gen))
    ref = plain_differential(h, w, m)
    one_map = plain_differential(h, dict(w, lq1=w["lq1"] * 0, lq2=w["lq2"] * 0), dict(m, diff=0.0))
    assert (ref - one_map).abs().max() > 0.05 * ref.abs().max(), "the second map does not matter in this test"
    part = bind_differential(w, hidden, m, dtype)
    rounded = plain_differential(h, w, m, rounded=True)
    for cuts in ([T], [1] * T, [19, 1, 2, 2, 1, 17, 3], [2, 43]):
        (got,) = run_mixers([part], [h], cuts, dtype, warm=9)
        close(got, ref, rounded, dtype, f"{shape} {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("masks", [((6, 2), (11, 1), (3, 9)), ((5, 0), (0, 0), (20, 3)), ((0, 0), (4, 2), (9, 0))])
def test_layers_that_read_another_layers_keys(masks, dtype):
    """One layer with keys and values of its own and two that read them with queries, a lambda and masks of their own,
    wider and narrower: the pages keep what the widest reader sees, also when the tokens come one by one."""
    hidden, T = 48, 50
    gen = torch.Generator().manual_seed(3)
    base = {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 32}
    ms = [dict(base, scale=s, diff=d, mask=mask_of(*mask)) for mask, s, d in zip(masks, (0.25, 0.3, 0.2), (0.3, 0.5, 0.1))]
    ms[1]["kv_from"] = ms[2]["kv_from"] = 0
    ws = [differential_weights(hidden, m, gen) for m in ms]
    hs = [bf(torch.randn(T, hidden, generator=gen)) for _ in ms]
    kept, kept_rounded = {}, {}
    refs = [plain_differential(h, w, m, kept, i) for i, (h, w, m) in enumerate(zip(hs, ws, ms))]
    rounded = [plain_differential(h, w, m, kept_rounded, i, rounded=True) for i, (h, w, m) in enumerate(zip(hs, ws, ms))]
    window = 0 if any(w == 0 for w, _ in masks) else max(w for w, _ in masks)
    cache = (window, max(k for _, k in masks) if window else 0)
    parts = [bind_differential(w, hidden, m, dtype, own=i == 0, cache=cache) for i, (w, m) in enumerate(zip(ws, ms))]
    for cuts in ([T], [1] * T, [17, 2, 1, 30], [2] * 25):
        got = run_mixers(parts, hs, cuts, dtype, block_size=4 if dtype == "float32" else 16, warm=5, reads={1: 0, 2: 0})
        for i, g in enumerate(got):
            close(g, refs[i], rounded[i], dtype, f"layer {i} {cuts[:4]}")


@pytest.mark.parametrize("dtype,block_size", [("float32", 8), ("bfloat16", 16), ("bfloat16", 64)])
def test_keys_just_inside_and_just_outside_a_window_and_the_first_tokens(dtype, block_size):
    """One token's keys stand out for every query and its value is large: outputs change by their own size where the
    token enters or leaves what a position sees.  The token stands in the middle (seen for exactly `size` positions), as
    the last of the kept first tokens (seen for good) and as the one behind it (seen for `size` positions only); its
    readers come in one prompt, in portions and token by token, hundreds of positions on."""
    hidden, T, size, keep = 32, 230, 40, 6
    m = {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 32, "scale": 1.0, "diff": 0.3, "mask": mask_of(size, keep)}
    for mark in (0, keep - 1, keep, block_size - 1, 70, 2 * block_size):
        gen = torch.Generator().manual_seed(500 + mark)
        w = differential_weights(hidden, m, gen, std=0.2)
        direction = bf(torch.randn(w["k"].shape[0], generator=gen))  # keys of both maps of both kv heads
        w["k"] = w["k"] * 0.2
        w["k"][:, 0] = 0.4 * direction
        w["q"] = w["q"] * 0.2
        w["q"][:, 1] = torch.cat([0.4 * direction.view(2, -1)[g] for g in (0, 0, 1, 1)])
        h = bf(torch.randn(T, hidden, generator=gen) * 0.3)
        h[:, 0], h[:, 1] = 0.0, 4.0  # every query asks, one key answers
        h[mark, 0] = 4.0
        h[mark, 2:] *= 6.0
        ref = plain_differential(h, w, m)
        blind = h.clone()
        blind[mark, 0] = 0.0
        shows = (plain_differential(blind, w, m) - ref).abs().amax(-1) > 0.1 * ref.abs().max()
        assert bool(shows[mark + 1 : mark + size].all()) and bool(shows[max(mark + size, keep) :].all()) == (mark < keep)
        assert mark < keep or not bool(shows[mark + size :].any())
        part = bind_differential(w, hidden, m, dtype)
        rounded = plain_differential(h, w, m, rounded=True)
        edge = mark + size
        for cuts in ([T], [edge - 1, 1, 1, T - edge - 1], [edge - 3, 2, 2, 2, T - edge - 3], [mark + 1, 5] + [1] * (T - mark - 6), [64, 64, 64, 38]):
            (got,) = run_mixers([part], [h], [c for c in cuts if c > 0], dtype, block_size=block_size, warm=20)
            close(got, ref, rounded, dtype, f"mark {mark} {cuts[:4]}")


def parallel_weights(hidden, left, right, gen):
    def mat(*s, sd=0.3):
        return bf(torch.randn(*s, generator=gen) * sd)

    H, G, D, E = left["heads"], left["kv_heads"], left["dim"], left["vdim"]
    w = {}
    for name, rows, cols in (("q", H * D, hidden), ("k", G * D, hidden), ("v", G * E, hidden), ("o", hidden, H * E)):
        w["left." + name], w["left." + name + ".b"] = mat(rows, cols), mat(rows)
    H, D, E, R = right["heads"], right["dim"], right["vdim"], right["rank"]
    w.update({"right.q": mat(H * D, hidden), "right.k": mat(H * D, hidden), "right.v": mat(H * E, hidden), "right.g": mat(H * E, hidden),
              "right.o": mat(hidden, H * E), "right.norm": bf(1 + 0.2 * torch.randn(E, generator=gen)), "right.a1": mat(R, hidden),
              "right.a2": mat(H * D, R, sd=0.6), "right.a2.b": mat(H * D, sd=1.5),
              "left.out": bf(1 + 0.2 * torch.randn(hidden, generator=gen)), "right.out": bf(1 + 0.2 * torch.randn(hidden, generator=gen))})  # fmt: skip
    return w


def bind_parallel(w, hidden, left, right, dtype):
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import ChannelDecaySpec, JoinedMixerSpec, NeighbourRotarySpec, SoftmaxCoreSpec

    rot = left.get("rot")
    position = NeighbourRotarySpec("rope_neighbours", rot["dims"], rot["base"], slower=(rot.get("scaling") or {"factor": 1.0})["factor"]) if rot else None
    cores = (SoftmaxCoreSpec("softmax_core", left["heads"], left["kv_heads"], left["dim"], left["vdim"], left["scale"], bias=True,
                             position=position, softcap=left.get("softcap", 0.0), sink=True),
             ChannelDecaySpec("channel_decay", right["heads"], right["dim"], right["vdim"], right["rank"], right["tau"], 1e-5))  # fmt: skip
    part = build("mixer", JoinedMixerSpec("joined", hidden, cores, (0.5, 0.5), out_norm_eps=1e-5, out_bias=(True, False)), env_for(dtype))
    t = {"in.weight": torch.cat([w["left." + k] for k in "qkv"] + [w["right." + k] for k in ("q", "k", "v", "g", "a1")]),
         "out0.weight": w["left.o"], "out0.bias": w["left.o.b"], "out0.norm": w["left.out"], "out1.weight": w["right.o"],
         "out1.norm": w["right.out"], "c1.decay_up": w["right.a2"], "c1.decay_bias": w["right.a2.b"], "c1.out_norm": w["right.norm"]}  # fmt: skip
    t.update({f"c0.{k}_bias": w[f"left.{k}.b"] for k in "qkv"})
    return give(part, t, dtype)


PARALLELS = [  # left: heads, kv heads, keys, values, rotation, cap; right: heads, keys, values, tau, rank
    (4, 2, 16, 24, (8, 100.0, 3.0), 4.0, (3, 16, 8, 8.0, 5)), (3, 3, 10, 14, (10, 500.0, None), None, (2, 6, 13, 1.0, 1)),
    (8, 2, 64, 64, (64, 1e5, 2.0), 10.0, (2, 128, 64, 16.0, 8)), (2, 1, 96, 32, (2, 50.0, None), 1.5, (1, 40, 72, 0.5, 3)),
    (2, 2, 24, 264, (24, 2000.0, 5.0), 3.0, (2, 150, 12, 4.0, 9)),
]  # fmt: skip


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", PARALLELS)
def test_sink_attention_beside_linear_attention(shape, dtype):
    """Both halves, their biases, the norms of their outputs and the half sum; and each half alone, the other's output
    matrix being zero."""
    H, G, D, E, rot, cap, (rh, rd, rv, tau, rank) = shape
    hidden, T = 64, 75
    gen = torch.Generator().manual_seed(H * 100 + D)
    left = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": 2 * D**-0.5, "rot": {"dims": rot[0], "base": rot[1]}}
    if rot[2]:
        left["rot"]["scaling"] = {"factor": rot[2]}
    if cap:
        left["softcap"] = cap
    right = {"heads": rh, "dim": rd, "vdim": rv, "tau": tau, "rank": rank}
    w = parallel_weights(hidden, left, right, gen)
    h = bf(torch.randn(T, hidden, generator=gen))
    for without in (None, "left.o", "right.o"):
        ww = dict(w)
        if without:
            ww[without] = torch.zeros_like(w[without])
            if without == "left.o":
                ww["left.o.b"] = torch.zeros_like(w["left.o.b"])
        ref = plain.parallel_mixer(h.double(), {"x." + k: v.double() for k, v in ww.items()}, "x.", {"left": left, "right": right},
                                   torch.arange(T), 1e-5, False).float()  # fmt: skip
        part = bind_parallel(ww, hidden, left, right, dtype)
        tol = (5e-5 if dtype == "float32" else 6e-2) * max(1.0, float(ref.abs().max()))
        for cuts in ([T], [1] * T, [19, 1, 2, 2, 1, 47, 3], [33, 42]) if without is None else ([T], [40, 1, 34]):
            (got,) = run_mixers([part], [h], cuts, dtype, warm=9)
            assert (got - ref).abs().max() <= tol, f"{shape} {without} {cuts}: {float((got - ref).abs().max()):.3e} of {float(ref.abs().max()):.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(3, 64, 40), (2, 128, 96), (1, 24, 72), (2, 10, 6), (4, 36, 32), (2, 200, 16)])
def test_channel_decays_and_the_three_ways_to_run_them(sizes, dtype):
    """The decays from their two-step projection, and the recurrence token by token, one token a row and in chunks of 32,
    over several rows of one step, from states that another request left.  Decays lie anywhere between 0 and 1, some are
    1 exactly, some so small that a product of a few leaves the range of 32-bit numbers."""
    from atomserve_amd.kernels import ops

    H, D, E = sizes
    dt = DTYPES[dtype]
    gen = torch.Generator().manual_seed(D + E)
    rank, tau = 6, 2.0
    lens, starts, slots = [70, 1, 33, 32], [0, 5, 9, 0], [2, 0, 1, 3]
    T = sum(lens)
    proj = bf(torch.randn(T, 2 * H * D + H * E + rank, generator=gen))
    up, bias = bf(torch.randn(H * D, rank, generator=gen)), bf(torch.randn(H * D, generator=gen) * 3)
    alpha = torch.empty((T, H * D), dtype=torch.float32, device=DEV)
    ops.channel_decays(proj.to(DEV).to(dt), 2 * H * D + H * E, rank, up.to(DEV).to(dt), bias.to(DEV), tau, alpha)
    z = proj[:, -rank:].double() @ up.double().t() + bias.double()
    exact = plain.channel_decays(z, tau)
    assert (alpha.cpu().double() - exact).abs().max() <= 2e-6
    for n, wide, tau_ in ((8, 8, 0.25), (77, 40, 16.0), (130, 64, 1.0)):  # ranks whose second step runs on the matrix cores
        low, up_, b_ = bf(torch.randn(n, wide + 8, generator=gen)), bf(torch.randn(H * D, wide, generator=gen)), torch.randn(H * D, generator=gen) * 20
        out = torch.full((n, H * D), float("nan"), dtype=torch.float32, device=DEV)
        ops.channel_decays(low.to(DEV).to(dt), 8, wide, up_.to(DEV).to(dt), b_.to(DEV), tau_, out)
        want_ = plain.channel_decays(low[:, 8:].double() @ up_.double().t() + b_.double(), tau_)
        assert (out.cpu().double() - want_).abs().max() <= 2e-6, (n, wide, tau_)
    al = exact.float().view(T, H, D).clone()
    pick = torch.rand(T, H, D, generator=gen)
    al[pick < 0.1] = 1.0
    al[pick > 0.93] = 1e-7
    al[:, 0, 0] = torch.where(torch.arange(T) % 7 == 3, torch.tensor(3e-13), torch.tensor(1.0))
    state0 = torch.randn(5, H, D, E, generator=gen)
    want, final, at = torch.zeros(T, H, E, dtype=torch.float64), state0.double().clone(), 0
    q, k = proj[:, : H * D].double().view(T, H, D), proj[:, H * D : 2 * H * D].double().view(T, H, D) * 0.3
    v = proj[:, 2 * H * D : 2 * H * D + H * E].double().view(T, H, E)
    for n, start, slot in zip(lens, starts, slots):
        S = final[slot].clone() if start > 0 else torch.zeros(H, D, E, dtype=torch.float64)
        for t in range(at, at + n):
            S = al[t].double().unsqueeze(2) * S + k[t].unsqueeze(2) * v[t].unsqueeze(1)
            want[t] = torch.einsum("hde,hd->he", S, q[t])
        final[slot] = S
        at += n
    firsts = [sum(lens[:i]) for i in range(len(lens))]
    ints = [torch.tensor(x, dtype=I32, device=DEV) for x in (firsts, lens, starts, slots)]
    pd = proj.to(DEV).to(dt)
    for kernel in ("scan", "chunks"):
        if kernel == "chunks" and D > ops.DECAY_CHUNKS_MAX_DIM:
            continue
        state = state0.clone().to(DEV)
        out = torch.empty((T, H, E), dtype=torch.float32, device=DEV)
        rows = (torch.cat([torch.full((n,), i, dtype=I32) for i, n in enumerate(lens)]).to(DEV), *ints)
        ops.channel_attention(pd, 0, H * D, 2 * H * D, H, D, E, 0.3, al.view(T, -1).to(DEV), state, rows, out, kernel=kernel)
        assert (out.cpu().double() - want).abs().max() <= 2e-5 * float(want.abs().max()), kernel
        assert (state.cpu().double() - final).abs().max() <= 2e-5 * float(final.abs().max()), f"{kernel}: the state"
    # one token a row: the first token of each row
    ones = torch.ones(len(lens), dtype=I32, device=DEV)
    for kernel in ("scan", "step"):
        if kernel == "step" and (E % 4 or D > ops.DECAY_CHUNKS_MAX_DIM):
            continue
        state = state0.clone().to(DEV)
        out = torch.full((T, H, E), float("nan"), dtype=torch.float32, device=DEV)
        rows = (torch.zeros(T, dtype=I32, device=DEV), ints[0], ones, ints[2], ints[3])
        ops.channel_attention(pd, 0, H * D, 2 * H * D, H, D, E, 0.3, al.view(T, -1).to(DEV), state, rows, out, kernel=kernel)
        assert (out.cpu().double()[firsts] - want[firsts]).abs().max() <= 2e-5 * float(want.abs().max()), kernel
        for f, start, slot in zip(firsts, starts, slots):
            S = al[f].double().unsqueeze(2) * state0[slot].double() if start else torch.zeros(H, D, E, dtype=torch.float64)
            S = S + k[f].unsqueeze(2) * v[f].unsqueeze(1)
            assert (state.cpu()[slot].double() - S).abs().max() <= 2e-5 * float(S.abs().max()), f"{kernel}: the state"


def test_linear_attention_keeps_a_far_token():
    """With decays near one and a query that asks for one early token's key, the output hundreds of tokens later is that
    token's value: a state that was lost or restarted on the way shows as a difference of the output's size."""
    hidden, T = 48, 300
    left = {"heads": 2, "kv_heads": 1, "dim": 8, "vdim": 8, "scale": 0.3, "rot": {"dims": 4, "base": 100.0}}
    right = {"heads": 2, "dim": 32, "vdim": 16, "tau": 16.0, "rank": 4}
    gen = torch.Generator().manual_seed(5)
    w = parallel_weights(hidden, left, right, gen)
    w["right.a2"], w["right.a2.b"] = w["right.a2"] * 0, torch.full_like(w["right.a2.b"], 9.0)
    w["left.o"], w["left.o.b"] = w["left.o"] * 0, w["left.o.b"] * 0
    h = bf(torch.randn(T, hidden, generator=gen) * 0.05)
    half = hidden // 2  # queries and keys read one half of the input, values the other
    w["right.q"][:, :half], w["right.k"][:, :half], w["right.v"][:, half:] = 0.0, 0.0, 0.0
    h[3] = bf(torch.randn(hidden, generator=gen) * 4)
    h[T - 1, half:], h[T - 1, :half] = h[3, half:], bf(torch.randn(half, generator=gen) * 0.3)
    wd = {"x." + k: v.double() for k, v in w.items()}
    raw = {"left": left, "right": right}
    ref = plain.parallel_mixer(h.double(), wd, "x.", raw, torch.arange(T), 1e-5, False).float()
    forgot = plain.parallel_mixer(torch.cat([h[:3], h[4:]]).double(), wd, "x.", raw, torch.arange(T - 1), 1e-5, False).float()
    assert (forgot[-1] - ref[-1]).abs().max() > 0.1 * ref[-1].abs().max(), "the far token does not matter in this test"
    part = bind_parallel(w, hidden, left, right, "float32")
    for cuts in ([T], [150, 149, 1], [7] * 42 + [6], [299, 1], [4, 296], [3, 1, 296]):
        (got,) = run_mixers([part], [h], cuts, "float32", warm=11)
        assert (got - ref).abs().max() <= 1e-4 * max(1.0, float(ref.abs().max())), cuts


LATENTS = [  # heads, plain, turned, values, latent, window
    (3, 16, 8, 24, 40, 17), (5, 10, 6, 14, 22, 0), (4, 32, 32, 32, 96, 33), (6, 64, 32, 64, 128, 5), (2, 24, 0, 16, 30, 9), (17, 8, 4, 8, 12, 12),
    (2, 20, 12, 8, 250, 10),
]  # fmt: skip


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", LATENTS)
def test_latent_attention_over_a_window_alone(shape, dtype):
    """Queries that are a plain projection, a turned part of neighbouring pairs (or none), windows, no gate; one head's
    group larger than a tile, a latent wider than the paged kernels' heads."""
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import LatentAttentionSpec, NeighbourRotarySpec

    H, D, R, E, C, window = shape
    hidden, T = 64, 45
    gen = torch.Generator().manual_seed(sum(shape))

    def mat(*s, sd=0.3):
        return bf(torch.randn(*s, generator=gen) * sd)

    w = {"q": mat(H * (D + R), hidden), "dkv": mat(C + R, hidden), "dkv.norm": bf(1 + 0.2 * torch.randn(C, generator=gen)),
         "uk": mat(H * D, C, sd=0.15), "uv": mat(H * E, C, sd=0.15), "o": mat(hidden, H * E)}  # fmt: skip
    m = {"heads": H, "dim": D, "rot_dim": R, "vdim": E, "kv_rank": C, "scale": 0.2, "rot": {"dims": R, "base": 300.0}, "mask": mask_of(window, 0)}
    h = bf(torch.randn(T, hidden, generator=gen))
    ref = plain.latent_attention(h.double(), {"x." + k: v.double() for k, v in w.items()}, "x.", m, torch.arange(T), 1e-5, False).float()
    spec = LatentAttentionSpec("latent_attention", hidden, H, D, R, E, 0, C, 0.2, 1e-5,
                               NeighbourRotarySpec("rope_neighbours", R, 300.0) if R else None, out_gate=False, window=window)  # fmt: skip
    part = build("mixer", spec, env_for(dtype))
    give(part, {"in.weight": torch.cat([w["q"], w["dkv"]]), "kv_norm.weight": w["dkv.norm"], "uk.weight": w["uk"], "uv.weight": w["uv"],
                "o.weight": w["o"]}, dtype)  # fmt: skip
    tol = (3e-5 if dtype == "float32" else 4e-2) * max(1.0, float(ref.abs().max()))
    for cuts in ([T], [1] * T, [19, 1, 2, 2, 1, 17, 3], [2, 43]):
        (got,) = run_mixers([part], [h], cuts, dtype, block_size=4 if dtype == "float32" else 16, warm=9)
        assert (got - ref).abs().max() <= tol, f"{shape} {cuts}: {float((got - ref).abs().max()):.3e} of {float(ref.abs().max()):.3e}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [40, 90, 256, 1000, 4096, 5121, 16384, 20000])
def test_norm_residual_sum_and_next_norm_in_one_pass(n, dtype):
    from atomserve_amd.kernels import ops

    dt = DTYPES[dtype]
    tol = 2e-5 if dtype == "float32" else 1e-2
    for T in (3, 600) if n <= 4096 else (3,):
        gen = torch.Generator().manual_seed(n + T)
        x, y1, y2 = torch.randn(T, n, generator=gen) * 3, bf(torch.randn(T, n, generator=gen)), bf(torch.randn(T, n, generator=gen) * 9)
        post, gain, g1, g2 = (1 + 0.3 * torch.randn(n, generator=gen) for _ in range(4))
        b1, b2 = torch.randn(n, generator=gen), torch.randn(n, generator=gen)
        dev = lambda t: t.to(DEV)  # noqa: E731
        for pair, biases in ((False, (None, None)), (False, (b1, None)), (True, (None, None)), (True, (b1, b2)), (True, (None, b2))):
            d = y1.double() + (0 if biases[0] is None else biases[0].double())
            if pair:
                d2 = y2.double() + (0 if biases[1] is None else biases[1].double())
                d = plain.rms(d, 1e-3) * g1.double() + plain.rms(d2, 1e-3) * g2.double()
            v = x.double() + plain.rms(d, 1e-5) * post.double()
            want = plain.rms(v, 1e-4) * gain.double()
            extra = dict(other=dev(y2).to(dt), gains=(dev(g1), dev(g2)), eps_in=1e-3) if pair else {}
            bd = tuple(None if b is None else dev(b) for b in biases)
            xs, out = dev(x).clone(), torch.empty((T, n), dtype=dt, device=DEV)
            ops.post_norm_add(xs, dev(y1).to(dt), dev(post), 1e-5, dev(gain), 1e-4, out, biases=bd, **extra)
            assert (xs.cpu().double() - v).abs().max() <= 2e-5 * float(v.abs().max())
            assert (out.float().cpu() - want).abs().max() <= tol * float(want.abs().max())
            rows = torch.tensor([T - 1, 0], dtype=I32, device=DEV)
            xs, out = dev(x).clone(), torch.empty((2, n), dtype=dt, device=DEV)
            ops.post_norm_add(xs, dev(y1).to(dt), dev(post), 1e-5, dev(gain), 1e-4, out, rows=rows, update_x=False, biases=bd, **extra)
            assert torch.equal(xs.cpu(), x) and (out.float().cpu() - want[[T - 1, 0]]).abs().max() <= tol * float(want.abs().max())
        xs = dev(x).clone()
        ops.post_norm_add(xs, dev(y1).to(dt), dev(post), 1e-5)  # the sum alone
        v = x.double() + plain.rms(y1.double(), 1e-5) * post.double()
        assert (xs.cpu().double() - v).abs().max() <= 2e-5 * float(v.abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_polynomial_of_normed_powers_alone(dtype):
    from atomserve_amd.kernels import ops
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import PolyNormMLPSpec

    gen = torch.Generator().manual_seed(8)
    coef = torch.tensor([0.8, -0.6, 1.2, 0.3])
    for T, n in ((5, 50), (1, 3), (700, 384), (9, 4096), (4, 12288), (2, 16387)):
        z = bf(torch.randn(T, n, generator=gen) * 4)
        want = plain.poly_norm(z.double(), coef, 1e-2)
        out = torch.empty((T, n), dtype=DTYPES[dtype], device=DEV)
        ops.poly_norm(z.to(DEV).to(DTYPES[dtype]), coef.to(DEV), 1e-2, out)
        assert (out.float().cpu() - want).abs().max() <= (1e-5 if dtype == "float32" else 1e-2) * float(want.abs().max()), (T, n)
    for hidden, ff in ((64, 80), (90, 50), (256, 768)):
        w = {"x.up": bf(torch.randn(ff, hidden, generator=gen) * 0.3), "x.down": bf(torch.randn(hidden, ff, generator=gen) * 0.3), "x.act": bf(coef)}
        part = give(build("feed_forward", PolyNormMLPSpec("poly_norm_mlp", hidden, ff, 1e-5), env_for(dtype)),
                    {"up.weight": w["x.up"], "down.weight": w["x.down"], "act": w["x.act"]}, dtype)  # fmt: skip
        for T in (1, 7, 40, 130):
            h = bf(torch.randn(T, hidden, generator=gen))
            want = plain.poly_mlp(h.double(), {k: v.double() for k, v in w.items()}, "x.", 1e-5, False)
            got = part.forward(h.to(DEV).to(DTYPES[dtype]), None).float().cpu()
            assert (got - want).abs().max() <= (3e-5 if dtype == "float32" else 4e-2) * float(want.abs().max()), (hidden, T)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_difference_of_two_maps_alone(dtype):
    from atomserve_amd.kernels import ops

    gen = torch.Generator().manual_seed(6)
    for T, H, E, Dp, off in ((5, 3, 14, 16, 0), (9, 4, 64, 64, 8), (2, 2, 128, 160, 4), (3, 1, 264, 272, 3), (1, 2, 500, 500, 0)):
        heads = bf(torch.randn(T, 2 * H, Dp, generator=gen))
        heads[:, 1::2] = bf(heads[:, 0::2] + 0.1 * heads[:, 1::2])  # maps that nearly cancel
        want = plain.differential_combine(heads[:, 0::2, :E].double(), heads[:, 1::2, :E].double(), 0.9, 0.2, 1e-5)
        out = torch.full((T, off + H * E + 4), 5.0, dtype=DTYPES[dtype], device=DEV)
        for heads_dtype in {DTYPES[dtype], torch.float32}:
            out[:, off : off + H * E] = float("nan")
            ops.map_difference(heads.to(DEV).to(heads_dtype), E, 0.9, 1e-5, 0.8, out, off)
        got = out.float().cpu()
        assert (got[:, off : off + H * E].view(T, H, E) - want).abs().max() <= (2e-5 if dtype == "float32" else 1e-2) * float(want.abs().max())
        assert bool((got[:, :off] == 5.0).all()) and bool((got[:, off + H * E :] == 5.0).all())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(6, 2, 2, 40, 24), (4, 0, 4, 24, 8), (2, 3, 4, 16, 16), (12, 1, 3, 264, 96), (1, 1, 1, 32, 8), (70, 10, 6, 96, 16)])
def test_corrected_choice_and_identity_experts(sizes, dtype):
    """Chosen by the corrected scores, weighed by the scores alone, identity experts returning the input; also with more
    chosen than there are experts with matrices; a token alone gives bit for bit what it gives in company (32-bit)."""
    from atomserve_amd.kernels import ops
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import GatedRoutedExpertsSpec

    experts, same, top, hidden, ff = sizes
    gen = torch.Generator().manual_seed(sum(sizes))
    outputs = experts + same
    W = {"x.router": bf(torch.randn(outputs, hidden, generator=gen) * 0.3), "x.correction": bf(torch.randn(outputs, generator=gen) * 0.3)}
    for e in range(experts):
        W[f"x.e{e}.gate"], W[f"x.e{e}.up"] = bf(torch.randn(ff, hidden, generator=gen) * 0.3), bf(torch.randn(ff, hidden, generator=gen) * 0.3)
        W[f"x.e{e}.down"] = bf(torch.randn(hidden, ff, generator=gen) * 0.3)
    raw = {"expert": {"ff": ff}, "router": {"experts": experts, "top": top, "identity": same}}
    T = 70
    h = bf(torch.randn(T, hidden, generator=gen))
    ref = plain.experts(h.double(), {k: v.double() for k, v in W.items()}, "x.", raw, False).float()
    if top < outputs:
        plain_choice = plain.experts(h.double(), {k: v.double() * (0 if k == "x.correction" else 1) for k, v in W.items()}, "x.", raw, False).float()
        assert (plain_choice - ref).abs().max() > 1e-3, "the corrections do not matter in this test"
    spec = GatedRoutedExpertsSpec("gated_routed_experts", hidden, ff, experts, top, "silu", 0.0, score="softmax", router_bias=False,
                                  correction=True, identity=same)  # fmt: skip
    part = build("feed_forward", spec, env_for(dtype))
    t = {"router.weight": W["x.router"], "correction": W["x.correction"]}
    for name in ("gate", "up", "down"):
        t[name + ".weight"] = torch.stack([W[f"x.e{e}.{name}"] for e in range(experts)])
    give(part, t, dtype)
    hd = h.to(DEV).to(DTYPES[dtype])
    got = part.forward(hd, None).float().cpu()
    rows = (got - ref).abs().max(-1).values
    tol = (3e-5 if dtype == "float32" else 4e-2) * max(1.0, float(ref.abs().max()))
    assert (rows <= tol).sum() >= T - 2, "a token whose scores lie within rounding of each other may take another expert"
    if dtype == "float32":
        for t_ in (0, 17, 69):
            assert torch.equal(part.forward(hd[t_ : t_ + 1].contiguous(), None).float().cpu()[0], got[t_])
    # equal corrected scores: the lower number
    route = ops.moe_route_scores(torch.zeros(2, 16, device=DEV, dtype=DTYPES[dtype]), torch.zeros(6, 16, device=DEV, dtype=DTYPES[dtype]), 2,
                                 "softmax", correction=torch.tensor([0.0, 1.0, 0.0, 0.0, 0.0, 0.0], device=DEV), identity=2)  # fmt: skip
    assert route.pair_expert.cpu().tolist() == [1, 0, 1, 0]
    assert torch.allclose(route.pair_weight.cpu(), torch.full((4,), 1 / 6))


def test_models_of_these_shapes_say_they_replay():
    for case in sorted(CASES):
        assert build_model(CASES[case], random_weights(CASES[case], seed=1), "bfloat16").capturable
