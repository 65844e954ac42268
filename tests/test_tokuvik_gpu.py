"""Tokuvik on the GPU against the plain implementation (tests/plain_tokuvik.py): each mechanism alone, and whole models of
several shapes stepped whole, token by token, in portions down to two tokens, in mixed batches with pages and state slots
used again, and through the engine's scheduler.  Configurations and weights are made here; where random weights would hide a
fault (a far key among hundreds, a chunk's edge, a sink, a lost state) the inputs are made so that it shows."""

import json
import os

import pytest
import torch

from tests import plain_tokuvik as plain
from tests import replay_cases as rc
from tests.test_teberax_gpu import Against, bf, close, env_for, give, paged, run_mixers
from tests.tokuvik_cases import CASES, random_weights

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
I32 = torch.int32
F = torch.float64


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
    requests = {"a": rc.random_ids(vocab, 231, 1), "b": rc.random_ids(vocab, 37, 2), "c": rc.random_ids(vocab, 2, 3),
                "d": rc.random_ids(vocab, 1, 4), "e": rc.random_ids(vocab, 50, 5)}  # fmt: skip
    refs = {}
    replay = make_replay(raw, weights, dtype, max_tokens=4 * 256)
    manager = replay.manager
    free_pages = manager.num_free
    ways = [(rid + " whole", rc.whole(rid, ids)) for rid, ids in requests.items()]
    ways.append(("a decoded", rc.prefill_then_decode("a", requests["a"], tail=30)))
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
    """A short prompt and 150 tokens decoded one by one (captured steps) over pages of 8 tokens, past many chunks; a
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
    """The replay tool's own main on a model folder written here: config.json names the architecture."""
    import io

    import numpy as np
    from safetensors.torch import save_file

    from atomserve_amd.engine import replay

    raw = CASES["odd_sizes"]
    weights = random_weights(raw, seed=17)
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
    ref = plain.logits(raw, weights, ids)
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


def settled(delta):
    """What a pending output adds to the stream, in float64."""
    y, norm = delta.y.double(), delta.norm
    return (plain.layer_norm if norm.spec.kind == "layernorm" else plain.rms_norm)(y, norm.gain_f32, norm.spec.eps)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("case", sorted(CASES))
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
            assert float(rows.max()) <= 3e-5 * float(ref.abs().max()), f"layer {i}: {float(rows.max()):.3e} of {float(ref.abs().max()):.3e}"
            continue
        noise = (rounded[i] - ref).abs().max(-1).values
        assert float(rows.median()) <= 2.0 * float(noise.median()) and float(rows.quantile(0.9)) <= 2.0 * float(noise.quantile(0.9)), (
            f"layer {i}: rows' median {float(rows.median()):.3e} and ninth decile {float(rows.quantile(0.9)):.3e}; the plain "
            f"model's {float(noise.median()):.3e} and {float(noise.quantile(0.9)):.3e}")  # fmt: skip


# ---- chunks and sinks: the attention kernels alone --------------------------------------------------------------------

CHUNKS = [(0, True), (1, False), (2, True), (31, False), (32, True), (33, False), (64, True), (65, True), (100, False), (250, True), (500, True)]


@pytest.mark.parametrize("sight", CHUNKS)
@pytest.mark.parametrize("sizes", [(4, 2, 64, 16), (2, 1, 96, 16), (20, 1, 32, 32), (3, 3, 40, 8), (2, 2, 272, 16)])
def test_attention_kernels_over_chunks_with_sinks(sizes, sight):
    """Chunks and a sink per head in every attention kernel: single queries in 32 bits and on the matrix cores (several
    partitions and one, groups of more heads than a tile), prompts (both tilings, cut into pieces and whole, whole and behind a
    cached prefix), and heads of any width; some sinks take nearly everything, some nothing."""
    from atomserve_amd.kernels import ops

    H, G, D, bs = sizes
    chunk, with_sink = sight
    L = 331
    gen = torch.Generator().manual_seed(H * 1000 + D + chunk)
    q, k, v = torch.randn(L, H, D, generator=gen), torch.randn(L, G, D, generator=gen), torch.randn(L, G, D, generator=gen)
    q[:, H - 1] *= 3.0
    q, k, v = (t.bfloat16().float() for t in (q, k, v))
    sinks = torch.linspace(9.0, -30.0, H) if with_sink else None
    scale = 2.0 * D**-0.5
    want = plain.attention(q.double(), k.double(), v.double(), scale, chunk, sinks).float()
    how = dict(chunk=chunk, sink=sinks.to(DEV) if with_sink else False)
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

        out = torch.empty(L, H, D, dtype=dtype, device=DEV)
        ops.wide_attend(qd, kp, vp, pos, row, table, out, scale, L, 0, **how)
        check(out, "any width")
        if D > ops.SINGLE_QUERY_MAX_HEAD_DIM:
            continue
        for part in (None, 64, 32 * -(-(L + 64) // 32)):
            for generic in (False, True):
                out = torch.full((L, H, D), float("nan"), dtype=dtype, device=DEV)
                ops.attn_single_query(qd, kp, vp, None, pos, row, table, out, scale, 0, L, part, force_generic=generic, **how)
                check(out, f"single queries, partitions of {part}, general {generic}")
        if ops.attn_prefill_supported(dtype, D, bs):
            for first in (0, 77):
                tiles = [[t, min(64, L - t), 0, t] for t in range(first, L, 64)]
                for kind in (1, 2):
                    for pieces in (1, 3):
                        before, ops.PREFILL_PIECES = ops.PREFILL_PIECES, pieces
                        out = want.to(DEV).to(dtype).clone()
                        out[first:] = float("nan")
                        try:
                            ops.attn_prefill(qd, kp, vp, torch.tensor(tiles[::-1], dtype=I32, device=DEV), table, out, scale, 0, L, kind, **how)
                        finally:
                            ops.PREFILL_PIECES = before
                        check(out, f"prompt from {first}, {kind} query tiles, {pieces} pieces")
    assert checks >= 2


def test_chunks_and_windows_do_not_mix():
    from atomserve_amd.kernels import ops
    from atomserve_amd.kernels.lib import KernelError

    q = torch.zeros(1, 2, 32, device=DEV)
    pages = torch.zeros(2, 2, 16, 32, device=DEV)
    zero = torch.zeros(1, dtype=I32, device=DEV)
    args = (q, pages, pages.view(2, 2, 32, 16), None, zero, zero, zero.view(1, 1), torch.empty_like(q), 1.0)
    with pytest.raises(KernelError, match="chunk"):
        ops.attn_single_query(*args, 4, 1, chunk=4)
    with pytest.raises(KernelError, match="sinks"):
        ops.attn_single_query(*args, 0, 1, sink=torch.zeros(3, device=DEV))


# ---- each mechanism alone -------------------------------------------------------------------------------------


def chunked_weights(hidden, m, gen, std=0.3):
    def mat(*s):
        return bf(torch.randn(*s, generator=gen) * std)

    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    return {"q": mat(H * D, hidden), "k": mat(G * D, hidden), "v": mat(G * E, hidden), "g": mat(H, hidden), "o": mat(hidden, H * E),
            "q.norm": bf(2 + torch.randn(H * D, generator=gen) * 0.5), "k.norm": bf(1 + torch.randn(G * D, generator=gen) * 0.3)}  # fmt: skip


def bind_chunked(w, hidden, m, dtype, own=True, cache_window=None):
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import JoinedMixerSpec, SoftmaxCoreSpec

    core = SoftmaxCoreSpec("softmax_core", m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], whole_norm_eps=1e-5,
                           chunk=(m.get("mask") or {}).get("size", 0), head_gate=True, own_kv=own, cache_window=cache_window)  # fmt: skip
    part = build("mixer", JoinedMixerSpec("joined", hidden, (core,), (1.0,)), env_for(dtype))
    t = {"in.weight": torch.cat([w[k] for k in (("q", "k", "v", "g") if own else ("q", "g"))]), "out_t.weight": w["o"].t(),
         "c0.q_norm": w["q.norm"]}  # fmt: skip
    if own:
        t["c0.k_norm"] = w["k.norm"]
    return give(part, t, dtype)


def plain_chunked(h, w, m, kept=None, index=0, rounded=False):
    return plain.chunked_attention(h.double(), {"x." + k: v.double() for k, v in w.items()}, "x.", m, 1e-5, rounded,
                                   {} if kept is None else kept, index).float()  # fmt: skip


ATTENTIONS = [  # heads, kv heads, keys, values, chunk
    (4, 2, 16, 32, 13), (3, 3, 5, 14, 0), (8, 2, 32, 64, 32), (5, 1, 64, 40, 1), (2, 2, 24, 96, 20), (2, 1, 272, 24, 10), (6, 2, 128, 128, 100),
]  # fmt: skip


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", ATTENTIONS)
def test_chunked_attention_alone(shape, dtype):
    H, G, D, E, chunk = shape
    hidden, T = 64, 145
    gen = torch.Generator().manual_seed(H * 100 + D)
    m = {"heads": H, "kv_heads": G, "dim": D, "vdim": E, "scale": 0.6 * D**-0.5, "mask": {"size": chunk} if chunk else None}
    w = chunked_weights(hidden, m, gen)
    h = bf(torch.randn(T, hidden, generator=gen))
    ref, rounded = plain_chunked(h, w, m), plain_chunked(h, w, m, rounded=True)
    even = plain_chunked(h, dict(w, g=w["g"] * 0), m)
    assert (ref - even).abs().max() > 0.05 * ref.abs().max(), "the gates do not matter in this test"
    part = bind_chunked(w, hidden, m, dtype)
    for cuts in ([T], [1] * T, [19, 1, 2, 2, 1, 117, 3], [2, 143]):
        (got,) = run_mixers([part], [h], cuts, dtype, warm=9)
        close(got, ref, rounded, dtype, f"{shape} {cuts}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(6, 11, 3), (5, 0, 20), (0, 4, 9), (16, 48, 64)])
def test_layers_that_read_another_layers_keys(sizes, dtype):
    """One layer with keys and values of its own and two that read them with queries, gates and chunks of their own, longer
    and shorter: the pages keep what the widest reader sees, also when the tokens come one by one."""
    hidden, T = 48, 150
    gen = torch.Generator().manual_seed(3)
    base = {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 32}
    ms = [dict(base, scale=s, mask={"size": c} if c else None) for c, s in zip(sizes, (0.2, 0.25, 0.15))]
    ms[1]["kv_from"] = ms[2]["kv_from"] = 0
    ws = [chunked_weights(hidden, m, gen) for m in ms]
    hs = [bf(torch.randn(T, hidden, generator=gen)) for _ in ms]
    kept, kept_rounded = {}, {}
    refs = [plain_chunked(h, w, m, kept, i) for i, (h, w, m) in enumerate(zip(hs, ws, ms))]
    rounded = [plain_chunked(h, w, m, kept_rounded, i, rounded=True) for i, (h, w, m) in enumerate(zip(hs, ws, ms))]
    window = 0 if 0 in sizes else max(sizes)
    parts = [bind_chunked(w, hidden, m, dtype, own=i == 0, cache_window=window) for i, (w, m) in enumerate(zip(ws, ms))]
    for cuts in ([T], [1] * T, [17, 2, 1, 130], [2] * 75):
        got = run_mixers(parts, hs, cuts, dtype, block_size=4 if dtype == "float32" else 16, warm=5, reads={1: 0, 2: 0})
        for i, g in enumerate(got):
            close(g, refs[i], rounded[i], dtype, f"layer {i} {cuts[:4]}")


@pytest.mark.parametrize("dtype,block_size", [("float32", 8), ("bfloat16", 16), ("bfloat16", 64)])
@pytest.mark.parametrize("size", [40, 64, 0])
def test_keys_just_inside_and_just_outside_a_chunk(size, dtype, block_size):
    """One token's key stands out for every query and its value is large: outputs change by their own size where the token
    enters or leaves what a position sees.  The token stands first, last and in the middle of a chunk and of a page; its readers
    come in one prompt, in portions and token by token, up to the chunk's end and behind it (without chunks: hundreds of
    positions on)."""
    hidden, T = 32, 230
    m = {"heads": 4, "kv_heads": 2, "dim": 16, "vdim": 32, "scale": 1.0, "mask": {"size": size} if size else None}
    for mark in (0, 79, 80, block_size - 1, 95, 2 * block_size):
        gen = torch.Generator().manual_seed(500 + mark)
        w = chunked_weights(hidden, m, gen, std=0.2)
        direction = bf(torch.randn(w["k"].shape[0], generator=gen))
        w["k"] = w["k"] * 0.2
        w["k"][:, 0] = 0.4 * direction
        w["q"] = w["q"] * 0.2
        w["q"][:, 1] = torch.cat([0.4 * direction.view(2, -1)[g] for g in (0, 0, 1, 1)])
        w["q.norm"], w["k.norm"] = torch.full_like(w["q.norm"], 2.0), torch.ones_like(w["k.norm"])
        h = bf(torch.randn(T, hidden, generator=gen) * 0.3)
        h[:, 0], h[:, 1] = 0.0, 4.0  # every query asks, one key answers
        h[mark, 0] = 6.0
        h[mark, 2:] *= 6.0
        ref = plain_chunked(h, w, m)
        blind = h.clone()
        blind[mark, 0] = 0.0
        shows = (plain_chunked(blind, w, m) - ref).abs().amax(-1) > 0.1 * ref.abs().max()
        end = min(T, (mark // size + 1) * size if size else T)
        assert bool(shows[mark + 1 : end].all()) and not bool(shows[end:].any()) and not bool(shows[:mark].any())
        part = bind_chunked(w, hidden, m, dtype)
        rounded = plain_chunked(h, w, m, rounded=True)
        edge = min(end, T - 4)
        for cuts in ([T], [edge - 1, 1, 1, T - edge - 1], [edge - 3, 2, 2, 2, T - edge - 3], [mark + 1, 5] + [1] * (T - mark - 6), [64, 64, 64, 38]):
            (got,) = run_mixers([part], [h], [c for c in cuts if c > 0], dtype, block_size=block_size, warm=20)
            close(got, ref, rounded, dtype, f"mark {mark} {cuts[:4]}")


LATENTS = [  # heads, keys, values, query latent, latent
    (3, 16, 24, 40, 48), (5, 10, 14, 1, 22), (4, 32, 32, 64, 96), (6, 64, 64, 128, 128), (2, 24, 16, 9, 30), (17, 8, 8, 30, 12), (2, 20, 8, 20, 270),
]  # fmt: skip


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", LATENTS)
def test_latent_attention_with_sinks_alone(shape, dtype):
    """No turned part, a gate per coordinate, a sink per head (some large enough to take most of the softmax); one head's
    group larger than a tile, a latent wider than the paged kernels' heads."""
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import LatentAttentionSpec

    H, D, E, Q, C = shape
    hidden, T = 64, 145
    gen = torch.Generator().manual_seed(sum(shape))

    def mat(*s, sd=0.3):
        return bf(torch.randn(*s, generator=gen) * sd)

    w = {"dq": mat(Q, hidden), "dq.norm": bf(1 + mat(Q)), "uq": mat(H * D, Q), "dkv": mat(C, hidden), "dkv.norm": bf(1 + mat(C)),
         "uk": mat(H * D, C, sd=0.15), "uv": mat(H * E, C, sd=0.15), "sink": bf(torch.linspace(6.0, -4.0, H)), "g": mat(H * E, hidden),
         "o": mat(hidden, H * E)}  # fmt: skip
    m = {"heads": H, "dim": D, "vdim": E, "q_rank": Q, "kv_rank": C, "scale": 0.3}
    h = bf(torch.randn(T, hidden, generator=gen))

    def run_plain(weights, rounded=False):
        return plain.latent_attention(h.double(), {"x." + k: v.double() for k, v in weights.items()}, "x.", m, 1e-5, rounded).float()

    ref, rounded = run_plain(w), run_plain(w, True)
    assert (run_plain(dict(w, sink=w["sink"] * 0 - 50)) - ref).abs().max() > 0.05 * ref.abs().max(), "the sinks do not matter in this test"
    spec = LatentAttentionSpec("latent_attention", hidden, H, D, 0, E, Q, C, 0.3, 1e-5, None, head_sinks=True)
    part = build("mixer", spec, env_for(dtype))
    give(part, {"in.weight": torch.cat([w["dq"], w["dkv"], w["g"]]), "q_norm.weight": w["dq.norm"], "uq.weight": w["uq"],
                "kv_norm.weight": w["dkv.norm"], "uk.weight": w["uk"], "uv.weight": w["uv"], "sink": w["sink"], "o.weight": w["o"]}, dtype)  # fmt: skip
    for cuts in ([T], [1] * T, [19, 1, 2, 2, 1, 117, 3], [2, 143]):
        (got,) = run_mixers([part], [h], cuts, dtype, block_size=4 if dtype == "float32" else 16, warm=9)
        close(got, ref, rounded, dtype, f"{shape} {cuts}")


# ---- state spaces -------------------------------------------------------------------------------------------------------


def space_weights(hidden, m, gen):
    def mat(*s, sd=0.3):
        return bf(torch.randn(*s, generator=gen) * sd)

    H, E, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
    inner, channels = H * E, H * E + 2 * G * N
    return {"in": mat(inner + channels + H, hidden), "conv": mat(channels, m["conv"], sd=0.5), "conv.b": mat(channels), "dt_bias": mat(H, sd=1.0),
            "A_log": mat(H, sd=1.0), "D": mat(H, sd=1.0), "norm": bf(1 + mat(inner)), "o": mat(hidden, inner)}  # fmt: skip


def bind_space(w, hidden, m, dtype):
    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import ShortConvSpec, StateSpaceSpec

    spec = StateSpaceSpec("state_space", hidden, m["heads"], m["vdim"], m["state"], m["groups"], ShortConvSpec(m["conv"]), m["norm_groups"], 1e-5)
    names = {"in.weight": "in", "conv.weight": "conv", "conv.bias": "conv.b", "dt_bias": "dt_bias", "a_log": "A_log", "skip": "D",
             "out_norm.weight": "norm", "out.weight": "o"}  # fmt: skip
    return give(build("mixer", spec, env_for(dtype)), {to: w[name] for to, name in names.items()}, dtype)


def plain_space(h, w, m, rounded=False):
    return plain.state_space(h.double(), {"x." + k: v.double() for k, v in w.items()}, "x.", m, 1e-5, rounded).float()


SPACES = [  # heads, values, state, groups, taps, groups of the norm
    (6, 16, 24, 3, 4, 2), (3, 7, 5, 1, 3, 3), (8, 32, 64, 2, 4, 1), (4, 64, 128, 1, 2, 4), (2, 40, 96, 2, 1, 1), (5, 33, 20, 5, 8, 5), (2, 12, 200, 1, 4, 2),
]  # fmt: skip


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("shape", SPACES)
def test_state_space_mixer_alone(shape, dtype):
    m = dict(zip(("heads", "vdim", "state", "groups", "conv", "norm_groups"), shape))
    hidden, T = 64, 145
    gen = torch.Generator().manual_seed(sum(shape))
    w = space_weights(hidden, m, gen)
    h = bf(torch.randn(T, hidden, generator=gen))
    ref, rounded = plain_space(h, w, m), plain_space(h, w, m, True)
    part = bind_space(w, hidden, m, dtype)
    for cuts in ([T], [1] * T, [19, 1, 2, 2, 1, 117, 3], [33, 112], [2] * 72 + [1]):
        (got,) = run_mixers([part], [h], cuts, dtype, warm=9)
        close(got, ref, rounded, dtype, f"{shape} {cuts[:4]}")


def test_state_space_keeps_a_far_token():
    """With slow decays and one early token whose B answers a late token's C, the output hundreds of tokens later is that
    token's x: a state (or a segment's) that was lost or restarted on the way shows as a difference of the output's size."""
    m = {"heads": 2, "vdim": 16, "state": 32, "groups": 1, "conv": 3, "norm_groups": 1}
    hidden, T = 48, 700
    gen = torch.Generator().manual_seed(5)
    w = space_weights(hidden, m, gen)
    w["A_log"], w["dt_bias"] = torch.full_like(w["A_log"], -6.0), torch.full_like(w["dt_bias"], 0.5)
    w["conv.b"] *= 0
    w["D"] *= 0
    h = bf(torch.randn(T, hidden, generator=gen) * 0.02)
    h[3] = bf(torch.randn(hidden, generator=gen) * 4)
    h[T - 1] = h[3]
    ref = plain_space(h, w, m)
    forgot = plain_space(torch.cat([h[:3], h[4:]]), w, m)
    assert (forgot[-1] - ref[-1]).abs().max() > 0.1 * ref[-1].abs().max(), "the far token does not matter in this test"
    part = bind_space(w, hidden, m, "float32")
    for cuts in ([T], [350, 349, 1], [7] * 100, [T - 1, 1], [4, T - 4], [3, 1, T - 4], [230, 470]):
        (got,) = run_mixers([part], [h], cuts, "float32", warm=11)
        assert (got - ref).abs().max() <= 1e-4 * max(1.0, float(ref.abs().max())), cuts


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(3, 1, 64, 40), (4, 2, 128, 64), (1, 1, 24, 72), (6, 3, 10, 6), (8, 1, 36, 32), (2, 1, 200, 16), (2, 2, 128, 33)])
def test_the_ways_to_run_a_state_space(sizes, dtype):
    """Token by token, one token a row, in chunks and in segments of chunks, over several rows of one step, from states that
    another request left; steps from nearly nothing to so large that the past is forgotten at once."""
    from atomserve_amd.kernels import ops

    H, G, N, E = sizes
    dt_ = DTYPES[dtype]
    gen = torch.Generator().manual_seed(N + E)
    lens, starts, slots = [270, 1, 33, 128], [0, 5, 9, 0], [2, 0, 1, 3]
    T = sum(lens)
    xbc = torch.randn(T, H * E + 2 * G * N, generator=gen)
    xbc[:, H * E :] *= N**-0.25
    proj = bf(torch.randn(T, H + 3, generator=gen) * 3)
    proj[T // 3 : T // 3 + 2, 2] = 60.0
    dt_bias, a_log, skip = torch.randn(H, generator=gen), torch.randn(H, generator=gen), torch.randn(H, generator=gen)
    a_log[0] = 4.0
    a_log[-1] = -5.0
    state0 = torch.randn(5, H, N, E, generator=gen)
    x, B, C = (t.double() for t in torch.split(xbc, [H * E, G * N, G * N], dim=1))
    x, B, C = x.view(T, H, E), B.reshape(T, G, N), C.reshape(T, G, N)
    dt = plain.softplus(proj[:, 2 : 2 + H].double() + dt_bias.double())
    of = torch.arange(H) // (H // G)
    rate = torch.exp(a_log.double())

    def scan(at, n, S):
        out = []
        for t in range(at, at + n):
            S = torch.exp(-rate * dt[t]).view(H, 1, 1) * S + dt[t].view(H, 1, 1) * B[t][of].unsqueeze(2) * x[t].unsqueeze(1)
            out.append((S * C[t][of].unsqueeze(2)).sum(1) + skip.double().unsqueeze(1) * x[t])
        return torch.stack(out).view(n, H * E), S

    want, final, at, firsts = [], state0.double().clone(), 0, []
    for n, start, slot in zip(lens, starts, slots):
        y, final[slot] = scan(at, n, final[slot].clone() if start else torch.zeros(H, N, E, dtype=F))
        want.append(y)
        firsts.append(at)
        at += n
    want = torch.cat(want)
    ints = [torch.tensor(v, dtype=I32, device=DEV) for v in (firsts, lens, starts, slots)]
    tok_row = torch.cat([torch.full((n,), i, dtype=I32) for i, n in enumerate(lens)]).to(DEV)
    small = [t.to(DEV) for t in (dt_bias, a_log, skip)]
    tol = 3e-5
    for kernel, seg in (("scan", None), ("chunks", 0), ("chunks", 32), ("chunks", 96), ("chunks", 512), ("chunks", None)):
        if kernel == "chunks" and N > ops.STATE_SPACE_CHUNKS_MAX_STATE:
            continue
        for writes in (True, False):
            state, out = state0.clone().to(DEV), torch.full((T, H * E), float("nan"), device=DEV)
            ops.state_space(xbc.to(DEV), H, G, N, E, proj.to(DEV).to(dt_), 2, *small, state, (tok_row, *ints), out, writes=writes,
                            longest=max(lens), kernel=kernel, seg_len=seg)  # fmt: skip
            err = (out.cpu().double() - want).abs()
            assert err.max() <= tol * float(want.abs().max()), f"{kernel} {seg}: {float(err.max()):.3e} of {float(want.abs().max()):.3e} at {int(err.amax(1).argmax())}"
            kept = final if writes else state0.double()
            assert (state.cpu().double() - kept).abs().max() <= tol * float(kept.abs().max()), f"{kernel} {seg}: the state"
    ones = torch.ones(len(lens), dtype=I32, device=DEV)
    for kernel in ("scan", "step"):
        if kernel == "step" and (E % 4 or N > ops.STATE_SPACE_CHUNKS_MAX_STATE):
            continue
        state, out = state0.clone().to(DEV), torch.full((T, H * E), float("nan"), device=DEV)
        ops.state_space(xbc.to(DEV), H, G, N, E, proj.to(DEV).to(dt_), 2, *small, state, (tok_row, ints[0], ones, ints[2], ints[3]), out, kernel=kernel)
        assert (out.cpu().double()[firsts] - want[firsts]).abs().max() <= tol * float(want.abs().max()), kernel
        for f, start, slot in zip(firsts, starts, slots):
            _, S = scan(f, 1, state0[slot].double() if start else torch.zeros(H, N, E, dtype=F))
            assert (state.cpu()[slot].double() - S).abs().max() <= tol * float(S.abs().max()), f"{kernel}: the state"


# ---- norms, gates, placement ------------------------------------------------------------------------------------------------


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("n", [40, 90, 256, 1000, 4096, 5121, 16384])
def test_layer_norms_around_a_residual_sum(n, dtype):
    """Every pair of the norm after a sublayer and what follows (an RMS norm, a layer norm, nothing, the stream itself), rows
    whose mean is large beside their deviations, and the layer norm alone with and without a pending output."""
    from atomserve_amd.kernels import ops

    dt = DTYPES[dtype]
    tol = 3e-5 if dtype == "float32" else 1e-2
    for T in (3, 600) if n <= 4096 else (3,):
        gen = torch.Generator().manual_seed(n + T)
        x, y, other = torch.randn(T, n, generator=gen) * 3 + 5, bf(torch.randn(T, n, generator=gen) + 2), bf(torch.randn(T, n, generator=gen) * 9)
        post, gain, g1, g2 = (1 + 0.3 * torch.randn(n, generator=gen) for _ in range(4))
        dev = lambda t: t.to(DEV)  # noqa: E731
        rows = torch.tensor([T - 1, 0], dtype=I32, device=DEV)
        for centre_post in (False, True):
            for pair in (False, True):
                d = plain.rms_norm(y.double(), g1, 1e-3) + plain.rms_norm(other.double(), g2, 1e-3) if pair else y.double()
                v = x.double() + (plain.layer_norm if centre_post else plain.rms_norm)(d, post, 1e-5)
                extra = dict(other=dev(other).to(dt), gains=(dev(g1), dev(g2)), eps_in=1e-3) if pair else {}
                for centre in (False, True, None):
                    want = v if centre is None else (plain.layer_norm if centre else plain.rms_norm)(v, gain, 1e-4)
                    g = None if centre is None else dev(gain)
                    xs, out = dev(x).clone(), torch.empty((T, n), dtype=dt, device=DEV)
                    ops.post_norm_add(xs, dev(y).to(dt), dev(post), 1e-5, g, 1e-4, out, centre_post=centre_post, centre=bool(centre), **extra)
                    assert (xs.cpu().double() - v).abs().max() <= 2e-5 * float(v.abs().max())
                    assert (out.float().cpu() - want).abs().max() <= tol * float(want.abs().max())
                    xs, out = dev(x).clone(), torch.empty((2, n), dtype=dt, device=DEV)
                    ops.post_norm_add(xs, dev(y).to(dt), dev(post), 1e-5, g, 1e-4, out, rows=rows, update_x=False, centre_post=centre_post,
                                      centre=bool(centre), **extra)  # fmt: skip
                    assert torch.equal(xs.cpu(), x) and (out.float().cpu() - want[[T - 1, 0]]).abs().max() <= tol * float(want.abs().max())
        for delta in (None, y):
            v = x.double() + (0 if delta is None else delta.double())
            want = plain.layer_norm(v, gain, 1e-4)
            xs, out = dev(x).clone(), torch.empty((T, n), dtype=dt, device=DEV)
            d = None if delta is None else dev(delta).to(dt)
            ops.layer_norm(xs, dev(gain), 1e-4, out, d)
            assert (xs.cpu().double() - v).abs().max() <= 1e-6 * float(v.abs().max())
            assert (out.float().cpu() - want).abs().max() <= tol * float(want.abs().max())
            out = torch.empty((2, n), dtype=dt, device=DEV)
            ops.layer_norm(xs if delta is None else dev(x).clone(), dev(gain), 1e-4, out, d, rows, False)
            assert (out.float().cpu() - want[[T - 1, 0]]).abs().max() <= tol * float(want.abs().max())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_gated_norm_in_groups_alone(dtype):
    from atomserve_amd.kernels import ops

    gen = torch.Generator().manual_seed(4)
    for T, n, groups, off, ld in ((5, 48, 3, 0, 60), (1, 33, 3, 2, 40), (600, 1024, 4, 8, 2048), (9, 8192, 1, 0, 8200), (3, 10000, 2, 4, 20000), (2, 77, 1, 1, 90)):
        y, proj, gain = torch.randn(T, n, generator=gen) * 3, bf(torch.randn(T, ld, generator=gen) * 2), 1 + torch.randn(n, generator=gen) * 0.3
        z = proj[:, off : off + n].double()
        want = plain.grouped_rms_norm(y.double() * z * torch.sigmoid(z), gain, 1e-3, groups)
        out = torch.empty((T, n), dtype=DTYPES[dtype], device=DEV)
        ops.gated_group_norm(y.to(DEV), groups, 1e-3, gain.to(DEV), proj.to(DEV).to(DTYPES[dtype]), off, out)
        assert (out.float().cpu() - want).abs().max() <= (2e-5 if dtype == "float32" else 1e-2) * float(want.abs().max()), (T, n, groups)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_gates_per_head_and_per_coordinate(dtype):
    from atomserve_amd.kernels import ops

    gen = torch.Generator().manual_seed(7)
    for T, H, E, Dp, off in ((5, 3, 14, 16, 0), (300, 8, 64, 64, 8), (2, 5, 40, 96, 16), (1, 2, 264, 272, 3)):
        heads, gates = bf(torch.randn(T, H, Dp, generator=gen)), bf(torch.randn(T, 8 + H * E, generator=gen) * 3)
        for per_head in (True, False, None):
            out = torch.full((T, off + H * E + 8), 5.0, dtype=DTYPES[dtype], device=DEV)
            g = gates[:, 8 : 8 + H].double().unsqueeze(-1) if per_head else gates[:, 8:].double().view(T, H, E)
            want = 0.7 * heads[..., :E].double() * (1.0 if per_head is None else torch.sigmoid(g))
            ops.sigmoid_gate_heads(heads.to(DEV).to(DTYPES[dtype]), E, None if per_head is None else gates.to(DEV).to(DTYPES[dtype]), 8, 0.7, out, off,
                                   per_head=bool(per_head))  # fmt: skip
            got = out.float().cpu()
            assert (got[:, off : off + H * E].view(T, H, E) - want).abs().max() <= (1e-6 if dtype == "float32" else 1e-2) * float(want.abs().max())
            assert bool((got[:, :off] == 5.0).all()) and bool((got[:, off + H * E :] == 5.0).all())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(4, 2, 16, 24, 32), (5, 1, 11, 6, 16), (8, 2, 64, 64, 64), (3, 3, 32, 80, 96)])
def test_heads_normed_over_their_whole_projection_and_placed(sizes, dtype):
    """Few tokens and many (a pass of its own for the root mean squares), with keys to store and queries alone."""
    from atomserve_amd.kernels import ops

    H, G, D, E, Dp = sizes
    bs = 16
    dt = DTYPES[dtype]
    gen = torch.Generator().manual_seed(D)
    for T in (3, 40, 200):
        ld = H * D + G * (D + E)
        proj = bf(torch.randn(T, ld, generator=gen) * 2)
        qw, kw = 1 + torch.randn(H * D, generator=gen) * 0.3, 1 + torch.randn(G * D, generator=gen) * 0.3
        q = plain.rms_norm(proj[:, : H * D].double(), qw, 1e-3).view(T, H, D)
        k = plain.rms_norm(proj[:, H * D : H * D + G * D].double(), kw, 1e-3).view(T, G, D)
        v = proj[:, H * D + G * D :].double().view(T, G, E)
        pages = -(-T // bs) + 2
        slots = (torch.arange(T) + bs).to(I32)
        for own in (True, False):
            q_out = torch.full((T, H, Dp), 9.0, dtype=dt, device=DEV)
            kp, vp = torch.full((pages, G, bs, Dp), 9.0, dtype=dt, device=DEV), torch.full((pages, G, Dp, bs), 9.0, dtype=dt, device=DEV)
            src = proj if own else proj[:, : H * D].contiguous()
            ops.whole_norm_store(src.to(DEV).to(dt), 0, H * D, H * D + G * D, H, G, D, E, slots.to(DEV), q_out, kp, vp, store_kv=own,
                                 gains=(qw.to(DEV), kw.to(DEV) if own else None), eps=1e-3)  # fmt: skip
            tol = 2e-5 if dtype == "float32" else 2e-2
            got = q_out.float().cpu()
            assert (got[..., :D] - q).abs().max() <= tol * float(q.abs().max()) and bool((got[..., D:] == 0).all())
            keys = kp.float().cpu().permute(0, 2, 1, 3).reshape(-1, G, Dp)[bs : bs + T]
            values = vp.float().cpu().permute(0, 3, 1, 2).reshape(-1, G, Dp)[bs : bs + T]
            if not own:
                assert bool((keys == 9.0).all()) and bool((values == 9.0).all())
                continue
            assert (keys[..., :D] - k).abs().max() <= tol * float(k.abs().max()) and bool((keys[..., D:] == 0).all())
            assert (values[..., :E] - v).abs().max() <= tol * float(v.abs().max()) and bool((values[..., E:] == 0).all())


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("sizes", [(96, 12, 50), (90, 5, 33), (256, 64, 300), (64, 1, 7), (1032, 33, 40)])
def test_token_inputs_alone(sizes, dtype):
    from types import SimpleNamespace

    from atomserve_amd.parts.base import build
    from atomserve_amd.parts.plan import NormSpec, TokenInputSpec

    hidden, dim, vocab = sizes
    gen = torch.Generator().manual_seed(sum(sizes))
    W = {"l0.side.gate": bf(torch.randn(dim, hidden, generator=gen) * 0.3), "l0.side.proj": bf(torch.randn(hidden, dim, generator=gen)),
         "l0.side.norm": bf(1 + torch.randn(hidden, generator=gen) * 0.2)}  # fmt: skip
    table = bf(torch.randn(vocab, dim, generator=gen))
    part = build("token_input", TokenInputSpec("gated_table", hidden, dim, vocab, NormSpec("rmsnorm", hidden, 1e-5)), env_for(dtype))
    give(part, {"table": table, "gate.weight": W["l0.side.gate"], "proj.weight": W["l0.side.proj"]}, dtype)
    for T in (1, 2, 3, 7, 12, 16, 17, 40, 150):
        x, ids = bf(torch.randn(T, hidden, generator=gen) * 2), torch.randint(0, vocab, (T,), generator=gen)
        got = part.forward(x.to(DEV).to(DTYPES[dtype]), SimpleNamespace(token_ids=ids.to(I32).to(DEV))).float().cpu()
        args = ({k: v.double() for k, v in W.items()}, "l0.", table[ids].double(), 1e-5)
        ref, rounded = plain.token_input(x.double(), *args, False).float(), plain.token_input(x.double(), *args, True).float()
        close(plain.rms_norm(got.double(), W["l0.side.norm"], 1e-5).float(), ref, rounded, dtype, f"{sizes} {T}")


def test_models_of_these_shapes_say_they_replay():
    for case in sorted(CASES):
        assert build_model(CASES[case], random_weights(CASES[case], seed=1), "bfloat16").capturable
