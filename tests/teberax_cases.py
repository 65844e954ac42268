"""Small Teberax configurations for the tests, and random weights under the checkpoint's names.

The configurations differ from one another in every size and option: differential attentions with 1 to 4 query heads to
a kv head, two keys together narrower and wider than a value, windows of 1 to 64 tokens that keep none, some or more first
tokens than they are long, none at all, and layers that read an earlier layer's keys through a narrower, a wider and no
window; sink attentions with rotations over whole heads and parts of them, slowed or not, capped scores or not; linear
attentions with decays of rank 1 to 9 and keys narrower and wider than values; latents with and without a turned part and a
window; feed-forwards dense, routed with none, one and more identity experts, and absent; sizes that are multiples of
nothing, sizes the matrix-core kernels take, and heads wider than any of them."""

import torch


def _attention(heads, kv_heads, dim, vdim, scale, diff, mask=None, kv_from=None):
    raw = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "diff": diff}
    if mask:
        raw["mask"] = {"size": mask[0], "keep_first": mask[1]}
    if kv_from is not None:
        raw["kv_from"] = kv_from
    return {"type": "attention", "mixer": raw}


def _rot(dims, base, factor=None):
    raw = {"dims": dims, "base": base}
    if factor:
        raw["scaling"] = {"factor": factor}
    return raw


def _parallel(heads, kv_heads, dim, vdim, scale, rot, softcap, right):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale, "rot": rot}
    if softcap:
        left["softcap"] = softcap
    rh, rd, rv, tau, rank = right
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": rh, "dim": rd, "vdim": rv, "tau": tau, "rank": rank}}}


def _latent(heads, dim, rot_dim, vdim, kv_rank, scale, base=None, size=None):
    raw = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "scale": scale}
    if rot_dim:
        raw["rot"] = _rot(rot_dim, base)
    if size:
        raw["mask"] = {"size": size}
    return {"type": "latent_attention", "mixer": raw}


def _with(layer, mlp):
    return dict(layer, mlp=mlp)


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(ff, experts, top, identity=None):
    router = {"experts": experts, "top": top}
    if identity is not None:
        router["identity"] = identity
    return {"kind": "moe", "expert": {"ff": ff}, "router": router}


CASES = {
    # every mixer and feed-forward; a layer whose keys two later layers read, one through a narrower window that keeps more
    # first tokens, one through a wider window
    "all_kinds": {
        "architecture": "Teberax", "vocab": 200, "width": 96, "norm": {"eps": 1e-5}, "logit_softcap": 8.0,
        "layers": [
            _with(_attention(4, 2, 16, 24, 0.3, 0.25, (13, 3)), _dense(80)),
            _with(_parallel(4, 2, 24, 16, 0.25, _rot(10, 10000.0, 3.0), 6.0, (3, 16, 8, 8.0, 5)), _moe(24, 6, 2, 2)),
            _with(_latent(3, 16, 8, 24, 40, 0.22, 5000.0, 17), _moe(16, 4, 3, 1)),
            _with(_attention(4, 2, 16, 24, 0.27, 0.4, (7, 9), kv_from=0), None),
            _with(_attention(4, 2, 16, 24, 0.33, 0.1, (30, 2), kv_from=0), _moe(24, 5, 2)),
        ],
    },
    # sizes that are multiples of nothing; no masks, caps or scaling; a reader without a window of a windowed layer
    "odd_sizes": {
        "architecture": "Teberax", "vocab": 203, "width": 90, "norm": {"eps": 1e-6},
        "layers": [
            _with(_latent(5, 10, 6, 14, 22, 0.3, 700.0), _moe(18, 3, 4, 2)),
            _with(_attention(3, 3, 5, 14, 0.4, 0.6, (1, 2)), _moe(10, 7, 1)),
            _with(_parallel(3, 1, 11, 7, 0.35, _rot(6, 500.0), None, (2, 6, 13, 1.0, 1)), None),
            _with(_attention(3, 3, 5, 14, 0.35, 0.2, None, kv_from=1), _dense(50)),
        ],
    },
    # sizes the matrix-core kernels take, windows at the edges of their steps, more first tokens than the window is long
    "matrix_cores": {
        "architecture": "Teberax", "vocab": 320, "width": 128, "norm": {"eps": 1e-5}, "logit_softcap": 20.0,
        "layers": [
            _with(_parallel(4, 1, 64, 64, 0.125, _rot(64, 300000.0, 2.0), 12.0, (2, 64, 32, 16.0, 8)), _dense(192)),
            _with(_attention(4, 2, 32, 64, 0.18, 0.3, (32, 40)), _moe(64, 8, 2, 2)),
            _with(_latent(4, 32, 32, 32, 96, 0.12, 50000.0, 33), _moe(32, 4, 2, 1)),
            _with(_attention(2, 2, 64, 128, 0.12, 0.5, (64, 5)), _moe(32, 6, 2, 3)),
        ],
    },
    # heads wider than the paged kernels take; keys wider than the chunked scan takes; a latent without a turned part
    "wide": {
        "architecture": "Teberax", "vocab": 128, "width": 64, "norm": {"eps": 1e-5}, "logit_softcap": 5.0,
        "layers": [
            _with(_attention(4, 2, 136, 40, 0.08, 0.3, (11, 4)), _dense(64)),
            _with(_parallel(2, 2, 24, 264, 0.2, _rot(24, 2000.0), 4.0, (2, 136, 12, 4.0, 9)), _moe(16, 3, 2, 1)),
            _with(_latent(2, 24, 0, 16, 264, 0.2, size=9), None),
            _with(_latent(3, 20, 12, 8, 250, 0.2, 9000.0), _moe(8, 2, 2, 2)),
        ],
    },
}  # fmt: skip


def random_weights(raw: dict, seed: int, std: float = 0.15) -> dict:
    """Tensors under the checkpoint's names, float32 holding bfloat16 values (exact in both precisions)."""
    g = torch.Generator().manual_seed(seed)
    h, vocab = raw["width"], raw["vocab"]

    def mat(*shape, s=std):
        return (torch.randn(*shape, generator=g) * s).bfloat16().float()

    def gain(*shape):
        return (1.0 + torch.randn(shape, generator=g) * 0.2).bfloat16().float()

    w = {"embed": mat(vocab, h, s=1.0), "embed.norm": gain(), "final.norm": gain() * 2, "head": mat(vocab, h, s=0.3)}
    for i, layer in enumerate(raw["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp is not None else ()):
            w[p + name] = gain()
        x = p + "mix."
        if layer["type"] == "attention":
            H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w[x + "q"] = mat(H * 2 * D, h, s=0.3)
            if m.get("kv_from") is None:
                w[x + "k"], w[x + "v"] = mat(G * 2 * D, h, s=0.3), mat(G * E, h, s=0.3)
            for name in ("lq1", "lk1", "lq2", "lk2"):
                w[x + name] = mat(D, s=0.8 * D**-0.25)
            w[x + "o"] = mat(h, H * E)
        elif layer["type"] == "parallel":
            a, r = m["left"], m["right"]
            for name, rows, cols in (("q", a["heads"] * a["dim"], h), ("k", a["kv_heads"] * a["dim"], h),
                                     ("v", a["kv_heads"] * a["vdim"], h), ("o", h, a["heads"] * a["vdim"])):  # fmt: skip
                w[x + "left." + name], w[x + "left." + name + ".b"] = mat(rows, cols, s=0.25), mat(rows, s=0.3)
            H, D, E = r["heads"], r["dim"], r["vdim"]
            y = x + "right."
            w[y + "q"], w[y + "k"], w[y + "v"] = mat(H * D, h, s=0.3), mat(H * D, h, s=0.3), mat(H * E, h, s=0.3)
            w[y + "g"], w[y + "o"], w[y + "norm"] = mat(H * E, h), mat(h, H * E), gain(E)
            w[y + "a1"], w[y + "a2"] = mat(r["rank"], h, s=0.3), mat(H * D, r["rank"], s=0.6)
            w[y + "a2.b"] = (torch.randn(H * D, generator=g) * 1.5).bfloat16().float()
            w[x + "left.out"], w[x + "right.out"] = gain(h), gain(h)
        else:
            H, D, R, E, C = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
            w[x + "q"], w[x + "dkv"], w[x + "dkv.norm"] = mat(H * (D + R), h, s=0.3), mat(C + R, h, s=0.3), gain(C)
            w[x + "uk"], w[x + "uv"], w[x + "o"] = mat(H * D, C), mat(H * E, C), mat(h, H * E)
        if mlp is None:
            continue
        x = p + "mlp."
        if mlp["kind"] == "dense":
            w[x + "up"], w[x + "down"] = mat(mlp["ff"], h, s=0.3), mat(h, mlp["ff"])
            w[x + "act"] = (torch.randn(4, generator=g) * 0.5 + torch.tensor([1.0, -0.5, 0.7, 0.2])).bfloat16().float()
        else:
            r, ff = mlp["router"], mlp["expert"]["ff"]
            for e in range(r["experts"]):
                w[f"{x}e{e}.gate"], w[f"{x}e{e}.up"], w[f"{x}e{e}.down"] = mat(ff, h, s=0.3), mat(ff, h, s=0.3), mat(h, ff)
            outputs = r["experts"] + r.get("identity", 0)
            w[x + "router"], w[x + "correction"] = mat(outputs, h, s=0.3), mat(outputs, s=0.2)
    return w
