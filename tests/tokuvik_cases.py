"""Small Tokuvik configurations for the tests, and random weights under the checkpoint's names.

The configurations differ from one another in every size and option: attentions with 1 to 5 query heads to a kv head, keys
narrower and wider than values, chunks of 1 to 64 tokens and none, layers that read an earlier layer's keys through shorter,
longer and no chunks; latents narrower and wider than a head and than the paged kernels take, query latents of 7 to 72;
state spaces with 1 to 3 groups, states narrower and wider than values and than the chunked kernel takes, 1 to 5 taps,
norms in groups that are not those of B and C; layers without a feed-forward; token inputs 9 to 24 wide and none; sizes that
are multiples of nothing and sizes the matrix-core kernels take."""

import torch


def _attention(heads, kv_heads, dim, vdim, scale, size=None, kv_from=None):
    raw = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size:
        raw["mask"] = {"size": size}
    if kv_from is not None:
        raw["kv_from"] = kv_from
    return {"type": "attention", "mixer": raw}


def _latent(heads, dim, vdim, q_rank, kv_rank, scale):
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                                  "scale": scale}}  # fmt: skip


def _mamba(heads, vdim, state, groups, conv, norm_groups):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                                        "norm_groups": norm_groups}}  # fmt: skip


def _with(layer, ff):
    return dict(layer, mlp={"kind": "dense", "ff": ff} if ff else None)


CASES = {
    # every mixer; a layer whose keys two later layers read, one through shorter chunks and one through longer ones
    "all_kinds": {
        "architecture": "Tokuvik", "vocab": 200, "width": 96, "norm": {"eps": 1e-5}, "token_side": {"dim": 12},
        "layers": [
            _with(_attention(4, 2, 16, 24, 0.3, 13), 80),
            _with(_mamba(6, 16, 24, 3, 4, 2), 72),
            _with(_latent(3, 16, 24, 40, 48, 0.25), 64),
            _with(_attention(4, 2, 16, 24, 0.27, 7, kv_from=0), 0),
            _with(_attention(4, 2, 16, 24, 0.33, 30, kv_from=0), 56),
        ],
    },
    # sizes that are multiples of nothing; a norm in one group; a reader without chunks of a layer with chunks
    "odd_sizes": {
        "architecture": "Tokuvik", "vocab": 203, "width": 90, "norm": {"eps": 2e-5}, "token_side": {"dim": 9},
        "layers": [
            _with(_mamba(3, 7, 5, 1, 3, 3), 50),
            _with(_attention(5, 1, 11, 6, 0.4, 1), 0),
            _with(_latent(5, 10, 14, 7, 22, 0.3), 34),
            _with(_mamba(2, 9, 11, 2, 1, 1), 0),
            _with(_attention(5, 1, 11, 6, 0.35, None, kv_from=1), 50),
        ],
    },
    # sizes the matrix-core kernels take, chunks at the edges of their steps
    "matrix_cores": {
        "architecture": "Tokuvik", "vocab": 320, "width": 128, "norm": {"eps": 1e-5}, "token_side": {"dim": 24},
        "layers": [
            _with(_latent(4, 64, 32, 72, 96, 0.15), 192),
            _with(_mamba(8, 32, 64, 2, 4, 4), 192),
            _with(_attention(4, 1, 64, 64, 0.2, 64), 192),
            _with(_mamba(2, 64, 128, 1, 5, 1), 0),
            _with(_attention(8, 2, 32, 64, 0.25, 33), 160),
        ],
    },
    # heads and a latent wider than the paged kernels take, a state wider than the chunked kernel takes; no token inputs
    "wide": {
        "architecture": "Tokuvik", "vocab": 128, "width": 64, "norm": {"eps": 1e-5},
        "layers": [
            _with(_latent(2, 24, 16, 20, 264, 0.2), 64),
            _with(_mamba(2, 12, 136, 1, 2, 2), 40),
            _with(_attention(2, 2, 264, 40, 0.1, 11), 0),
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

    side = raw.get("token_side")
    w = {"embed": mat(vocab, h, s=0.5), "final.norm": gain(h)}
    if side:
        w["side.embed"] = mat(vocab, side["dim"] * len(raw["layers"]), s=1.0)
    for i, layer in enumerate(raw["layers"]):
        p, m, mlp = f"l{i}.", layer["mixer"], layer["mlp"]
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if mlp is not None else ()):
            w[p + name] = gain(h)
        x = p + "mix."
        if layer["type"] == "attention":
            H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            w[x + "q"], w[x + "q.norm"] = mat(H * D, h, s=0.3), gain(H * D) * 2
            if m.get("kv_from") is None:
                w[x + "k"], w[x + "k.norm"], w[x + "v"] = mat(G * D, h, s=0.3), gain(G * D) * 2, mat(G * E, h, s=0.3)
            w[x + "g"], w[x + "o"] = mat(H, h, s=0.3), mat(h, H * E)
        elif layer["type"] == "latent_attention":
            H, D, E, Q, C = m["heads"], m["dim"], m["vdim"], m["q_rank"], m["kv_rank"]
            w[x + "dq"], w[x + "dq.norm"], w[x + "uq"] = mat(Q, h, s=0.3), gain(Q), mat(H * D, Q, s=0.4)
            w[x + "dkv"], w[x + "dkv.norm"] = mat(C, h, s=0.3), gain(C)
            w[x + "uk"], w[x + "uv"], w[x + "sink"] = mat(H * D, C), mat(H * E, C), mat(H, s=2.0)
            w[x + "g"], w[x + "o"] = mat(H * E, h), mat(h, H * E)
        else:
            H, E, N, G = m["heads"], m["vdim"], m["state"], m["groups"]
            inner, channels = H * E, H * E + 2 * G * N
            w[x + "in"] = mat(inner + channels + H, h, s=0.3)
            w[x + "conv"], w[x + "conv.b"] = mat(channels, m["conv"], s=0.5), mat(channels, s=0.3)
            w[x + "dt_bias"], w[x + "A_log"] = mat(H, s=1.0) - 2.0, mat(H, s=1.0)
            w[x + "D"], w[x + "norm"], w[x + "o"] = gain(H), gain(inner), mat(h, inner)
        if mlp is not None:
            ff = mlp["ff"]
            w[p + "mlp.gate"], w[p + "mlp.up"], w[p + "mlp.down"] = mat(ff, h, s=0.3), mat(ff, h, s=0.3), mat(h, ff)
        if side:
            w[p + "side.gate"], w[p + "side.proj"], w[p + "side.norm"] = mat(side["dim"], h, s=0.3), mat(h, side["dim"], s=0.4), gain(h)
    return {k: v.bfloat16().float() for k, v in w.items()}
