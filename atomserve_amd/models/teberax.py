"""Teberax: configuration -> layer plan, and the checkpoint's tensor names.

Layers with a norm before and after each sublayer; every norm of a layer (and the embedding's and the last one) has one
number as its gain.  The mixer is a differential attention over a window that keeps the first tokens, which may read an
earlier layer's keys and values ("attention"), a rotary attention with biases, capped scores and a sink beside a gated
linear attention with a decay per key channel, each normed before the two are averaged ("parallel"), or an attention
through a cached latent over a window ("latent_attention"); the feed-forward is a dense one without a gate whose
activation is a polynomial of normed powers, or gated experts chosen by corrected softmax scores, some of which are the
input itself.  A layer that reads an earlier layer's keys is a run whose cache is that layer's run and that writes
nothing; the pages keep what the widest of their readers sees.
"""

from atomserve_amd.config.model_config import ConfigError, TeberaxConfig
from atomserve_amd.config.registry import Architecture, register_architecture
from atomserve_amd.parts.plan import (
    BlockSpec,
    ChannelDecaySpec,
    GatedRoutedExpertsSpec,
    JoinedMixerSpec,
    LatentAttentionSpec,
    ModelPlan,
    NeighbourRotarySpec,
    NormSpec,
    PolyNormMLPSpec,
    Run,
    SoftmaxCoreSpec,
)
from atomserve_amd.weights.loader import Stack, Take

MAX_POSITIONS = 1 << 30  # nothing in the design depends on a position's size


def _rotation(rot):
    return None if rot is None else NeighbourRotarySpec("rope_neighbours", rot.dims, rot.base, slower=rot.factor)


def _kept_for_readers(c: TeberaxConfig, i: int) -> tuple:
    """(window, first tokens) that the pages of attention layer i keep: the most that it or a layer that reads them sees."""
    masks = [layer.mixer.mask for j, layer in enumerate(c.layers)
             if layer.type == "attention" and (j == i or layer.mixer.kv_from == i)]  # fmt: skip
    window = 0 if any(m.size == 0 for m in masks) else max(m.size for m in masks)
    return window, max(m.keep_first for m in masks) if window else 0


def _mixer_spec(c: TeberaxConfig, i: int):
    layer = c.layers[i]
    m = layer.mixer
    if layer.type == "attention":
        window, keep = _kept_for_readers(c, i)
        core = SoftmaxCoreSpec("softmax_core", m.heads, m.kv_heads, m.dim, m.vdim, m.scale, window=m.mask.size,
                               keep_first=m.mask.keep_first, maps=2, difference=m.diff, difference_eps=c.norm_eps,
                               own_kv=m.kv_from < 0, cache_window=window, cache_keep_first=keep)  # fmt: skip
        return JoinedMixerSpec("joined", c.hidden_size, (core,), (1.0,))
    if layer.type == "parallel":
        a, r = m.left, m.right
        if r.rank < 1:
            raise ConfigError(f"layers[{i}]: the rank of the decays' two-step projection is unknown (no checkpoint names it and "
                              "the configuration has no rank)")  # fmt: skip
        left = SoftmaxCoreSpec("softmax_core", a.heads, a.kv_heads, a.dim, a.vdim, a.scale, bias=True, position=_rotation(a.rot),
                               window=a.mask.size, keep_first=a.mask.keep_first, softcap=a.softcap, sink=True)  # fmt: skip
        right = ChannelDecaySpec("channel_decay", r.heads, r.dim, r.vdim, r.rank, r.tau, c.norm_eps)
        return JoinedMixerSpec("joined", c.hidden_size, (left, right), (0.5, 0.5), out_norm_eps=c.norm_eps, out_bias=(True, False))
    return LatentAttentionSpec("latent_attention", c.hidden_size, m.heads, m.dim, m.rot_dim, m.vdim, 0, m.kv_rank, m.scale, c.norm_eps,
                               _rotation(m.rot), out_gate=False, window=m.mask.size, keep_first=m.mask.keep_first)  # fmt: skip


def build_plan(c: TeberaxConfig) -> ModelPlan:
    def norm():
        return NormSpec("rmsnorm", c.hidden_size, c.norm_eps, one_gain=True)

    layers, run = [], []
    for i, layer in enumerate(c.layers):
        f = layer.mlp
        if f is None:
            ffn = None
        elif f.kind == "dense":
            ffn = PolyNormMLPSpec("poly_norm_mlp", c.hidden_size, f.ff, c.norm_eps)
        else:
            ffn = GatedRoutedExpertsSpec("gated_routed_experts", c.hidden_size, f.ff, f.experts, f.top, "silu", 0.0, score="softmax",
                                         router_bias=False, correction=True, identity=f.identity)  # fmt: skip
        layers.append(BlockSpec("sandwich", _mixer_spec(c, i), norm(), ffn, None if ffn is None else norm(),
                                mixer_post_norm=norm(), ffn_post_norm=None if ffn is None else norm()))  # fmt: skip
        reads = layer.mixer.kv_from if layer.type == "attention" else -1
        run.append(Run(i, cache=reads, writes=False) if reads >= 0 else Run(i))
    return ModelPlan(
        vocab_size=c.vocab_size,
        hidden_size=c.hidden_size,
        layers=tuple(layers),
        run=tuple(run),
        final_norm=norm(),
        tied_head=False,
        max_positions=MAX_POSITIONS,
        logit_softcap=c.logit_softcap,
        embed_norm=norm(),
    )


def checkpoint_map(c: TeberaxConfig) -> dict:
    """Plan tensor name -> checkpoint names.  The projections that read a mixer's input are stacked into one matrix, in
    the order the parts expect their columns."""
    names = {"embed.weight": "embed", "embed_norm.weight": "embed.norm", "final_norm.weight": "final.norm", "head.weight": "head"}
    for i, layer in enumerate(c.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        names[dst + "mixer_norm.weight"] = src + "norm1"
        names[dst + "mixer_post_norm.weight"] = src + "norm1b"
        mix, to = src + "mix.", dst + "mixer."
        if layer.type == "attention":
            names[to + "in.weight"] = [mix + p for p in (("q", "k", "v") if layer.mixer.kv_from < 0 else ("q",))]
            names[to + "out_t.weight"] = Take(mix + "o", transpose=True)
            for p in ("lq1", "lk1", "lq2", "lk2"):
                names[to + "c0." + p] = mix + p
        elif layer.type == "parallel":
            left, right = mix + "left.", mix + "right."
            names[to + "in.weight"] = [left + p for p in ("q", "k", "v")] + [right + p for p in ("q", "k", "v", "g", "a1")]
            for p in ("q", "k", "v"):
                names[to + f"c0.{p}_bias"] = left + p + ".b"
            names[to + "c1.decay_up"] = right + "a2"
            names[to + "c1.decay_bias"] = right + "a2.b"
            names[to + "c1.out_norm"] = right + "norm"
            for n, half in enumerate((left, right)):
                names[to + f"out{n}.weight"] = half + "o"
                names[to + f"out{n}.norm"] = half + "out"
            names[to + "out0.bias"] = left + "o.b"
        else:
            names[to + "in.weight"] = [mix + "q", mix + "dkv"]
            names[to + "kv_norm.weight"] = mix + "dkv.norm"
            for p in ("uk", "uv", "o"):
                names[to + p + ".weight"] = mix + p
        f = layer.mlp
        if f is None:
            continue
        names[dst + "ffn_norm.weight"] = src + "norm2"
        names[dst + "ffn_post_norm.weight"] = src + "norm2b"
        mlp, to = src + "mlp.", dst + "ffn."
        if f.kind == "dense":
            for p in ("up", "down"):
                names[to + p + ".weight"] = mlp + p
            names[to + "act"] = mlp + "act"
        else:
            names[to + "router.weight"] = mlp + "router"
            names[to + "correction"] = mlp + "correction"
            for p in ("gate", "up", "down"):
                names[to + p + ".weight"] = Stack(tuple(Take(f"{mlp}e{e}.{p}") for e in range(f.experts)), new_axis=True)
    return names


def checkpoint_shapes(c: TeberaxConfig) -> dict:
    """Checkpoint name -> (shape, role), in the order in which random weights are drawn."""
    h = c.hidden_size
    shapes = {"embed": ((c.vocab_size, h), "matrix"), "embed.norm": ((), "vector")}
    for i, layer in enumerate(c.layers):
        p, m = f"l{i}.", layer.mixer
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if layer.mlp is not None else ()):
            shapes[p + name] = ((), "vector")
        x = p + "mix."
        if layer.type == "attention":
            shapes[x + "q"] = ((m.heads * 2 * m.dim, h), "matrix")
            if m.kv_from < 0:
                shapes[x + "k"] = ((m.kv_heads * 2 * m.dim, h), "matrix")
                shapes[x + "v"] = ((m.kv_heads * m.vdim, h), "matrix")
            for name in ("lq1", "lk1", "lq2", "lk2"):
                shapes[x + name] = ((m.dim,), "bias")
            shapes[x + "o"] = ((h, m.heads * m.vdim), "matrix")
        elif layer.type == "parallel":
            a, r = m.left, m.right
            for name, rows, cols in (("q", a.heads * a.dim, h), ("k", a.kv_heads * a.dim, h), ("v", a.kv_heads * a.vdim, h),
                                     ("o", h, a.heads * a.vdim)):  # fmt: skip
                shapes[x + "left." + name] = ((rows, cols), "matrix")
                shapes[x + "left." + name + ".b"] = ((rows,), "bias")
            y = x + "right."
            shapes[y + "q"] = ((r.heads * r.dim, h), "matrix")
            shapes[y + "k"] = ((r.heads * r.dim, h), "matrix")
            shapes[y + "v"] = ((r.heads * r.vdim, h), "matrix")
            shapes[y + "g"] = ((r.heads * r.vdim, h), "matrix")
            shapes[y + "o"] = ((h, r.heads * r.vdim), "matrix")
            shapes[y + "norm"] = ((r.vdim,), "vector")
            shapes[y + "a1"] = ((r.rank, h), "matrix")
            shapes[y + "a2"] = ((r.heads * r.dim, r.rank), "matrix")
            shapes[y + "a2.b"] = ((r.heads * r.dim,), "bias")
            shapes[x + "left.out"] = ((h,), "vector")
            shapes[x + "right.out"] = ((h,), "vector")
        else:
            shapes[x + "q"] = ((m.heads * (m.dim + m.rot_dim), h), "matrix")
            shapes[x + "dkv"] = ((m.kv_rank + m.rot_dim, h), "matrix")
            shapes[x + "dkv.norm"] = ((m.kv_rank,), "vector")
            shapes[x + "uk"] = ((m.heads * m.dim, m.kv_rank), "matrix")
            shapes[x + "uv"] = ((m.heads * m.vdim, m.kv_rank), "matrix")
            shapes[x + "o"] = ((h, m.heads * m.vdim), "matrix")
        f = layer.mlp
        if f is None:
            continue
        x = p + "mlp."
        if f.kind == "dense":
            shapes[x + "up"] = ((f.ff, h), "matrix")
            shapes[x + "down"] = ((h, f.ff), "matrix")
            shapes[x + "act"] = ((4,), "vector")
        else:
            for e in range(f.experts):
                shapes[f"{x}e{e}.gate"] = ((f.ff, h), "matrix")
                shapes[f"{x}e{e}.up"] = ((f.ff, h), "matrix")
                shapes[f"{x}e{e}.down"] = ((h, f.ff), "matrix")
            shapes[x + "router"] = ((f.experts + f.identity, h), "matrix")
            shapes[x + "correction"] = ((f.experts + f.identity,), "bias")
    shapes["final.norm"] = ((), "vector")
    shapes["head"] = ((c.vocab_size, h), "matrix")
    return shapes


TEBERAX = register_architecture(
    Architecture(
        name=TeberaxConfig.architecture,
        parse_config=TeberaxConfig.from_dict,
        build_plan=build_plan,
        checkpoint_map=checkpoint_map,
        checkpoint_shapes=checkpoint_shapes,
        complete=lambda config, shape_of: config.completed(shape_of),
    ),
    replace=True,
)
