"""Tokuvik: configuration -> layer plan, and the checkpoint's tensor names.

Layers with a layer norm before and after each sublayer that end with an input of the tokens' own: the stream gates the
layer's share of the row that a second table holds for the token, and the projected result enters the stream through an RMS
norm.  The mixer is a grouped-query attention without positions whose queries see their own chunk, with queries and keys normed
over their whole projections and a gate per head, on its own or an earlier layer's keys and values ("attention"), an attention
through a cached latent with a sink per head ("latent_attention"), or a state space per head ("mamba2"); the feed-forward is a
gated one or absent; the embedding table is also the head.  A layer that reads an earlier layer's keys is a run whose cache is
that layer's run and that writes nothing; the pages keep what the widest of their readers sees.
"""

from atomserve_amd.config.model_config import TokuvikConfig
from atomserve_amd.config.registry import Architecture, register_architecture
from atomserve_amd.parts.plan import (
    BlockSpec,
    GatedMLPSpec,
    JoinedMixerSpec,
    LatentAttentionSpec,
    ModelPlan,
    NormSpec,
    Run,
    ShortConvSpec,
    SoftmaxCoreSpec,
    StateSpaceSpec,
    TokenInputSpec,
)
from atomserve_amd.weights.loader import Take

MAX_POSITIONS = 1 << 30  # nothing in the design depends on a position's size


def _kept_for_readers(c: TokuvikConfig, i: int) -> int:
    """The window that the pages of attention layer i keep: as long as the longest chunk of it and of the layers that read
    them (0: everything)."""
    chunks = [layer.mixer.chunk for j, layer in enumerate(c.layers)
              if layer.type == "attention" and (j == i or layer.mixer.kv_from == i)]  # fmt: skip
    return 0 if 0 in chunks else max(chunks)


def _mixer_spec(c: TokuvikConfig, i: int):
    layer = c.layers[i]
    m = layer.mixer
    if layer.type == "attention":
        core = SoftmaxCoreSpec("softmax_core", m.heads, m.kv_heads, m.dim, m.vdim, m.scale, whole_norm_eps=c.norm_eps, chunk=m.chunk,
                               head_gate=True, own_kv=m.kv_from < 0, cache_window=_kept_for_readers(c, i))  # fmt: skip
        return JoinedMixerSpec("joined", c.hidden_size, (core,), (1.0,))
    if layer.type == "latent_attention":
        return LatentAttentionSpec("latent_attention", c.hidden_size, m.heads, m.dim, 0, m.vdim, m.q_rank, m.kv_rank, m.scale, c.norm_eps,
                                   None, head_sinks=True)  # fmt: skip
    return StateSpaceSpec("state_space", c.hidden_size, m.heads, m.vdim, m.state, m.groups, ShortConvSpec(m.conv), m.norm_groups, c.norm_eps)


def build_plan(c: TokuvikConfig) -> ModelPlan:
    def norm():
        return NormSpec("layernorm", c.hidden_size, c.norm_eps)

    side = None
    if c.side_dim:
        side = TokenInputSpec("gated_table", c.hidden_size, c.side_dim, c.vocab_size, NormSpec("rmsnorm", c.hidden_size, c.norm_eps))
    layers, run = [], []
    for i, layer in enumerate(c.layers):
        ffn = GatedMLPSpec("gated_mlp", c.hidden_size, layer.ff, "silu") if layer.ff else None
        layers.append(BlockSpec("sandwich", _mixer_spec(c, i), norm(), ffn, norm() if layer.ff else None, mixer_post_norm=norm(),
                                ffn_post_norm=norm() if layer.ff else None, token_input=side))  # fmt: skip
        reads = layer.mixer.kv_from if layer.type == "attention" else -1
        run.append(Run(i, cache=reads, writes=False) if reads >= 0 else Run(i))
    return ModelPlan(
        vocab_size=c.vocab_size,
        hidden_size=c.hidden_size,
        layers=tuple(layers),
        run=tuple(run),
        final_norm=norm(),
        tied_head=True,
        max_positions=MAX_POSITIONS,
    )


def checkpoint_map(c: TokuvikConfig) -> dict:
    """Plan tensor name -> checkpoint names.  The projections that read a mixer's input are stacked into one matrix, in
    the order the parts expect their columns; a layer's table of token inputs is its columns of the one that is stored."""
    names = {"embed.weight": "embed", "final_norm.weight": "final.norm"}
    for i, layer in enumerate(c.layers):
        src, dst = f"l{i}.", f"layers.{i}."
        names[dst + "mixer_norm.weight"] = src + "norm1"
        names[dst + "mixer_post_norm.weight"] = src + "norm1b"
        mix, to = src + "mix.", dst + "mixer."
        if layer.type == "attention":
            own = layer.mixer.kv_from < 0
            names[to + "in.weight"] = [mix + p for p in (("q", "k", "v", "g") if own else ("q", "g"))]
            names[to + "out_t.weight"] = Take(mix + "o", transpose=True)
            for p in ("q", "k") if own else ("q",):
                names[to + f"c0.{p}_norm"] = mix + p + ".norm"
        elif layer.type == "latent_attention":
            names[to + "in.weight"] = [mix + "dq", mix + "dkv", mix + "g"]
            names[to + "q_norm.weight"] = mix + "dq.norm"
            names[to + "kv_norm.weight"] = mix + "dkv.norm"
            names[to + "sink"] = mix + "sink"
            for p in ("uq", "uk", "uv", "o"):
                names[to + p + ".weight"] = mix + p
        else:
            names[to + "in.weight"] = mix + "in"
            names[to + "conv.weight"] = mix + "conv"
            names[to + "conv.bias"] = mix + "conv.b"
            names[to + "a_log"] = mix + "A_log"
            names[to + "dt_bias"] = mix + "dt_bias"
            names[to + "skip"] = mix + "D"
            names[to + "out_norm.weight"] = mix + "norm"
            names[to + "out.weight"] = mix + "o"
        if layer.ff:
            names[dst + "ffn_norm.weight"] = src + "norm2"
            names[dst + "ffn_post_norm.weight"] = src + "norm2b"
            names[dst + "ffn.gate_up.weight"] = [src + "mlp.gate", src + "mlp.up"]
            names[dst + "ffn.down.weight"] = src + "mlp.down"
        if c.side_dim:
            names[dst + "token_input.table"] = Take("side.embed", cols=(i * c.side_dim, (i + 1) * c.side_dim))
            names[dst + "token_input.gate.weight"] = src + "side.gate"
            names[dst + "token_input.proj.weight"] = src + "side.proj"
            names[dst + "token_norm.weight"] = src + "side.norm"
    return names


def checkpoint_shapes(c: TokuvikConfig) -> dict:
    """Checkpoint name -> (shape, role), in the order in which random weights are drawn."""
    h = c.hidden_size
    shapes = {"embed": ((c.vocab_size, h), "matrix")}
    if c.side_dim:
        shapes["side.embed"] = ((c.vocab_size, len(c.layers) * c.side_dim), "matrix")
    for i, layer in enumerate(c.layers):
        p, m = f"l{i}.", layer.mixer
        for name in ("norm1", "norm1b") + (("norm2", "norm2b") if layer.ff else ()):
            shapes[p + name] = ((h,), "vector")
        x = p + "mix."
        if layer.type == "attention":
            shapes[x + "q"] = ((m.heads * m.dim, h), "matrix")
            shapes[x + "q.norm"] = ((m.heads * m.dim,), "vector")
            if m.kv_from < 0:
                shapes[x + "k"] = ((m.kv_heads * m.dim, h), "matrix")
                shapes[x + "k.norm"] = ((m.kv_heads * m.dim,), "vector")
                shapes[x + "v"] = ((m.kv_heads * m.vdim, h), "matrix")
            shapes[x + "g"] = ((m.heads, h), "matrix")
            shapes[x + "o"] = ((h, m.heads * m.vdim), "matrix")
        elif layer.type == "latent_attention":
            shapes[x + "dq"] = ((m.q_rank, h), "matrix")
            shapes[x + "dq.norm"] = ((m.q_rank,), "vector")
            shapes[x + "uq"] = ((m.heads * m.dim, m.q_rank), "matrix")
            shapes[x + "dkv"] = ((m.kv_rank, h), "matrix")
            shapes[x + "dkv.norm"] = ((m.kv_rank,), "vector")
            shapes[x + "uk"] = ((m.heads * m.dim, m.kv_rank), "matrix")
            shapes[x + "uv"] = ((m.heads * m.vdim, m.kv_rank), "matrix")
            shapes[x + "sink"] = ((m.heads,), "bias")
            shapes[x + "g"] = ((m.heads * m.vdim, h), "matrix")
            shapes[x + "o"] = ((h, m.heads * m.vdim), "matrix")
        else:
            inner = m.heads * m.vdim
            channels = inner + 2 * m.groups * m.state
            shapes[x + "in"] = ((inner + channels + m.heads, h), "matrix")
            shapes[x + "conv"] = ((channels, m.conv), "matrix")
            shapes[x + "conv.b"] = ((channels,), "bias")
            shapes[x + "dt_bias"] = ((m.heads,), "bias")
            shapes[x + "A_log"] = ((m.heads,), "log_rate")
            shapes[x + "D"] = ((m.heads,), "vector")
            shapes[x + "norm"] = ((inner,), "vector")
            shapes[x + "o"] = ((h, inner), "matrix")
        if layer.ff:
            shapes[p + "mlp.gate"] = ((layer.ff, h), "matrix")
            shapes[p + "mlp.up"] = ((layer.ff, h), "matrix")
            shapes[p + "mlp.down"] = ((h, layer.ff), "matrix")
        if c.side_dim:
            shapes[p + "side.gate"] = ((c.side_dim, h), "matrix")
            shapes[p + "side.proj"] = ((h, c.side_dim), "matrix")
            shapes[p + "side.norm"] = ((h,), "vector")
    shapes["final.norm"] = ((h,), "vector")
    return shapes


TOKUVIK = register_architecture(
    Architecture(
        name=TokuvikConfig.architecture,
        parse_config=TokuvikConfig.from_dict,
        build_plan=build_plan,
        checkpoint_map=checkpoint_map,
        checkpoint_shapes=checkpoint_shapes,
    ),
    replace=True,
)
