"""A state space per head (Mamba-2) as a mixer.

    [z | x | B | C | step] = W_in h;   x, B, C <- silu(conv([x | B | C]) + bias)      (causal, per channel)
    dt = softplus(step + dt_bias);   S_t = exp(-exp(A_log) dt) S_(t-1) + dt B_t x_t^T;   y_t = S_t^T C_t + D x_t
    out = W_o (norm(y * silu(z)) * gain)      (the norm in equal groups)

The state [heads, state_dim, value_dim] and the convolution's last taps - 1 inputs are fp32 and wait in slots per request; a
row that starts its sequence starts from zero, a later row goes on where the row before stopped, so a prompt may be cut
anywhere.  Everything between the input and the output product is fp32 in both precisions.
"""

import torch

from atomserve_amd.kernels import ops
from atomserve_amd.parts.base import Mixer, StateCacheRequest, WeightDecl, register
from atomserve_amd.parts.recurrent import _step_rows


class StateSpace(Mixer):
    capturable = True

    def __init__(self, spec, env):
        super().__init__(spec, env)
        s = spec
        if min(s.num_heads, s.value_dim, s.state_dim, s.groups, s.norm_groups) < 1:
            raise ValueError("sizes of a state space are positive")
        if s.num_heads % s.groups:
            raise ValueError(f"{s.num_heads} heads do not divide over {s.groups} groups of B and C")
        self.inner = s.num_heads * s.value_dim
        if self.inner % s.norm_groups:
            raise ValueError(f"an output of {self.inner} does not divide into {s.norm_groups} groups of the norm")
        if not 1 <= s.conv.taps <= ops.CONV_MAX_TAPS:
            raise ValueError(f"a short convolution has 1 to {ops.CONV_MAX_TAPS} taps, not {s.conv.taps}")
        if s.state_dim > ops.STATE_SPACE_MAX_STATE:
            raise ValueError(f"a state of {s.state_dim} rows exceeds the scan's {ops.STATE_SPACE_MAX_STATE}")
        self.channels = self.inner + 2 * s.groups * s.state_dim  # what passes the convolution: x, B, C
        self.conv_off, self.step_off = self.inner, self.inner + self.channels
        self.in_rows = self.step_off + s.num_heads

    def weight_decls(self) -> dict:
        s = self.spec
        decls = {
            "in.weight": WeightDecl((self.in_rows, s.hidden_size)),
            "conv.weight": WeightDecl((self.channels, s.conv.taps), role="vector"),
            "conv.bias": WeightDecl((self.channels,), role="vector"),
            "out_norm.weight": WeightDecl((self.inner,), role="vector"),
            "out.weight": WeightDecl((s.hidden_size, self.inner)),
        }
        decls.update({name: WeightDecl((s.num_heads,), role="vector") for name in ("a_log", "dt_bias", "skip")})
        return decls

    def bind(self, tensors: dict) -> None:
        super().bind(tensors)
        # what the recurrence reads is fp32 (a bfloat16 checkpoint's values widen exactly)
        for name in ("conv_weight", "conv_bias", "a_log", "dt_bias", "skip", "out_norm_weight"):
            setattr(self, name, getattr(self, name).float().contiguous())
        self.inp = ops.Streamed(self.in_weight, self.env.stream_copies)
        self.out = ops.Streamed(self.out_weight, self.env.stream_copies)

    def streamed(self) -> list:
        return [self.inp, self.out]

    def cache_request(self):
        s = self.spec
        asked = {"state": StateCacheRequest((s.num_heads, s.state_dim, s.value_dim), torch.float32)}
        if s.conv.taps > 1:
            asked["conv"] = StateCacheRequest((s.conv.taps - 1, self.channels), torch.float32)
        return asked

    def forward(self, h, step, cache):
        s, env = self.spec, self.env
        T, dev = h.shape[0], h.device
        proj = torch.empty((T, self.in_rows), dtype=env.dtype, device=dev)
        ops.gemm(h, self.inp, proj, env.products)
        rows = _step_rows(step)
        state = cache["state"]
        history = cache["conv"].state if "conv" in cache else torch.empty((1, 0, self.channels), dtype=torch.float32, device=dev)
        xbc = torch.empty((T, self.channels), dtype=torch.float32, device=dev)
        ops.short_conv(proj, self.conv_off, self.conv_weight, history, rows, xbc, bias=self.conv_bias, silu=True, writes=state.writes)
        y = torch.empty((T, self.inner), dtype=torch.float32, device=dev)
        ops.state_space(xbc, s.num_heads, s.groups, s.state_dim, s.value_dim, proj, self.step_off, self.dt_bias, self.a_log, self.skip,
                        state.state, rows, y, writes=state.writes, longest=step.longest_row)  # fmt: skip
        act = torch.empty((T, self.inner), dtype=env.dtype, device=dev)
        ops.gated_group_norm(y, s.norm_groups, s.out_norm_eps, self.out_norm_weight, proj, 0, act)
        out = torch.empty((T, s.hidden_size), dtype=env.dtype, device=dev)
        ops.gemm(act, self.out, out, env.products)
        return out


register("mixer", "state_space", StateSpace)
