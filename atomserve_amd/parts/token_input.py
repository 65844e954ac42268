"""What a layer adds to the stream for the tokens themselves, beside its mixer and feed-forward.

    e = the token's row of a table of the layer's own [vocab, dim];   y = P (gelu(G x) * e)

x is the stream as it is, not a norm of it; the norm of y belongs to the arrangement, which adds it into the stream.
"""

import torch

from atomserve_amd.kernels import ops
from atomserve_amd.parts.base import Part, WeightDecl, register


class GatedTableInput(Part):
    capturable = True

    def __init__(self, spec, env):
        super().__init__(spec, env)
        if min(spec.dim, spec.hidden_size, spec.vocab_size) < 1:
            raise ValueError("sizes of a layer's token input are positive")

    def weight_decls(self) -> dict:
        s = self.spec
        return {
            "table": WeightDecl((s.vocab_size, s.dim)),
            "gate.weight": WeightDecl((s.dim, s.hidden_size)),
            "proj.weight": WeightDecl((s.hidden_size, s.dim)),
        }

    def bind(self, tensors: dict) -> None:
        super().bind(tensors)
        self.gate = ops.Streamed(self.gate_weight, self.env.stream_copies)
        self.proj = ops.Streamed(self.proj_weight, self.env.stream_copies)

    def streamed(self) -> list:
        return [self.gate, self.proj]

    def forward(self, x, step):
        """x [T, hidden] in the compute dtype -> [T, hidden]."""
        s, env = self.spec, self.env
        T, dev = x.shape[0], x.device
        g = torch.empty((T, s.dim), dtype=env.dtype, device=dev)
        ops.gemm_token_gate(x, self.gate, self.table, step.token_ids, g, env.products)
        y = torch.empty((T, s.hidden_size), dtype=env.dtype, device=dev)
        ops.gemm(g, self.proj, y, env.products)
        return y


register("token_input", "gated_table", GatedTableInput)
