"""The gated delta rule (Gated DeltaNet) as a mixer. One fused projection gives, per token, gate | v | k | q | a | b
(heads x value_dim twice, groups x head_dim twice, a number per head twice), 32-bit on its way out, in rows of a multiple of
eight numbers. v, k and q pass a causal convolution per channel (`conv_taps` taps, no bias) and silu; k and q are made unit
vectors per head, x / sqrt(sum(x^2) + 1e-6), q also times head_dim^(-1/2); head h reads the k and q of group
h // (heads / groups). With beta = sigmoid(b) and g = exp(-exp(A_log) softplus(a + dt_bias)) a head's state moves as
    S <- g S,   u = beta (v - S^T k),   S <- S + k u^T,   o = S^T q;
each head's o is divided by its root mean square, times a weight that all heads share, times silu(gate), and the output
projection follows. S and the convolution's last conv_taps - 1 inputs are kept in 32-bit floats in the request's state slot,
zero at its start, and carried from step to step (`hip.delta_scan`: token by token, or in chunks on the matrix cores where a
request feeds many). Unit factors, steps, decays, the state, its read-out and the norm are 32-bit in every storage type; v, k
and q leave the convolution in the engine's."""

from __future__ import annotations

import torch

from tinyserve_llm_amd.ops import hip
from tinyserve_llm_amd.parts.base import LayerMemory, Mixer, ParamSpec, StateSpec, StepContext, register
from tinyserve_llm_amd.parts.linear import linear, streaming_copy


@register("mixer", "gated_delta")
class GatedDelta(Mixer):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, groups: int, head_dim: int, value_dim: int, conv_taps: int, norm_eps: float) -> None:
        self.sizes = hip.SsdSizes(num_heads, value_dim, groups, head_dim, conv_taps)
        self.hidden_size, self.norm_eps = hidden_size, norm_eps
        self.proj: torch.Tensor | None = None
        self.conv: torch.Tensor | None = None
        self.dt_bias: torch.Tensor | None = None
        self.a_log: torch.Tensor | None = None
        self.norm: torch.Tensor | None = None
        self.o: torch.Tensor | None = None
        self.proj_packed = self.o_packed = None
        self._conv: torch.Tensor | None = None         # the convolution's weights [taps, row] in a mixed row's places

    @property
    def projected(self) -> int:
        return self.sizes.projected + self.sizes.heads

    def param_specs(self) -> dict[str, ParamSpec]:
        z = self.sizes
        # (rows of zeros fill the projection up to a multiple of eight: its result's rows then start at 16-byte borders)
        return {"proj": ParamSpec((-(-self.projected // 8) * 8, self.hidden_size)),
                "conv": ParamSpec((z.channels, z.taps), "float32", init=(0.0, z.taps ** -0.5)),      # v | k | q
                "dt_bias": ParamSpec((z.heads,), "float32", init=(-2.0, 1.0)),
                "a_log": ParamSpec((z.heads,), "float32", init=(0.0, 0.7)),
                "norm": ParamSpec((z.vdim,), "float32", init=(1.0, 0.1)),
                "o": ParamSpec((self.hidden_size, z.inner))}

    def bind(self, params) -> None:
        super().bind(params)
        self.proj[self.projected:].zero_()
        self._conv = self.sizes.spread(self.conv).t().contiguous()

    def state_spec(self) -> StateSpec:
        return StateSpec((self.sizes.matrix + self.sizes.kept,), torch.float32)

    def widest_activation(self) -> int:
        # (a long portion's chunks of 64 tokens each keep four 64 x 64 tiles a head, keys three times and values once more)
        z = self.sizes
        return max(self.projected + 7, z.row, z.heads * (4 * hip.SSD_CHUNK + z.vp) + 3 * z.groups * z.np)

    def keep_streaming_copies(self) -> int:
        self.proj_packed, self.o_packed = streaming_copy(self.proj), streaming_copy(self.o)
        return sum(c.nbytes() for c in (self.proj_packed, self.o_packed) if c is not None)

    def forward(self, x: torch.Tensor, ctx: StepContext, mem: LayerMemory) -> torch.Tensor:
        z = self.sizes
        proj = linear(x, self.proj, out_dtype=torch.float32, packed=self.proj_packed)
        rows = hip.delta_prepare(proj, self._conv, self.dt_bias, self.a_log, mem.state, ctx, z, x.dtype)
        o = hip.delta_scan(rows, mem.state, ctx, z)
        gated = hip.mlstm_finish(o, self.norm, proj[:, :z.inner], z.heads, z.vdim, self.norm_eps, x.dtype, silu_gate=True)
        return linear(gated, self.o, out_dtype=torch.float32, packed=self.o_packed)
