"""A state-space mixer with one decay per head (Mamba-2). One fused projection gives, per token, z | x | B | C | dt
(heads x value_dim, as much again, groups x state_size twice, a number per head), 32-bit on its way out, in rows of a
multiple of eight numbers. x, B and C pass a causal convolution per channel (`conv_taps` taps, with a bias) and silu; with
d = softplus(dt + dt_bias) and head h reading the B and C of its group, a head's state moves as
    S <- exp(-exp(A_log) d) S + d x B^T,   y = S C + D x;
the heads side by side are multiplied by silu(z), divided part by part (`norm_groups` equal parts) by their root mean
square, times a weight, and the output projection follows. S and the convolution's last conv_taps - 1 inputs are kept in
32-bit floats in the request's state slot, zero at its start, and carried from step to step (`hip.ssd_scan`: token by token,
or in chunks on the matrix cores where a request feeds many). Step sizes, decays, the state, its read-out and the norm are
32-bit in every storage type; x, B and C leave the convolution in the engine's."""

from __future__ import annotations

import torch

from tinyserve_llm_amd.ops import hip
from tinyserve_llm_amd.parts.base import LayerMemory, Mixer, ParamSpec, StateSpec, StepContext, register
from tinyserve_llm_amd.parts.linear import linear, streaming_copy


@register("mixer", "mamba2")
class Mamba2(Mixer):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, value_dim: int, state_size: int, groups: int, conv_taps: int, norm_groups: int,
                 norm_eps: float) -> None:
        self.sizes = hip.SsdSizes(num_heads, value_dim, groups, state_size, conv_taps)
        if norm_groups < 1 or self.sizes.inner % norm_groups:
            raise ValueError(f"norm_groups {norm_groups}: {self.sizes.inner} channels in equal parts")
        self.hidden_size, self.norm_groups, self.norm_eps = hidden_size, norm_groups, norm_eps
        self.proj: torch.Tensor | None = None
        self.conv: torch.Tensor | None = None
        self.conv_bias: torch.Tensor | None = None
        self.dt_bias: torch.Tensor | None = None
        self.a_log: torch.Tensor | None = None
        self.skip: torch.Tensor | None = None          # D
        self.norm: torch.Tensor | None = None
        self.o: torch.Tensor | None = None
        self.proj_packed = self.o_packed = None
        self._conv: tuple[torch.Tensor, torch.Tensor] | None = None      # weights [taps, row] and bias [row] in a mixed row's places

    def param_specs(self) -> dict[str, ParamSpec]:
        z = self.sizes
        # (rows of zeros fill the projection up to a multiple of eight: its result's rows then start at 16-byte borders)
        return {"proj": ParamSpec((-(-z.projected // 8) * 8, self.hidden_size)),
                "conv": ParamSpec((z.channels, z.taps), "float32", init=(0.0, z.taps ** -0.5)),
                "conv_bias": ParamSpec((z.channels,), "float32", init=(0.0, 0.2)),
                "dt_bias": ParamSpec((z.heads,), "float32", init=(-2.0, 1.0)),
                "a_log": ParamSpec((z.heads,), "float32", init=(0.0, 0.7)),
                "skip": ParamSpec((z.heads,), "float32", init=(1.0, 0.3)),
                "norm": ParamSpec((z.inner,), "float32", init=(1.0, 0.1)),
                "o": ParamSpec((self.hidden_size, z.inner))}

    def bind(self, params) -> None:
        super().bind(params)
        self.proj[self.sizes.projected:].zero_()
        self._conv = (self.sizes.spread(self.conv).t().contiguous(), self.sizes.spread(self.conv_bias))

    def state_spec(self) -> StateSpec:
        return StateSpec((self.sizes.matrix + self.sizes.kept,), torch.float32)

    def widest_activation(self) -> int:
        # (a long portion's chunks of 64 tokens each keep a state)
        return max(self.sizes.projected + 7, self.sizes.row, -(-self.sizes.matrix // hip.SSD_CHUNK))

    def keep_streaming_copies(self) -> int:
        self.proj_packed, self.o_packed = streaming_copy(self.proj), streaming_copy(self.o)
        return sum(c.nbytes() for c in (self.proj_packed, self.o_packed) if c is not None)

    def forward(self, x: torch.Tensor, ctx: StepContext, mem: LayerMemory) -> torch.Tensor:
        proj = linear(x, self.proj, out_dtype=torch.float32, packed=self.proj_packed)
        mixed, steps, logs = hip.ssd_prepare(proj, *self._conv, self.dt_bias, self.a_log, mem.state, ctx, self.sizes, x.dtype)
        y = hip.ssd_scan(mixed, steps, logs, self.skip, mem.state, ctx, self.sizes)
        gated = hip.gated_group_norm(y, proj[:, :self.sizes.inner], self.norm, self.norm_groups, self.norm_eps, x.dtype)
        return linear(gated, self.o, out_dtype=torch.float32, packed=self.o_packed)
