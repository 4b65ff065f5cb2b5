"""Retention as a mixer: linear attention with a fixed decay per head and no softmax or denominator. One fused projection
gives v | k | q | gate (heads x value_dim, heads x head_dim twice, heads x value_dim), 32-bit on its way out; k and q turn by
their positions (`position` names a `rotary_frequencies` encoding in halves), k is multiplied by head_dim^(-1/2), and a head's
state moves as S <- decay S + k v^T, o = S^T q. Each head's o is divided by its root mean square (no weight), the heads side by
side are multiplied by silu(gate), and the output projection follows. S is kept in 32-bit floats in the request's state slot,
zero at its start, and carried from step to step by the state-space mixer's kernels (`hip.ssd_scan`: v as its input, k and q as
its B and C, a group per head, head_dim^(-1/2) as every token's step size). Angles, decays, the state, its read-out and the norm
are 32-bit in every storage type; v and the turned k and q enter the recurrence in the engine's."""

from __future__ import annotations

import math
from typing import Sequence

import torch

from tinyserve_llm_amd.ops import hip
from tinyserve_llm_amd.parts.base import LayerMemory, Mixer, ParamSpec, StateSpec, StepContext, register
from tinyserve_llm_amd.parts.linear import linear, streaming_copy


@register("mixer", "retention")
class Retention(Mixer):
    graph_safe = True

    def __init__(self, hidden_size: int, num_heads: int, head_dim: int, value_dim: int, decay: Sequence[float], norm_eps: float,
                 position: str | None = None) -> None:
        if len(decay) != num_heads or not all(0.0 <= d <= 1.0 for d in decay):
            raise ValueError(f"decay {list(decay)}: a number from 0 to 1 for each of {num_heads} heads")
        self.sizes = hip.SsdSizes(num_heads, value_dim, num_heads, head_dim, 1)
        self.hidden_size, self.decay, self.norm_eps, self.position = hidden_size, tuple(float(d) for d in decay), norm_eps, position
        self.proj: torch.Tensor | None = None
        self.o: torch.Tensor | None = None
        self.proj_packed = self.o_packed = None
        self._keeps: torch.Tensor | None = None        # per head: the decay, its logarithm, the step size
        self._logs: torch.Tensor | None = None
        self._steps: torch.Tensor | None = None

    @property
    def projected(self) -> int:
        return self.sizes.channels + self.sizes.inner

    def param_specs(self) -> dict[str, ParamSpec]:
        # (rows of zeros fill the projection up to a multiple of eight: its result's rows then start at 16-byte borders)
        return {"proj": ParamSpec((-(-self.projected // 8) * 8, self.hidden_size)),
                "o": ParamSpec((self.hidden_size, self.sizes.inner))}

    def bind(self, params) -> None:
        super().bind(params)
        self.proj[self.projected:].zero_()
        logs = [math.log(d) if d > 0 else -math.inf for d in self.decay]
        self._keeps, self._logs, self._steps = (torch.tensor(v, dtype=torch.float32).to(self.proj.device) for v in (
            self.decay, logs, [self.sizes.state ** -0.5] * self.sizes.heads))

    def state_spec(self) -> StateSpec:
        return StateSpec((self.sizes.matrix,), torch.float32)

    def widest_activation(self) -> int:
        # (a long portion's chunks of 64 tokens each keep a state)
        return max(self.projected + 7, self.sizes.row, -(-self.sizes.matrix // hip.SSD_CHUNK))

    def keep_streaming_copies(self) -> int:
        self.proj_packed, self.o_packed = streaming_copy(self.proj), streaming_copy(self.o)
        return sum(c.nbytes() for c in (self.proj_packed, self.o_packed) if c is not None)

    def forward(self, x: torch.Tensor, ctx: StepContext, mem: LayerMemory) -> torch.Tensor:
        z = self.sizes
        enc = ctx.position_encodings[self.position] if self.position else None
        proj = linear(x, self.proj, out_dtype=torch.float32, packed=self.proj_packed)
        mixed = hip.retention_prepare(proj, enc.frequencies() if enc is not None else None, ctx.positions, z, x.dtype)
        o = hip.ssd_scan(mixed, self._steps, self._logs, None, mem.state, ctx, z, keeps=self._keeps)
        gated = hip.mlstm_finish(o, None, proj[:, z.channels:z.channels + z.inner], z.heads, z.vdim, self.norm_eps, x.dtype, silu_gate=True)
        return linear(gated, self.o, out_dtype=torch.float32, packed=self.o_packed)
