"""What a pass through a looped stretch of layers starts from (`parts.base.PassInput`).

`ProjectedPassInput` ("projected_pass_input"): x <- W [x; x0] + step[n], with x the 32-bit stream as the run before left
it, x0 the embedding's rows and step[n] a learned vector of the pass. The projection's operand is made by the kernel that
does the stream's pending sum; its result is 32-bit and is the new stream, to which the kernel of the first layer's norm
adds step[n]."""

from __future__ import annotations

import torch

from tinyserve_llm_amd.parts.base import ParamSpec, PassInput, StepContext, register
from tinyserve_llm_amd.parts.linear import linear, streaming_copy
from tinyserve_llm_amd.parts.stream import ResidualStream


@register("pass_input", "projected_pass_input")
class ProjectedPassInput(PassInput):
    graph_safe = True

    def __init__(self, hidden_size: int, passes: int) -> None:
        if passes < 1:
            raise ValueError(f"{passes} passes: at least one")
        self.hidden_size, self.passes = hidden_size, passes
        self.weight: torch.Tensor | None = None        # [hidden, 2 hidden]: the stream's columns, then the embedding's
        self.step: torch.Tensor | None = None
        self.weight_packed = None

    def param_specs(self) -> dict[str, ParamSpec]:
        return {"weight": ParamSpec((self.hidden_size, 2 * self.hidden_size), init=(0.0, (2 * self.hidden_size) ** -0.5)),
                "step": ParamSpec((self.passes, self.hidden_size), init=(0.0, 0.3))}

    def keep_streaming_copies(self) -> int:
        self.weight_packed = streaming_copy(self.weight)
        return 0 if self.weight_packed is None else self.weight_packed.nbytes()

    def widest_activation(self) -> int:
        return 2 * self.hidden_size

    def forward(self, stream: ResidualStream, start: torch.Tensor, ctx: StepContext, n: int) -> ResidualStream:
        rows = stream.joined_with(start, self.weight.dtype)
        return ResidualStream(linear(rows, self.weight, out_dtype=torch.float32, packed=self.weight_packed), bias=self.step[n])
