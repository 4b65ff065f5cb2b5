"""Parts that layers are assembled from. Importing the package registers the built-in parts."""

from tinyserve_llm_amd.parts import base  # noqa: F401
from tinyserve_llm_amd.parts import (attention, block, ends, gated_delta, latent, linear_attention, mamba2, mingru, mlp, mlstm, moe, norm,  # noqa: F401
                                     pass_input, retention, rope, side_by_side, stream, token_input)  # noqa: F401  (registration)
