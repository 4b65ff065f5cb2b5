"""The Morulix decoder as a ModelSpec. Token rows start a 32-bit residual stream; every layer is
x <- x + (mixer(n x) + ff(n x)) with one RMS norm for both sublayers, its weight stored around zero
(n(x) = rms(x) (1 + w)). The mixer is, layer by layer, a state-space mixer (`parts.mamba2.Mamba2`), grouped-query
attention in a sliding window with rotate-half positions whose frequencies are slowed by wavelength
(`parts.attention.GeneralAttention`), or attention through a low-rank latent without positions, with queries straight
from the layer's input, a learned sink and a gate per head (`parts.latent.LatentAttention`); the feed-forward is a
silu-gated unit or absent. A stretch of layers runs several times in a row with the same weights, every pass with caches
and states of its own; ahead of each pass the stream is made anew from itself and the embedded tokens
(`parts.pass_input.ProjectedPassInput`). Checkpoint names: `embed`, `loop.{in,step}`, `l<i>.norm1`,
`l<i>.mix.{in,conv,conv.b,dt_bias,A_log,D,norm,o}` or `l<i>.mix.{q,k,v,o}` or
`l<i>.mix.{q,dkv,dkv.norm,uk,uv,sink,g,o}`, `l<i>.mlp.{gate,up,down}`, `final.norm`, `head`."""

from __future__ import annotations

from tinyserve_llm_amd.config.morulix import MorulixAttention, MorulixConfig, MorulixLatentAttention, MorulixMamba2, MorulixRotation
from tinyserve_llm_amd.models.fanotar import _unit_names
from tinyserve_llm_amd.models.registry import Architecture, register_architecture
from tinyserve_llm_amd.models.spec import Destination, LayerRun, LayerSpec, ModelSpec
from tinyserve_llm_amd.models.tegolix import SILU_UNIT
from tinyserve_llm_amd.parts.base import PartSpec


def _encoding(encodings: dict[str, PartSpec], rot: MorulixRotation) -> str | None:
    """The name of the position encoding for a rotation (one per distinct set of constants), made if new."""
    if not rot.dims:
        return None
    bands = None if rot.bands is None else dict(factor=rot.bands.factor, low=rot.bands.low, high=rot.bands.high, original=rot.bands.original)
    name = f"rotary_{rot.dims}_{rot.base!r}_halves" + ("" if bands is None else "_bands_" + "_".join(repr(v) for v in bands.values()))
    encodings.setdefault(name, PartSpec("rotary_frequencies", dict(rotary_dim=rot.dims, theta=rot.base, interleaved=False, bands=bands)))
    return name


def morulix_spec(config: MorulixConfig) -> ModelSpec:
    c = config
    norm = PartSpec("rmsnorm", dict(hidden_size=c.width, eps=c.norm_eps, one_plus=True))
    ckpt: dict[str, Destination] = {"embed": Destination("embed.weight"), "final.norm": Destination("final_norm.weight"),
                                    "head": Destination("head.weight")}
    encodings: dict[str, PartSpec] = {}
    layers: list[LayerSpec] = []
    for i, layer in enumerate(c.layers):
        src, dst, m = f"l{i}", f"layers.{i}", layer.mixer
        ckpt[f"{src}.norm1"] = Destination(f"{dst}.norm1.weight")
        if isinstance(m, MorulixMamba2):
            mixer = PartSpec("mamba2", dict(hidden_size=c.width, num_heads=m.heads, value_dim=m.vdim, state_size=m.state, groups=m.groups,
                                            conv_taps=m.conv, norm_groups=m.norm_groups, norm_eps=c.norm_eps))
            inner, shared = m.heads * m.vdim, m.groups * m.state
            ckpt[f"{src}.mix.in"] = Destination(f"{dst}.mixer.proj", 0, 2 * inner + 2 * shared + m.heads)
            for name, param in (("conv", "conv"), ("conv.b", "conv_bias"), ("dt_bias", "dt_bias"), ("A_log", "a_log"), ("D", "skip"),
                                ("norm", "norm")):
                ckpt[f"{src}.mix.{name}"] = Destination(f"{dst}.mixer.{param}")
        elif isinstance(m, MorulixAttention):
            mixer = PartSpec("attention_general", dict(
                hidden_size=c.width, num_heads=m.heads, num_kv_heads=m.kv_heads, head_dim=m.dim, value_dim=m.vdim,
                position=_encoding(encodings, m.rot), scale=m.scale, window=m.window))
            q, k, v = m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim
            ckpt[f"{src}.mix.q"] = Destination(f"{dst}.mixer.qkv", 0, q)
            ckpt[f"{src}.mix.k"] = Destination(f"{dst}.mixer.qkv", q, k)
            ckpt[f"{src}.mix.v"] = Destination(f"{dst}.mixer.qkv", q + k, v)
        else:
            assert isinstance(m, MorulixLatentAttention)
            mixer = PartSpec("latent_attention", dict(
                hidden_size=c.width, num_heads=m.heads, head_dim=m.dim, rot_dim=0, value_dim=m.vdim, kv_rank=m.kv_rank, q_rank=0,
                position=None, scale=m.scale, norm_eps=c.norm_eps, sink=True, head_gate=True))
            at = 0
            for name, rows in (("q", m.heads * m.dim), ("dkv", m.kv_rank), ("g", m.heads)):
                ckpt[f"{src}.mix.{name}"] = Destination(f"{dst}.mixer.down", at, rows)
                at += rows
            for name, param in (("dkv.norm", "kv_norm"), ("uk", "uk"), ("uv", "uv"), ("sink", "sinks")):
                ckpt[f"{src}.mix.{name}"] = Destination(f"{dst}.mixer.{param}")
        ckpt[f"{src}.mix.o"] = Destination(f"{dst}.mixer.o")
        if layer.ff is None:
            ff = PartSpec("none")
        else:
            ff = PartSpec("capped_glu", dict(hidden_size=c.width, intermediate_size=layer.ff, **SILU_UNIT))
            _unit_names(ckpt, f"{src}.mlp", f"{dst}.ff.", layer.ff)
        layers.append(LayerSpec(mixer, ff, {"norm1": norm}, "parallel_one_norm"))
    inputs = {}
    if c.loop_times:
        inputs["loop"] = PartSpec("projected_pass_input", dict(hidden_size=c.width, passes=c.loop_times))
        ckpt["loop.in"] = Destination("pass_inputs.loop.weight")
        ckpt["loop.step"] = Destination("pass_inputs.loop.step")
    order = [LayerRun(i, begins=None if t is None else ("loop", t)) for i, t in c.run_order()]
    table = PartSpec("table", dict(vocab_size=c.vocab, hidden_size=c.width, float32_stream=True, init=(0.0, 1.0)))
    return ModelSpec(
        architecture=c.architecture, vocab_size=c.vocab, hidden_size=c.width, max_position=None, layers=layers, order=order,
        final_norm=norm, position_encodings=encodings, tie_word_embeddings=False, residual_dtype="float32", embedding=table,
        pass_inputs=inputs, checkpoint=ckpt)


MORULIX = register_architecture(Architecture(
    name="Morulix", model_types=("morulix",), config_from_dict=MorulixConfig.from_dict, build_spec=morulix_spec,
    config_to_dict=MorulixConfig.to_dict))
