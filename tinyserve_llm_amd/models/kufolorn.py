"""The Kufolorn decoder as a ModelSpec. Token rows start a 32-bit residual stream, whose rows the sublayers read as they are;
every layer is x <- x + n1(mixer(x)), x <- x + n2(ff(x)) with RMS norms whose weights are stored around zero
(n(x) = rms(x) (1 + w)). The mixer is, layer by layer, a gated delta rule behind short convolutions
(`parts.gated_delta.GatedDelta`) or two mixers side by side (`parts.side_by_side.SideBySide`): grouped-query attention over
every position before with biases, norms over the whole query and key projections, rotate-half positions with linear scaling,
a learned sink and a gate per head (`parts.attention.GeneralAttention`), beside retention with a fixed decay per head
(`parts.retention.Retention`). The feed-forward is a gelu-gated unit, a mixture of capped experts scored by a softmax over all
router outputs and chosen inside the best groups, the last router outputs standing for identity experts, or absent. The head
is the embedding's table, its logits capped. Checkpoint names: `embed`, `l<i>.{norm1,norm2}`,
`l<i>.mix.{q,k,v,q.conv,k.conv,v.conv,b,a,A_log,dt_bias,g,norm,o}` or
`l<i>.mix.left.{q,k,v,q.b,k.b,v.b,q.norm,k.norm,sink,g,o}` with `l<i>.mix.right.{q,k,v,g,o}`, `l<i>.mlp.{gate,up,down}` or
`l<i>.mlp.{router,correction}`, `l<i>.mlp.e<j>.{gate,up,down}`, `final.norm`."""

from __future__ import annotations

from tinyserve_llm_amd.config.kufolorn import KufolornConfig, KufolornDelta, KufolornDense, KufolornExperts, KufolornParallel, KufolornRotation
from tinyserve_llm_amd.models.fanotar import _unit_names
from tinyserve_llm_amd.models.registry import Architecture, register_architecture
from tinyserve_llm_amd.models.spec import Destination, LayerRun, LayerSpec, ModelSpec
from tinyserve_llm_amd.parts.base import PartSpec

EXPERT_SLOPE, EXPERT_SHIFT = 1.702, 1.0        # an expert's unit: g sigmoid(1.702 g) (u + 1)


def _encoding(encodings: dict[str, PartSpec], rot: KufolornRotation) -> str | None:
    """The name of the position encoding for a rotation (one per distinct set of constants), made if new."""
    if not rot.dims:
        return None
    name = f"rotary_{rot.dims}_{rot.base!r}_halves" + ("" if rot.factor == 1.0 else f"_over_{rot.factor!r}")
    encodings.setdefault(name, PartSpec("rotary_frequencies", dict(rotary_dim=rot.dims, theta=rot.base, interleaved=False, divide=rot.factor)))
    return name


def _stretches(ckpt: dict[str, Destination], src: str, param: str, stretches) -> None:
    """Tensors `<src><name>` one behind the other in the rows of one parameter; `stretches`: (name, rows)."""
    at = 0
    for name, rows in stretches:
        ckpt[src + name] = Destination(param, at, rows)
        at += rows


def kufolorn_spec(config: KufolornConfig) -> ModelSpec:
    c = config
    norm = PartSpec("rmsnorm", dict(hidden_size=c.width, eps=c.norm_eps, one_plus=True))
    ckpt: dict[str, Destination] = {"embed": Destination("embed.weight"), "final.norm": Destination("final_norm.weight")}
    encodings: dict[str, PartSpec] = {}
    layers: list[LayerSpec] = []
    for i, layer in enumerate(c.layers):
        src, dst, m = f"l{i}", f"layers.{i}", layer.mixer
        if isinstance(m, KufolornDelta):
            mixer = PartSpec("gated_delta", dict(hidden_size=c.width, num_heads=m.heads, groups=m.kv_heads, head_dim=m.dim, value_dim=m.vdim,
                                                 conv_taps=m.conv, norm_eps=c.norm_eps))
            shared, inner = m.kv_heads * m.dim, m.heads * m.vdim
            _stretches(ckpt, f"{src}.mix.", f"{dst}.mixer.proj", (("g", inner), ("v", inner), ("k", shared), ("q", shared), ("a", m.heads), ("b", m.heads)))
            _stretches(ckpt, f"{src}.mix.", f"{dst}.mixer.conv", (("v.conv", inner), ("k.conv", shared), ("q.conv", shared)))
            for name, param in (("dt_bias", "dt_bias"), ("A_log", "a_log"), ("norm", "norm"), ("o", "o")):
                ckpt[f"{src}.mix.{name}"] = Destination(f"{dst}.mixer.{param}")
        else:
            assert isinstance(m, KufolornParallel)
            a, r = m.left, m.right
            left = PartSpec("attention_general", dict(
                hidden_size=c.width, num_heads=a.heads, num_kv_heads=a.kv_heads, head_dim=a.dim, value_dim=a.vdim,
                position=_encoding(encodings, a.rot), scale=a.scale, learned_sink=True, projection_norm_eps=c.norm_eps, head_gate=True, bias=True))
            right = PartSpec("retention", dict(hidden_size=c.width, num_heads=r.heads, head_dim=r.dim, value_dim=r.vdim, decay=r.decay,
                                               norm_eps=c.norm_eps, position=_encoding(encodings, r.rot)))
            mixer = PartSpec("side_by_side", dict(left=left, right=right, left_scale=m.left_scale, right_scale=m.right_scale))
            q, k, v = a.heads * a.dim, a.kv_heads * a.dim, a.kv_heads * a.vdim
            _stretches(ckpt, f"{src}.mix.left.", f"{dst}.mixer.left_qkv", (("q", q), ("k", k), ("v", v), ("g", a.heads)))
            _stretches(ckpt, f"{src}.mix.left.", f"{dst}.mixer.left_qkv_bias", (("q.b", q), ("k.b", k), ("v.b", v)))
            for name, param in (("q.norm", "q_norm"), ("k.norm", "k_norm"), ("sink", "sinks"), ("o", "o")):
                ckpt[f"{src}.mix.left.{name}"] = Destination(f"{dst}.mixer.left_{param}")
            keys, values = r.heads * r.dim, r.heads * r.vdim
            _stretches(ckpt, f"{src}.mix.right.", f"{dst}.mixer.right_proj", (("v", values), ("k", keys), ("q", keys), ("g", values)))
            ckpt[f"{src}.mix.right.o"] = Destination(f"{dst}.mixer.right_o")
        norms = {"norm1": norm}
        ckpt[f"{src}.norm1"] = Destination(f"{dst}.norm1.weight")
        if layer.mlp is None:
            ff = PartSpec("none")
        else:
            norms["norm2"] = norm
            ckpt[f"{src}.norm2"] = Destination(f"{dst}.norm2.weight")
            if isinstance(layer.mlp, KufolornDense):
                ff = PartSpec("capped_glu", dict(hidden_size=c.width, intermediate_size=layer.mlp.ff, limit=0.0, up_shift=0.0, activation="gelu_tanh"))
                _unit_names(ckpt, f"{src}.mlp", f"{dst}.ff.", layer.mlp.ff)
            else:
                e: KufolornExperts = layer.mlp
                ff = PartSpec("routed_experts", dict(
                    hidden_size=c.width, num_experts=e.experts, top=e.top, intermediate_size=e.ff, limit=e.limit, slope=EXPERT_SLOPE,
                    up_shift=EXPERT_SHIFT, router_scale=1.0, normalize=False, correction=True, scoring="softmax_all", identity=e.identity,
                    groups=(e.groups, e.keep)))
                ckpt[f"{src}.mlp.router"] = Destination(f"{dst}.ff.router")
                ckpt[f"{src}.mlp.correction"] = Destination(f"{dst}.ff.correction")
                for j in range(e.experts):
                    _unit_names(ckpt, f"{src}.mlp.e{j}", f"{dst}.ff.", e.ff, index=(j,))
        layers.append(LayerSpec(mixer, ff, norms, "post_norm_stream"))
    table = PartSpec("table", dict(vocab_size=c.vocab, hidden_size=c.width, float32_stream=True, init=(0.0, 0.3)))
    head = PartSpec("projection", dict(vocab_size=c.vocab, hidden_size=c.width, tied=True, softcap=c.logit_softcap))
    return ModelSpec(
        architecture=c.architecture, vocab_size=c.vocab, hidden_size=c.width, max_position=None, layers=layers,
        order=[LayerRun(i) for i in range(len(layers))], final_norm=norm, position_encodings=encodings, tie_word_embeddings=True,
        residual_dtype="float32", embedding=table, head=head, checkpoint=ckpt)


KUFOLORN = register_architecture(Architecture(
    name="Kufolorn", model_types=("kufolorn",), config_from_dict=KufolornConfig.from_dict, build_spec=kufolorn_spec,
    config_to_dict=KufolornConfig.to_dict))
