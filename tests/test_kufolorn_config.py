"""The Kufolorn configuration and model description on the CPU: config.json round trip, errors that name the key, cache and
state plans, the checkpoint table against the tensors a model folder holds, and the plain implementation's own mechanisms
worked out by hand."""

from __future__ import annotations

import json
import math

import pytest
import torch

from tests.helpers import kufolorn_configs, prompt
from tests.plain import kufolorn as plain
from tinyserve_llm_amd.config.kufolorn import KufolornConfig
from tinyserve_llm_amd.config.llama import ConfigError
from tinyserve_llm_amd.models.decoder import DecoderModel
from tinyserve_llm_amd.models.registry import architecture_of, read_config, resolve
from tinyserve_llm_amd.weights.random_init import write_random_model

F64 = torch.float64
NAMES = ["P", "Q", "R", "S", "T"]


@pytest.mark.parametrize("name", NAMES)
def test_round_trip_through_config_json(name, tmp_path):
    config, seed = kufolorn_configs()[name]
    raw = json.loads(json.dumps(architecture_of(config).to_dict(config)))
    assert raw["architecture"] == "Kufolorn" and resolve(raw).name == "Kufolorn"
    assert KufolornConfig.from_dict(raw) == config
    if name in "PQR":
        write_random_model(str(tmp_path), config, seed, torch.bfloat16)
        arch, again = read_config(str(tmp_path))
        assert arch.name == "Kufolorn" and again == config


def test_errors_name_the_key():
    config, _ = kufolorn_configs()["P"]
    raw = architecture_of(config).to_dict(config)

    def broken(edit):
        r = json.loads(json.dumps(raw))
        edit(r)
        return r
    left, right = (lambda r: r["layers"][1]["mixer"]["left"]), (lambda r: r["layers"][1]["mixer"]["right"])
    moe = lambda r: r["layers"][1]["mlp"]
    for edit, word in ((lambda r: r.pop("vocab"), "vocab"), (lambda r: r["norm"].pop("eps"), "eps"), (lambda r: r.update(logit_softcap=-1.0), "softcap"),
                       (lambda r: r["layers"][0]["mixer"].pop("conv"), "conv"), (lambda r: r["layers"][0]["mixer"].update(kv_heads=3), "kv_heads"),
                       (lambda r: r["layers"][0]["mixer"].update(conv=0), "conv"), (lambda r: left(r).update(kv_heads=3), "kv_heads"),
                       (lambda r: left(r)["rot"].update(dims=34), "rot"), (lambda r: left(r)["rot"].update(dims=15), "rot"),
                       (lambda r: left(r)["rot"]["scaling"].pop("factor"), "factor"), (lambda r: left(r)["rot"]["scaling"].update(factor=-2.0), "factor"),
                       (lambda r: left(r).pop("scale"), "scale"), (lambda r: r["layers"][1]["mixer"].pop("right_scale"), "right_scale"),
                       (lambda r: right(r)["decay"].pop(), "decay"), (lambda r: right(r).update(decay=[0.9, 0.9, 1.5]), "decay"),
                       (lambda r: right(r).update(decay=0.9), "decay"), (lambda r: right(r)["rot"].update(dims=22), "rot"),
                       (lambda r: moe(r)["router"].update(top=7), "top"), (lambda r: moe(r)["router"]["groups"].update(count=4), "groups"),
                       (lambda r: moe(r)["router"]["groups"].update(keep=4), "groups"), (lambda r: moe(r)["router"]["groups"].pop("keep"), "keep"),
                       (lambda r: moe(r)["expert"].update(limit=0.0), "limit"), (lambda r: moe(r)["expert"].pop("limit"), "limit"),
                       (lambda r: moe(r).update(kind="sparse"), "kind"), (lambda r: r["layers"][0].update(type="gla"), "type")):
        with pytest.raises(ConfigError, match=word):
            KufolornConfig.from_dict(broken(edit))


def test_plans():
    config, _ = kufolorn_configs()["P"]
    model = DecoderModel(architecture_of(config).build_spec(config))
    assert [(e.owner, e.kv.window, e.kv.num_kv_heads, e.kv.head_dim, e.kv.v_dim) for e in model.cache_plan()] == [(1, 0, 2, 32, 48)]
    # S in places of 32 x 32 a head, then three rows of the convolutions' inputs (4 x 32 + 2 x 2 x 32 places); the pair's S alone
    assert [(e.run, tuple(e.state.shape)) for e in model.state_plan()] == \
        [(0, (4 * 32 * 32 + 3 * 256,)), (1, (3 * 32 * 32,)), (2, (3 * 32 * 32 + 2 * 288,))]
    assert model.graph_safe()
    assert set(model.spec.position_encodings) == {"rotary_16_10000.0_halves_over_3.0", "rotary_12_500.0_halves"}
    config, _ = kufolorn_configs()["Q"]
    model = DecoderModel(architecture_of(config).build_spec(config))
    assert [e.owner for e in model.cache_plan()] == [0, 2] and [e.run for e in model.state_plan()] == [0, 1, 2, 3]
    assert model.head.softcap == 0.0 and model.spec.tie_word_embeddings


def test_checkpoint_names_and_shapes(tmp_path):
    from safetensors import safe_open
    config, seed = kufolorn_configs()["P"]
    write_random_model(str(tmp_path), config, seed, torch.bfloat16)
    with safe_open(str(tmp_path / "model.safetensors"), "pt", "cpu") as f:
        shapes = {k: tuple(f.get_slice(k).get_shape()) for k in f.keys()}
        tensors = {k: f.get_tensor(k) for k in f.keys()}
    assert shapes["embed"] == (200, 80) and shapes["final.norm"] == (80,) and "head" not in shapes
    assert shapes["l0.mix.q"] == shapes["l0.mix.k"] == (40, 80) and shapes["l0.mix.v"] == shapes["l0.mix.g"] == (112, 80)
    assert shapes["l0.mix.q.conv"] == shapes["l0.mix.k.conv"] == (40, 4) and shapes["l0.mix.v.conv"] == (112, 4)
    assert shapes["l0.mix.a"] == shapes["l0.mix.b"] == (4, 80) and shapes["l0.mix.A_log"] == shapes["l0.mix.dt_bias"] == (4,)
    assert shapes["l0.mix.norm"] == (28,) and shapes["l0.mix.o"] == (80, 112)
    assert shapes["l1.mix.left.q"] == (128, 80) and shapes["l1.mix.left.k"] == (64, 80) and shapes["l1.mix.left.v"] == (96, 80)
    assert shapes["l1.mix.left.q.b"] == shapes["l1.mix.left.q.norm"] == (128,) and shapes["l1.mix.left.k.b"] == shapes["l1.mix.left.k.norm"] == (64,)
    assert shapes["l1.mix.left.v.b"] == (96,) and shapes["l1.mix.left.sink"] == (4,) and shapes["l1.mix.left.g"] == (4, 80)
    assert shapes["l1.mix.left.o"] == (80, 192)
    assert shapes["l1.mix.right.q"] == shapes["l1.mix.right.k"] == (60, 80) and shapes["l1.mix.right.v"] == shapes["l1.mix.right.g"] == (84, 80)
    assert shapes["l1.mix.right.o"] == (80, 84)
    assert shapes["l0.mlp.gate"] == shapes["l0.mlp.up"] == (96, 80) and shapes["l0.mlp.down"] == (80, 96)
    assert shapes["l1.mlp.router"] == (9, 80) and shapes["l1.mlp.correction"] == (9,) and shapes["l1.mlp.e6.down"] == (80, 40)
    assert "l1.mlp.e7.down" not in shapes and not any(k.startswith("l2.mlp") or k == "l2.norm2" for k in shapes)
    # the loader puts every tensor back where the writer took it from; the rows that fill the projections up are zeros
    from tinyserve_llm_amd.weights.loader import load_params
    model = DecoderModel(architecture_of(config).build_spec(config))
    params = load_params(model, str(tmp_path), torch.bfloat16, "cpu")
    model.bind(params, torch.bfloat16, torch.device("cpu"))
    proj = params["layers.0.mixer.proj"]
    assert proj.shape == (312, 80), "112 + 112 + 40 + 40 + 4 + 4 rows"
    assert torch.equal(proj, torch.cat([tensors[f"l0.mix.{n}"] for n in ("g", "v", "k", "q", "a", "b")]))
    left, right = params["layers.1.mixer.left_qkv"], params["layers.1.mixer.right_proj"]
    assert torch.equal(left[:292], torch.cat([tensors[f"l1.mix.left.{n}"] for n in "qkvg"])) and left.shape == (296, 80)
    assert float(left[292:].abs().max()) == 0.0 and right.shape == (288, 80)
    assert torch.equal(params["layers.1.mixer.left_qkv_bias"], torch.cat([tensors[f"l1.mix.left.{n}.b"] for n in "qkv"]).float())
    assert torch.equal(right, torch.cat([tensors[f"l1.mix.right.{n}"] for n in "vkqg"]))
    # the convolutions' weights, taps first, in the places that the kernels work on: v of 4 heads, k and q of 2 groups
    conv = model.layers[0].mixer._conv
    assert conv.shape == (4, 256)
    assert torch.equal(conv[:, 32:60], tensors["l0.mix.v.conv"][28:56].t().float()) and float(conv[:, 60:64].abs().max()) == 0.0
    assert torch.equal(conv[:, 160:180], tensors["l0.mix.k.conv"][20:40].t().float()) and torch.equal(conv[:, 192:212], tensors["l0.mix.q.conv"][:20].t().float())
    # the head reads the embedding's table, capped
    assert model.head.weight is model.embedding.weight and model.head.softcap == 2.0


def test_parts_refuse_what_they_cannot_do():
    from tinyserve_llm_amd.parts.attention import GeneralAttention
    from tinyserve_llm_amd.parts.ends import ProjectionHead
    from tinyserve_llm_amd.parts.gated_delta import GatedDelta
    from tinyserve_llm_amd.parts.moe import RoutedExperts
    from tinyserve_llm_amd.parts.retention import Retention
    from tinyserve_llm_amd.parts.rope import RotaryFrequencies
    with pytest.raises(ValueError, match="bias"):
        GeneralAttention(64, 2, 2, 32, bias=True)
    with pytest.raises(ValueError, match="decay"):
        Retention(64, 2, 32, 32, [0.9], 1e-5)
    with pytest.raises(Exception, match="groups"):
        GatedDelta(64, 4, 3, 16, 16, 4, 1e-5)
    with pytest.raises(ValueError, match="groups"):
        RoutedExperts(64, 7, 2, 16, groups=(3, 1))
    with pytest.raises(ValueError, match="groups"):
        RoutedExperts(64, 6, 3, 16, groups=(3, 1))
    with pytest.raises(ValueError, match="softcap"):
        ProjectionHead(10, 4, softcap=-1.0)
    with pytest.raises(ValueError):
        RotaryFrequencies(8, 300.0, False, divide=0.0)
    with pytest.raises(ValueError):
        RotaryFrequencies(8, 300.0, False, divide=2.0, bands=dict(factor=2.0, low=1.0, high=4.0, original=64.0))


def test_the_engines_frequencies_are_the_plain_ones():
    from tinyserve_llm_amd.parts.rope import RotaryFrequencies
    for dims, base, factor in ((16, 10000.0, 3.0), (10, 50000.0, 1.0), (64, 250000.0, 0.5)):
        f = RotaryFrequencies(dims, base, False, divide=factor).host_frequencies()
        # the pair (1, 0) at position 1 turns to (cos f, sin f)
        x = torch.zeros(1, 1, dims, dtype=F64)
        x[0, 0, :dims // 2] = 1.0
        out = plain.rotate_halves(x, torch.tensor([1]), {"dims": dims, "base": base, "scaling": {"factor": factor}})[0, 0]
        torch.testing.assert_close(out, torch.cat([f.cos(), f.sin()]), atol=1e-14, rtol=1e-13)


# ---- the plain implementation's mechanisms by hand ------------------------------------------------

def test_halves_turn_slower_by_the_factor_and_the_rest_passes():
    x = torch.tensor([[[1.0, 0.0, 0.0, 1.0, 5.0]]], dtype=F64)
    # pairs (0, 2) and (1, 3): f = 1 / 4 and 1/2 / 4 with base 4, dims 4; at position 2 pi a quarter turn's twin each
    out = plain.rotate_halves(x, torch.tensor([2]), {"dims": 4, "base": 4.0, "scaling": {"factor": 4.0}})
    a, b = 2 / 4, 2 * 0.5 / 4
    assert out[0, 0].tolist() == pytest.approx([math.cos(a), -math.sin(b), math.sin(a), math.cos(b), 5.0])
    assert torch.equal(plain.rotate_halves(x, torch.tensor([9]), None), x)


def test_sinks_by_hand():
    # keys that all score 0, values 1, 2, ...: equal weights over what is seen; a sink of ln 2 counts as two more
    n = 6
    q, k = torch.zeros(n, 1, 2, dtype=F64), torch.zeros(n, 1, 2, dtype=F64)
    v = torch.arange(1, n + 1, dtype=F64).view(n, 1, 1)
    out = plain.sink_attention(q, k, v, torch.arange(n), 1.0, torch.tensor([math.log(2.0)], dtype=F64))
    assert out[:, 0, 0].tolist() == pytest.approx([1 / 3, 3 / 4, 6 / 5, 10 / 6, 15 / 7, 21 / 8])


def test_convolution_by_hand():
    u = torch.tensor([[1.0], [2.0], [3.0]], dtype=F64)
    w = torch.tensor([[10.0, 1.0, 0.1]], dtype=F64)
    silu = lambda z: z / (1 + math.exp(-z))
    assert plain.convolve(u, w, torch.zeros(2, 1, dtype=F64))[:, 0].tolist() == pytest.approx([silu(0.1), silu(1.2), silu(12.3)])
    assert plain.convolve(u[:1], w, torch.tensor([[7.0], [5.0]], dtype=F64))[0, 0].item() == pytest.approx(silu(70 + 5 + 0.1))


def test_unit_vectors_by_hand():
    out = plain.unit_vectors(torch.tensor([[3.0, 4.0], [0.0, 0.0], [1e-3, 0.0]], dtype=F64))
    assert out[0].tolist() == pytest.approx([0.6, 0.8], abs=1e-7) and out[1].tolist() == [0.0, 0.0]
    assert out[2, 0].item() == pytest.approx(1e-3 / math.sqrt(2e-6)), "eps counts where the vector is short"


def test_delta_rule_by_hand():
    # one head, two key dimensions, one value column: e0 is written, then overwritten with beta 1, e1 beside it
    e0, e1 = [1.0, 0.0], [0.0, 1.0]
    k = torch.tensor([[e0], [e1], [e0]], dtype=F64)
    q = torch.tensor([[e0], [[1.0, 1.0]], [e0]], dtype=F64)
    v = torch.tensor([[[8.0]], [[4.0]], [[6.0]]], dtype=F64)
    g = torch.tensor([[1.0], [0.5], [0.5]], dtype=F64)
    beta = torch.tensor([[0.5], [1.0], [1.0]], dtype=F64)
    o, S = plain.delta_rule(q, k, v, g, beta, torch.zeros(1, 2, 1, dtype=F64))
    # S = (4, 0); then (2, 0) + e1 4; then (1, 2) whose e0 entry becomes 6
    assert o[:, 0, 0].tolist() == pytest.approx([4.0, 6.0, 6.0]) and S[0, :, 0].tolist() == pytest.approx([6.0, 2.0])


def test_retention_by_hand():
    q = torch.tensor([[[1.0]], [[2.0]]], dtype=F64)
    k = torch.tensor([[[3.0]], [[1.0]]], dtype=F64)
    v = torch.tensor([[[5.0]], [[7.0]]], dtype=F64)
    o, S = plain.retention_rule(q, k, v, torch.tensor([0.5], dtype=F64), torch.zeros(1, 1, 1, dtype=F64))
    assert o[:, 0, 0].tolist() == pytest.approx([15.0, 2 * (7.5 + 7.0)]) and S[0, 0, 0].item() == pytest.approx(14.5)


def test_groups_by_hand():
    # three groups of two; scores are a softmax, choice scores negative everywhere: a group left out counts as minus infinity
    z = torch.log(torch.tensor([0.30, 0.02, 0.25, 0.03, 0.28, 0.12], dtype=F64))
    off = torch.full((6,), -2.0, dtype=F64)
    assert plain.choose(z, off, 3, 3, 2) == ([0, 4, 5], pytest.approx([0.30, 0.28, 0.12]))
    assert plain.choose(z, off, 3, 1, 1) == ([0, 4, 2], pytest.approx([0.30, 0.28, 0.25]))
    # the correction counts for the group too: it lifts the second group's weaker expert above everything
    off[3] = -1.0
    assert plain.choose(z, off, 3, 3, 2) == ([3, 0, 2], pytest.approx([0.03, 0.30, 0.25]))


def test_capped_expert_and_dense_unit_by_hand():
    one = torch.tensor([[1.0]], dtype=F64)
    y = plain.capped_expert(torch.tensor([[3.0], [-9.0]], dtype=F64), one, one, one, 2.0)
    sig = lambda z: 1 / (1 + math.exp(-z))
    assert y[:, 0].tolist() == pytest.approx([2 * sig(1.702 * 2) * 3, -9 * sig(-1.702 * 9) * -1])
    out = plain.dense_unit(torch.tensor([[2.0]], dtype=F64), {"gate": one, "up": 3 * one, "down": one})
    gelu = 0.5 * 2 * (1 + math.tanh(math.sqrt(2 / math.pi) * (2 + 0.044715 * 8)))
    assert out.item() == pytest.approx(gelu * 6)
    assert plain.softcap(torch.tensor(100.0, dtype=F64), 5.0).item() == pytest.approx(5.0)


@pytest.mark.parametrize("name", ["P", "Q", "R"])
def test_prefix_and_portions_of_the_plain_model(name, tmp_path):
    config, seed = kufolorn_configs()[name]
    write_random_model(str(tmp_path), config, seed, torch.bfloat16)
    oracle = plain.PlainKufolorn.from_folder(str(tmp_path))
    p = prompt(5, 60, config.vocab)
    whole = oracle.logits(p)
    torch.testing.assert_close(whole[:25], oracle.logits(p[:25]), atol=1e-10, rtol=0)
    oracle.reset()
    parts = torch.cat([oracle.forward(p[:7]), oracle.forward(p[7:9]), oracle.forward(p[9:58]), oracle.forward(p[58:59]), oracle.forward(p[59:])])
    torch.testing.assert_close(parts, whole, atol=1e-9, rtol=0)
    assert len(oracle.after_layers) == len(config.layers)
