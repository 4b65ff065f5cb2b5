"""The Morulix configuration and model description on the CPU: config.json round trip, errors that name the key, the run
order and passes of the looped stretch, cache and state plans, the checkpoint table against the tensors a model folder
holds, and the plain implementation's own mechanisms worked out by hand."""

from __future__ import annotations

import json
import math

import pytest
import torch

from tests.helpers import morulix_configs, prompt
from tests.plain import morulix as plain
from tinyserve_llm_amd.config.llama import ConfigError
from tinyserve_llm_amd.config.morulix import MorulixConfig
from tinyserve_llm_amd.models.decoder import DecoderModel
from tinyserve_llm_amd.models.registry import architecture_of, read_config, resolve
from tinyserve_llm_amd.weights.random_init import write_random_model

F64 = torch.float64
NAMES = ["P", "Q", "R", "S", "T"]


@pytest.mark.parametrize("name", NAMES)
def test_round_trip_through_config_json(name, tmp_path):
    config, seed = morulix_configs()[name]
    raw = json.loads(json.dumps(architecture_of(config).to_dict(config)))
    assert raw["architecture"] == "Morulix" and resolve(raw).name == "Morulix"
    assert MorulixConfig.from_dict(raw) == config
    if name in "PQR":
        write_random_model(str(tmp_path), config, seed, torch.bfloat16)
        arch, again = read_config(str(tmp_path))
        assert arch.name == "Morulix" and again == config


def test_errors_name_the_key():
    config, _ = morulix_configs()["P"]
    raw = architecture_of(config).to_dict(config)

    def broken(edit):
        r = json.loads(json.dumps(raw))
        edit(r)
        return r
    for edit, word in ((lambda r: r.pop("vocab"), "vocab"), (lambda r: r["norm"].pop("eps"), "eps"),
                       (lambda r: r["layers"][0]["mixer"].pop("state"), "state"),
                       (lambda r: r["layers"][0]["mixer"].update(groups=3), "groups"),
                       (lambda r: r["layers"][0]["mixer"].update(norm_groups=7), "norm_groups"),
                       (lambda r: r["layers"][0]["mixer"].update(conv=0), "conv"),
                       (lambda r: r["layers"][1]["mixer"].update(kv_heads=3), "kv_heads"),
                       (lambda r: r["layers"][1]["mixer"]["rot"].update(dims=34), "rot"),
                       (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].pop("low"), "low"),
                       (lambda r: r["layers"][1]["mixer"]["rot"]["scaling"].update(high=0.5), "high"),
                       (lambda r: r["layers"][1]["mixer"]["mask"].update(size=0), "mask"),
                       (lambda r: r["layers"][2]["mixer"].pop("kv_rank"), "kv_rank"),
                       (lambda r: r["layers"][0]["mlp"].update(kind="moe"), "kind"),
                       (lambda r: r["layers"][0].update(type="mlstm"), "type"),
                       (lambda r: r["loop"].update(stop=9), "loop"), (lambda r: r["loop"].update(times=0), "loop"),
                       (lambda r: r["loop"].update(start=3), "loop"), (lambda r: r["loop"].pop("times"), "times")):
        with pytest.raises(ConfigError, match=word):
            MorulixConfig.from_dict(broken(edit))


def test_run_order_and_passes():
    orders = {name: morulix_configs()[name][0].run_order() for name in NAMES}
    assert orders["P"] == [(0, None), (1, 0), (2, None), (1, 1), (2, None), (1, 2), (2, None), (3, None)]
    assert orders["Q"] == [(0, 0), (1, None), (2, None), (3, None), (4, None)], "one pass still begins with its input"
    assert orders["R"] == [(0, 0), (1, None), (2, None), (0, 1), (1, None), (2, None)]
    assert orders["S"] == [(0, None), (1, 0), (1, 1), (2, None)]
    assert orders["T"] == [(0, None), (1, None), (2, None)]
    # the plain model's own list of runs says the same
    for name in NAMES:
        raw = architecture_of(morulix_configs()[name][0]).to_dict(morulix_configs()[name][0])
        assert plain.PlainMorulix(raw, {}).runs() == orders[name]


def test_plans_of_looped_layers():
    config, _ = morulix_configs()["P"]
    model = DecoderModel(architecture_of(config).build_spec(config))
    assert [r.layer for r in model.spec.order] == [0, 1, 2, 1, 2, 1, 2, 3] and len(model.layers) == 4
    assert [r.begins for r in model.spec.order] == [None, ("loop", 0), None, ("loop", 1), None, ("loop", 2), None, None]
    assert all(r.cache is None and r.store for r in model.spec.order), "every pass keeps caches and states of its own"
    assert [(e.owner, e.kv.window, e.kv.num_kv_heads, e.kv.head_dim, e.kv.v_dim) for e in model.cache_plan()] == \
        [(1, 24, 2, 32, 48), (2, 0, 1, 40, 40), (3, 24, 2, 32, 48), (4, 0, 1, 40, 40), (5, 24, 2, 32, 48), (6, 0, 1, 40, 40), (7, 24, 2, 32, 48)]
    # S in places of 32 x 32 a head, then three rows of the convolution's inputs (4 x 32 + 2 x 2 x 32 places)
    assert [(e.run, tuple(e.state.shape)) for e in model.state_plan()] == [(0, (4 * 32 * 32 + 3 * 256,))]
    assert model.graph_safe()
    config, _ = morulix_configs()["S"]
    model = DecoderModel(architecture_of(config).build_spec(config))
    assert [e.run for e in model.state_plan()] == [1, 2], "a looped state-space layer has a state for every pass"


def test_checkpoint_names_and_shapes(tmp_path):
    from safetensors import safe_open
    config, seed = morulix_configs()["P"]
    write_random_model(str(tmp_path), config, seed, torch.bfloat16)
    with safe_open(str(tmp_path / "model.safetensors"), "pt", "cpu") as f:
        shapes = {k: tuple(f.get_slice(k).get_shape()) for k in f.keys()}
    assert shapes["embed"] == (200, 80) and shapes["head"] == (200, 80) and shapes["final.norm"] == (80,)
    assert shapes["loop.in"] == (80, 160) and shapes["loop.step"] == (3, 80)
    assert shapes["l0.mix.in"] == (80 + 80 + 48 + 48 + 4, 80) and shapes["l0.mix.conv"] == (176, 4) and shapes["l0.mix.conv.b"] == (176,)
    assert shapes["l0.mix.dt_bias"] == shapes["l0.mix.A_log"] == shapes["l0.mix.D"] == (4,)
    assert shapes["l0.mix.norm"] == (80,) and shapes["l0.mix.o"] == (80, 80) and shapes["l0.norm1"] == (80,)
    assert shapes["l1.mix.q"] == (128, 80) and shapes["l1.mix.k"] == (64, 80) and shapes["l1.mix.v"] == (96, 80) and shapes["l1.mix.o"] == (80, 192)
    assert shapes["l2.mix.q"] == (72, 80) and shapes["l2.mix.dkv"] == (40, 80) and shapes["l2.mix.dkv.norm"] == (40,)
    assert shapes["l2.mix.uk"] == (72, 40) and shapes["l2.mix.uv"] == (60, 40) and shapes["l2.mix.sink"] == (3,) and shapes["l2.mix.g"] == (3, 80)
    assert shapes["l0.mlp.gate"] == shapes["l0.mlp.up"] == (96, 80) and shapes["l0.mlp.down"] == (80, 96)
    assert not any(k.endswith("norm2") or k.startswith("l3.mlp") for k in shapes), "one norm a layer; the last has no feed-forward"
    # the loader puts every tensor back where the writer took it from; the rows that fill the projections up are zeros
    from tinyserve_llm_amd.weights.loader import load_params
    model = DecoderModel(architecture_of(config).build_spec(config))
    params = load_params(model, str(tmp_path), torch.bfloat16, "cpu")
    model.bind(params, torch.bfloat16, torch.device("cpu"))
    with safe_open(str(tmp_path / "model.safetensors"), "pt", "cpu") as f:
        down = params["layers.2.mixer.down"]
        assert down.shape == (120, 80) and float(down[115:].abs().max()) == 0.0
        assert torch.equal(down[72:112], f.get_tensor("l2.mix.dkv")) and torch.equal(down[112:115], f.get_tensor("l2.mix.g"))
        assert torch.equal(params["layers.0.mixer.proj"][:260], f.get_tensor("l0.mix.in")) and params["layers.0.mixer.proj"].shape == (264, 80)
        assert float(params["layers.0.mixer.proj"][260:].abs().max()) == 0.0
        assert torch.equal(params["layers.0.mixer.skip"], f.get_tensor("l0.mix.D").float())
        assert torch.equal(params["pass_inputs.loop.step"][1], f.get_tensor("loop.step")[1])
        # the convolution's weights, taps first, in the places that the kernels work on: x of 4 heads, B and C of 2 groups
        w = f.get_tensor("l0.mix.conv").float()
        conv, bias = model.layers[0].mixer._conv
        assert conv.shape == (4, 256) and bias.shape == (256,)
        assert torch.equal(conv[:, 32:52], w[20:40].t()) and torch.equal(conv[:, 160:184], w[80 + 24:80 + 48].t())
        assert torch.equal(conv[:, 224:248], w[152:176].t()) and float(conv[:, 52:64].abs().max()) == 0.0
        assert torch.equal(bias[192:216], f.get_tensor("l0.mix.conv.b").float()[128:152])


def test_a_run_that_begins_a_pass_needs_its_part():
    from dataclasses import replace
    config, _ = morulix_configs()["P"]
    spec = architecture_of(config).build_spec(config)
    spec.order[1] = replace(spec.order[1], begins=("loop", 3))
    with pytest.raises(ValueError, match="begins pass"):
        DecoderModel(spec)
    spec = architecture_of(config).build_spec(config)
    spec.pass_inputs = {}
    with pytest.raises(ValueError, match="begins pass"):
        DecoderModel(spec)


def test_the_engines_frequencies_are_the_plain_ones():
    from tinyserve_llm_amd.parts.rope import RotaryFrequencies, inverse_frequencies
    for dims, base, bands in ((16, 10000.0, dict(factor=3.0, low=1.0, high=4.0, original=64.0)), (10, 50000.0, dict(factor=8.0, low=0.5, high=2.0, original=32.0)),
                              (64, 500000.0, dict(factor=32.0, low=1.0, high=4.0, original=8192.0)), (8, 300.0, dict(factor=2.0, low=2.0, high=2.0, original=100.0)),
                              (12, 900.0, None)):
        f = RotaryFrequencies(dims, base, False, bands=bands).host_frequencies()
        want = torch.tensor(plain.banded_frequencies(dims, base, bands), dtype=F64)
        torch.testing.assert_close(f, want, atol=0, rtol=1e-13)
    with pytest.raises(ValueError):
        RotaryFrequencies(8, 300.0, False, ramp=dict(factor=2.0, original=64.0, fast=8.0, slow=2.0), bands=dict(factor=2.0, low=1.0, high=4.0, original=64.0))


# ---- the plain implementation's mechanisms by hand ------------------------------------------------

def test_frequency_bands_by_hand():
    # dims 8, base 16: f = 1, 1/2, 1/4, 1/8; over L = 2 pi 8 positions the pairs make 8, 4, 2, 1 turns
    L = 2 * math.pi * 8
    f = plain.banded_frequencies(8, 16.0, dict(factor=4.0, low=1.5, high=3.0, original=L))
    # more than 3 turns: kept; less than 1.5: a quarter; 2 turns: a third of the way up
    assert f == pytest.approx([1.0, 0.5, 0.25 * ((1 - 1 / 3) / 4 + 1 / 3), 0.125 / 4])
    assert plain.banded_frequencies(8, 16.0, None) == pytest.approx([1.0, 0.5, 0.25, 0.125])


def test_halves_turn_and_the_rest_passes():
    x = torch.tensor([[[1.0, 0.0, 0.0, 1.0, 5.0]]], dtype=F64)
    # pairs (0, 2) and (1, 3) at position 2: (1, 0) half a turn -> (-1, 0); (0, 1) a whole turn
    out = plain.rotate_halves(x, torch.tensor([2]), [math.pi / 2, math.pi])
    assert out[0, 0].tolist() == pytest.approx([-1.0, 0.0, 0.0, 1.0, 5.0])


def test_window_and_sink_by_hand():
    # keys that all score 0, values 1, 2, ...: equal weights over what is seen; a sink of ln 2 counts as two more
    n = 6
    q, k = torch.zeros(n, 1, 2, dtype=F64), torch.zeros(n, 1, 2, dtype=F64)
    v = torch.arange(1, n + 1, dtype=F64).view(n, 1, 1)
    out = plain.softmax_attention(q, k, v, torch.arange(n), 1.0, window=2)
    assert out[:, 0, 0].tolist() == pytest.approx([1.0, 1.5, 2.5, 3.5, 4.5, 5.5])
    out = plain.softmax_attention(q, k, v, torch.arange(n), 1.0, sinks=torch.tensor([math.log(2.0)], dtype=F64))
    assert out[:, 0, 0].tolist() == pytest.approx([1 / 3, 3 / 4, 6 / 5, 10 / 6, 15 / 7, 21 / 8])


def test_convolution_by_hand():
    u = torch.tensor([[1.0], [2.0], [3.0]], dtype=F64)
    w, b = torch.tensor([[10.0, 1.0, 0.1]], dtype=F64), torch.tensor([0.5], dtype=F64)
    silu = lambda z: z / (1 + math.exp(-z))
    out = plain.convolve(u, w, b, torch.zeros(2, 1, dtype=F64))
    assert out[:, 0].tolist() == pytest.approx([silu(0.6), silu(1.7), silu(12.8)])
    out = plain.convolve(u[:1], w, b, torch.tensor([[7.0], [5.0]], dtype=F64))
    assert out[0, 0].item() == pytest.approx(silu(70 + 5 + 0.1 + 0.5))


def test_state_space_by_hand():
    # two heads of one channel with a group each, one state row; A = -1 and -3
    x = torch.tensor([[[2.0], [1.0]], [[4.0], [1.0]]], dtype=F64)
    B = torch.tensor([[[3.0], [1.0]], [[1.0], [1.0]]], dtype=F64)
    C = torch.tensor([[[1.0], [5.0]], [[10.0], [1.0]]], dtype=F64)
    dt = torch.tensor([[0.5, 1.0], [math.log(2.0), 1.0]], dtype=F64)
    y, S = plain.state_space(x, B, C, dt, torch.tensor([0.0, math.log(3.0)], dtype=F64), torch.tensor([0.25, 0.0], dtype=F64),
                             torch.zeros(2, 1, 1, dtype=F64))
    # head 0: S = 0.5 3 2 = 3, then e^(-ln 2) 3 + ln 2 4; head 1: 1, then e^-3 + 1
    second = 1.5 + 4 * math.log(2.0)
    assert y[:, 0, 0].tolist() == pytest.approx([3 + 0.5, 10 * second + 1.0])
    assert y[:, 1, 0].tolist() == pytest.approx([5.0, math.exp(-3) + 1])
    assert S[0, 0, 0].item() == pytest.approx(second)
    # one group: both heads read its B and C
    y, _ = plain.state_space(x[:1], B[:1, :1], C[:1, :1], dt[:1], torch.zeros(2, dtype=F64), torch.zeros(2, dtype=F64), torch.zeros(2, 1, 1, dtype=F64))
    assert y[0, :, 0].tolist() == pytest.approx([0.5 * 3 * 2, 3.0])


def test_gate_before_a_norm_in_parts():
    y, z = torch.tensor([[3.0, 4.0, 5.0, 5.0]], dtype=F64), torch.tensor([[50.0, 50.0, 50.0, -50.0]], dtype=F64)
    out = plain.gated_group_norm(y, z, torch.tensor([1.0, 1.0, 2.0, 1.0], dtype=F64), 2, 0.0)
    rms = math.sqrt(12.5)
    assert out[0].tolist() == pytest.approx([3 / rms, 4 / rms, 2 * math.sqrt(2.0), 0.0], abs=1e-12)


def test_pass_input_by_hand():
    w = torch.tensor([[1.0, 0.0, 10.0, 0.0], [0.0, 1.0, 0.0, -1.0]], dtype=F64)
    out = plain.pass_input(torch.tensor([[1.0, 2.0]], dtype=F64), torch.tensor([[3.0, 4.0]], dtype=F64), w, torch.tensor([0.5, 0.25], dtype=F64))
    assert out.tolist() == [[31.5, -1.75]]


@pytest.mark.parametrize("name", ["P", "Q", "R"])
def test_prefix_and_portions_of_the_plain_model(name, tmp_path):
    config, seed = morulix_configs()[name]
    write_random_model(str(tmp_path), config, seed, torch.bfloat16)
    oracle = plain.PlainMorulix.from_folder(str(tmp_path))
    p = prompt(5, 60, config.vocab)
    whole = oracle.logits(p)
    torch.testing.assert_close(whole[:25], oracle.logits(p[:25]), atol=1e-10, rtol=0)
    oracle.reset()
    parts = torch.cat([oracle.forward(p[:7]), oracle.forward(p[7:9]), oracle.forward(p[9:58]), oracle.forward(p[58:59]), oracle.forward(p[59:])])
    torch.testing.assert_close(parts, whole, atol=1e-9, rtol=0)
    assert len(oracle.after_layers) == len(config.run_order())
