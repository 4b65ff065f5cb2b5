"""The Kufolorn decoder on the GPU against the plain implementation in tests/plain/kufolorn.py: each mechanism's kernel
alone (with inputs made so that a fault shows: a far key whose score stands out, keys at page borders, the first tokens
where a sink weighs most, keys that are written over, a state that is to be read out hundreds of tokens after it was
written, states and convolution inputs carried over steps and slots, choice scores that are all negative), then whole models
of five small configurations through trace replay (layer by layer, whole, token by token, in portions down to two tokens,
mixed batches on pages and state slots that are used again, long decoding), and greedy generation through `LLM.generate` and
the scheduler. float32 and bfloat16."""

from __future__ import annotations

import pytest
import torch

from tests.helpers import kufolorn_configs, prompt
from tests.plain import kufolorn as plain
from tests.test_gpu_fanotar import paged, rounded, step_context, tolerance

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16]


def hip():
    from tinyserve_llm_amd.ops import hip as h
    return h


# ---- the stream: rows as they are, norms on the way in; capped logits; the dense unit -------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [80, 99, 256, 2048, 4100])
def test_rows_leave_the_stream_as_they_are_and_branches_enter_it_normed(dtype, width):
    from tinyserve_llm_amd.parts.norm import RMSNorm
    from tinyserve_llm_amd.parts.stream import ResidualStream
    n, eps = 7, 1e-5
    x, a, b = torch.randn(n, width) * 3, torch.randn(n, width) * 5, torch.randn(n, width) * 1e-3
    norm = RMSNorm(width, eps, one_plus=True)
    w, w64 = rounded(torch.randn(width) * 0.3, dtype)
    norm.bind({"weight": w})
    stream = ResidualStream(x.to(DEV))
    got, rows = stream.rows_as(dtype)
    assert torch.equal(got.cpu(), x) and torch.equal(rows.cpu(), x.to(dtype)), "nothing is pending: the rows themselves"
    want = x.to(F64)
    for branch in (a, b):                                                    # (a branch so small that eps counts)
        got, rows = ResidualStream(got, branch.to(DEV), post=norm).rows_as(dtype)
        want = want + plain.layer_norm(branch.to(F64), w64, eps)
        torch.testing.assert_close(got.cpu().to(F64), want, atol=3e-6, rtol=1e-6)
        assert torch.equal(rows, got.to(dtype))
    # the model's last norm takes picked rows of a stream with a branch pending
    last = RMSNorm(width, eps, one_plus=True)
    last.bind({"weight": w})
    picked, _ = last(ResidualStream(got, a.to(DEV), post=norm), None, torch.tensor([5, 0], dtype=torch.int32, device=DEV))
    want = want + plain.layer_norm(a.to(F64), w64, eps)
    torch.testing.assert_close(picked.cpu().to(F64), plain.layer_norm(want, w64, eps)[[5, 0]], **tolerance(dtype))


@pytest.mark.parametrize("shape", [(1, 5), (3, 77), (7, 640), (2, 40001)])
def test_capped_logits(shape):
    h = hip()
    x = torch.randn(shape) * 40
    x.view(-1)[0], x.view(-1)[-1] = 1e4, -3e-5
    got = h.soft_cap(x.to(DEV), 12.5)
    torch.testing.assert_close(got.cpu().to(F64), plain.softcap(x.to(F64), 12.5), atol=1e-9, rtol=2e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("ff", [52, 53, 640])
def test_gelu_gated_unit(dtype, ff):
    h = hip()
    sums = torch.randn(9, 2 * ff + 4) * 3
    sums[0, :8] = torch.tensor([-60.0, -8.0, -1e-4, 0.0, 1e-4, 3.0, 8.0, 60.0])
    want = plain.gelu_tanh(sums[:, :ff].to(F64)) * sums[:, ff:2 * ff].to(F64)
    tol = dict(atol=1e-5, rtol=1e-5) if dtype == torch.float32 else dict(atol=1e-5, rtol=5e-3)
    torch.testing.assert_close(h.capped_glu(sums.to(DEV)[:, :2 * ff].contiguous(), 0.0, 1.0, 0.0, dtype, activation="gelu_tanh").cpu().to(F64), want, **tol)
    torch.testing.assert_close(h.capped_glu(sums.to(DEV)[:, :2 * ff], 0.0, 1.0, 0.0, dtype, activation="gelu_tanh").cpu().to(F64), want, **tol)
    # with caps the gelu takes the capped gate
    want = plain.gelu_tanh(sums[:, :ff].to(F64).clamp(max=0.7)) * (sums[:, ff:2 * ff].to(F64).clamp(-0.7, 0.7) + 1)
    torch.testing.assert_close(h.capped_glu(sums.to(DEV)[:, :2 * ff].contiguous(), 0.7, 1.0, 1.0, dtype, activation="gelu_tanh").cpu().to(F64), want, **tol)


# ---- the router: groups ------------------------------------------------------------------------------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("experts, groups, keep, top", [(9, 3, 2, 4), (9, 3, 1, 3), (12, 6, 3, 2), (6, 1, 1, 6), (64, 8, 4, 8), (128, 64, 5, 10),
                                                        (10, 5, 5, 10), (96, 3, 1, 32), (7, 7, 3, 3)])
@pytest.mark.parametrize("shift", [0.0, -3.0, 2.0])
def test_experts_are_chosen_inside_the_best_groups(dtype, experts, groups, keep, top, shift):
    """`shift` moves every choice score: below zero for all (a group left out is not in the running with a score of 0) or
    above; weights are the softmax's, without the correction and not over their sum."""
    h = hip()
    gen = torch.Generator().manual_seed(experts + groups)
    x, x64 = rounded(torch.randn(21, 72, generator=gen), dtype)
    router = torch.randn(experts, 72, generator=gen) * 0.25
    correction = torch.randn(experts, generator=gen) * 0.1 + shift
    ids, weights = h.moe_route(x, router.to(DEV), correction.to(DEV), top, 1.0, normalize=False, softmax_all=True, groups=(groups, keep))
    kept_out = 0
    for t in range(21):
        want, s = plain.choose(router.to(F64) @ x64[t], correction.to(F64), top, groups, keep)
        assert ids[t].tolist() == want
        torch.testing.assert_close(weights[t].cpu().to(F64), torch.tensor(s, dtype=F64), atol=1e-7, rtol=1e-5)
        kept_out += want != plain.choose(router.to(F64) @ x64[t], correction.to(F64), top, 1, 1)[0]
    assert keep >= min(groups, top) or kept_out, "the groups decided something"


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_mixture_with_groups_and_identity_experts(dtype):
    from tinyserve_llm_amd.parts.moe import RoutedExperts
    W, F, E, I = 64, 48, 7, 5
    part = RoutedExperts(W, E, 4, F, limit=0.9, slope=1.702, up_shift=1.0, normalize=False, scoring="softmax_all", identity=I, groups=(4, 3))
    gen = torch.Generator().manual_seed(2)
    params = {n: (torch.randn(s.shape, generator=gen) * (s.shape[-1] ** -0.5 if len(s.shape) == 3 else 0.4)).to(torch.float32 if s.storage == "float32" else dtype)
              for n, s in part.param_specs().items()}
    part.bind({n: t.to(DEV) for n, t in params.items()})
    p64 = {n: t.to(F64) for n, t in params.items()}
    Wt = {"router": p64["router"], "correction": p64["correction"]}
    for e in range(E):
        Wt.update({f"e{e}.gate": p64["gate_up"][e, :F], f"e{e}.up": p64["gate_up"][e, F:], f"e{e}.down": p64["down"][e]})
    c = {"router": {"experts": E, "top": 4, "groups": {"count": 4, "keep": 3}}, "expert": {"limit": 0.9}}
    for T in (1, 5, 70):
        x, x64 = rounded(torch.randn(T, W, generator=gen) * 2, dtype)
        want = plain.experts_unit(x64, Wt, c)
        tol = 2e-5 if dtype == torch.float32 else 1e-2
        torch.testing.assert_close(part.forward(x, None).cpu().to(F64), want, atol=tol * float(want.abs().max()), rtol=tol)


# ---- attention with a learned sink and a gate per head; biases and norms over whole projections ---------

@pytest.mark.parametrize("sizes", [(128, 64, 96), (60, 20, 12), (1500, 300, 77), (4096, 1024, 1024), (5000, 40, 8)])
def test_biases_and_norms_over_whole_projections(sizes):
    h = hip()
    q, k, v = sizes
    x, b = torch.randn(5, q + k + v + 6) * 2, torch.randn(q + k + v) * 0.7
    wq, wk = 1 + torch.randn(q) * 0.2, 1 + torch.randn(k) * 0.2
    x[2] *= 1e-4
    d = x.to(DEV)
    h.segment_rmsnorm_pair(d, (0, q, wq.to(DEV)), (q, k, wk.to(DEV)), 1e-5, bias=b.to(DEV), rest=(q + k, v))
    s = x.to(F64)
    s[:, :q + k + v] += b.to(F64)
    want = torch.cat([plain.unit_rms(s[:, :q], 1e-5) * wq.to(F64), plain.unit_rms(s[:, q:q + k], 1e-5) * wk.to(F64), s[:, q + k:]], 1)
    torch.testing.assert_close(d.cpu().to(F64), want, atol=3e-6, rtol=3e-6)
    # without biases the third stretch stays
    d = x.to(DEV)
    h.segment_rmsnorm_pair(d, (0, q, wq.to(DEV)), (q, k, wk.to(DEV)), 1e-5)
    s = x.to(F64)
    want = torch.cat([plain.unit_rms(s[:, :q], 1e-5) * wq.to(F64), plain.unit_rms(s[:, q:q + k], 1e-5) * wk.to(F64), s[:, q + k:]], 1)
    torch.testing.assert_close(d.cpu().to(F64), want, atol=3e-6, rtol=3e-6)


FORMS = {"decoded": None, "prompt": 0, "portion": 130}       # (a portion that starts inside a page)


def decides(want_row, value_row) -> bool:
    return float((want_row - value_row).abs().max()) < 0.2 * float(value_row.abs().max())


def sink_case(dtype, H, G, D, V, page, length, queries, stand_out, portion_from, sinks, gated, seed=5):
    """One request of `length` tokens on shuffled pages; queries as decoded tokens over the same pages, or every position
    from `portion_from` on as one portion. Queries and keys of unit size; a query's score for the key it is to find stands
    out at 11. Returns (kernel output, oracle output, values, query positions)."""
    h = hip()
    if portion_from is not None:
        queries = list(range(portion_from, length))
        stand_out = {q: key for q, key in stand_out.items() if q >= portion_from}
    gen = torch.Generator().manual_seed(seed)
    scale = D ** -0.5
    k64 = plain.unit_rms(torch.randn(length, G, D, generator=gen, dtype=F64), 0.0)
    q64 = plain.unit_rms(torch.randn(len(queries), H, D, generator=gen, dtype=F64), 0.0)
    for i, p in enumerate(queries):
        if p in stand_out:
            g_dir = plain.unit_rms(torch.randn(G, D, generator=gen, dtype=F64), 0.0)
            q64[i] = g_dir[torch.arange(H) // (H // G)]
            k64[stand_out[p]] = 11.0 / (D * scale) * g_dir
    v64 = torch.randn(length, G, V, generator=gen, dtype=F64)
    pages = -(-length // page)
    table = torch.randperm(pages + 3, generator=gen)[:pages].tolist()
    k, v = paged(pages + 3, page, G, D, V, dtype)
    kr, vr = k64.to(dtype), v64.to(dtype)
    at = torch.arange(length)
    pg, off = torch.tensor(table)[at // page].to(DEV), (at % page).to(DEV)
    k[pg, off], v[pg, off] = kr.to(DEV), vr.to(DEV)
    q = q64.to(dtype).to(DEV)
    wide = torch.randn(len(queries), H + 5, generator=gen) * 2                # (the gate's numbers are columns of wider rows)
    ctx = step_context([table] * len(queries), page, queries, [1] * len(queries)) if portion_from is None else \
        step_context([table], page, [portion_from], [len(queries)])
    out = h.paged_attention(q, k, v, ctx, 0, scale, sinks=sinks.float().to(DEV), gate=wide.to(DEV)[:, 2:2 + H] if gated else None)
    want = plain.sink_attention(q.cpu().to(F64), kr.to(F64), vr.to(F64), torch.tensor(queries), scale, sinks.to(F64))
    if gated:
        want = want * torch.sigmoid(wide[:, 2:2 + H].to(F64))[:, :, None]
    return out.cpu().to(F64).view(len(queries), H, V), want, vr.to(F64), queries


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sizes", [(2, 2, 16, 16), (4, 2, 32, 48), (8, 2, 64, 64), (3, 1, 20, 12), (10, 5, 48, 48), (4, 1, 96, 96), (8, 4, 128, 128),
                                   (16, 2, 32, 32), (4, 4, 64, 1)])
def test_sinks_and_gates_with_far_keys(dtype, sizes, form):
    """Far keys and keys at page borders stand out for their queries and decide their rows, beside a sink per head that
    differs from head to head; a gate per head multiplies whole heads, in every kernel that writes them (decoded tokens'
    keys cut into chunks that a second kernel adds up too)."""
    H, G, D, V = sizes
    stand_out = {699: 3, 650: 15, 651: 16, 652: 31, 653: 32, 654: 33, 655: 655, 500: 255, 501: 256, 33: 0}
    queries = [0, 1, 2, 3, 15, 16, 31, 32, 33, 500, 501, 650, 651, 652, 653, 654, 655, 699]
    sinks = torch.linspace(-3.0, 4.0, H)
    out, want, v, qs = sink_case(dtype, H, G, D, V, 32, 700, queries, stand_out, FORMS[form], sinks, True)
    torch.testing.assert_close(out, want, **tolerance(dtype))
    out, want, v, qs = sink_case(dtype, H, G, D, V, 32, 700, queries, stand_out, FORMS[form], torch.full((H,), -5.0), False)
    torch.testing.assert_close(out, want, **tolerance(dtype))
    for q, key in ((699, 3), (653, 32)):
        assert decides(want[qs.index(q), 0], v[key, 0]), "the far key decides the row"


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("D", [48, 64])
def test_a_sink_takes_its_share_and_no_more(dtype, D, form):
    """A sink far above every score takes nearly everything, one far below nothing, whatever their distance (no overflow)."""
    for value in (300.0, 6.0, 0.0, -40.0, -300.0):
        out, want, v, qs = sink_case(dtype, 4, 2, D, D, 32, 300, [0, 1, 2, 31, 32, 299], {}, FORMS[form], torch.full((4,), value), False)
        torch.testing.assert_close(out, want, **tolerance(dtype))
        if value >= 300:
            assert float(out.abs().max()) < 1e-6
        if value <= -300 and qs[0] == 0:
            torch.testing.assert_close(out[0, 0], v[0, 0], **tolerance(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("layer", ["P1", "Q0", "Q2", "R1", "S0", "T1", "T3"])
def test_whole_attention_mixer(dtype, layer):
    from tinyserve_llm_amd.models.kufolorn import _encoding
    from tinyserve_llm_amd.parts.attention import GeneralAttention
    from tinyserve_llm_amd.parts.base import LayerMemory, make
    config = kufolorn_configs()[layer[0]][0]
    m, eps = config.layers[int(layer[1])].mixer.left, config.norm_eps
    encodings = {}
    name = _encoding(encodings, m.rot)
    part = GeneralAttention(config.width, m.heads, m.kv_heads, m.dim, m.vdim, position=name, scale=m.scale, learned_sink=True,
                            projection_norm_eps=eps, head_gate=True, bias=True)
    gen = torch.Generator().manual_seed(4)
    params = {n: torch.randn(s.shape, generator=gen) * (s.shape[1] ** -0.5 if len(s.shape) == 2 else s.init[1] * 3) + (s.init[0] if len(s.shape) == 1 else 0)
              for n, s in part.param_specs().items()}
    params = {n: t.to(torch.float32 if part.param_specs()[n].storage == "float32" else dtype) for n, t in params.items()}
    part.bind({n: t.to(DEV) for n, t in params.items()})
    W = {n: t.to(F64) for n, t in params.items()}
    cut = [m.heads * m.dim, m.kv_heads * m.dim, m.kv_heads * m.vdim]
    q, k, v, g = W["qkv"][:sum(cut) + m.heads].split(cut + [m.heads])
    qb, kb, vb = W["qkv_bias"].split(cut)
    W = {"q": q, "k": k, "v": v, "g": g, "q.b": qb, "k.b": kb, "v.b": vb, "q.norm": W["q_norm"], "k.norm": W["k_norm"], "sink": W["sinks"], "o": W["o"]}
    x, x64 = rounded(torch.randn(170, config.width, generator=gen), dtype)
    kc, vc = paged(7, 32, m.kv_heads, m.dim, m.vdim, dtype)
    mem, past, out, want = LayerMemory(kc, vc), {}, [], []
    encs = {n: make("position_encoding", ps) for n, ps in encodings.items()}
    for e in encs.values():
        e.prepare(DEV)
    raw = config.to_dict()["layers"][int(layer[1])]["mixer"]["left"]
    for a, b in ((0, 1), (1, 3), (3, 100), (100, 101), (101, 170)):
        ctx = step_context([[5, 1, 6, 0, 2, 4]], 32, [a], [b - a])
        ctx.position_encodings = encs
        out.append(part.forward(x[a:b], ctx, mem))
        want.append(plain.left_attention(x64[a:b], torch.arange(a, b), W, raw, eps, past))
    want = torch.cat(want)
    tol = 3e-5 if dtype == torch.float32 else 3e-2
    torch.testing.assert_close(torch.cat(out).cpu().to(F64), want, atol=tol * float(want.abs().max()), rtol=tol)


# ---- retention: between projection and recurrence, the recurrence with fixed decays, the whole mixer ------

def packed_steps(lengths, portions, slots):
    """Steps that feed the requests' rows in changing portions until all are through: (request, first row, rows) lists."""
    cursors, tick = [0] * len(lengths), 0
    while any(c < n for c, n in zip(cursors, lengths)):
        live = [i for i in range(len(lengths)) if cursors[i] < lengths[i]]
        step = [(i, cursors[i], min(portions[(tick + 2 * i) % len(portions)], lengths[i] - cursors[i])) for i in live]
        tick += 1
        for i, _, n in step:
            cursors[i] += n
        yield step, step_context([[0]] * len(step), 1 << 20, [a for _, a, _ in step], [n for _, _, n in step], slots=[slots[i] for i, _, _ in step])


PORTIONS = {"few": [1, 2, 13, 1, 5, 3], "long beside single": [70, 1, 1, 2, 33], "whole": [400], "two": [2]}
RETENTION_SIZES = {"odd": (3, 37, 13, 10), "even": (4, 24, 20, 16), "one": (1, 16, 16, 16), "plain": (8, 64, 64, 64), "large": (4, 160, 80, 96),
                   "still": (2, 32, 16, 0), "tiny": (2, 2, 1, 2), "tall": (2, 300, 16, 40)}        # heads, dim, vdim, dims that turn


def retention_setup(kind):
    h = hip()
    H, D, V, rot = RETENTION_SIZES[kind]
    decay = torch.tensor([[0.999], [0.0, 0.999], [0.9, 0.5, 1.0]][H - 1] if H < 4 else [0.9995, 0.99, 0.9, 0.5, 0.97, 0.998, 0.0, 1.0][:H], dtype=F64)
    z = h.SsdSizes(H, V, H, D, 1)
    dev = [t.float().to(DEV) for t in (torch.full((H,), D ** -0.5), torch.log(decay), decay)]
    return z, decay, dict(zip(("steps", "logs", "keeps"), dev)), rot, torch.Generator().manual_seed(7)


@pytest.mark.parametrize("kind", sorted(RETENTION_SIZES))
@pytest.mark.parametrize("tokens", [1, 5, 300])
@pytest.mark.parametrize("dtype", DTYPES)
def test_what_lies_between_projection_and_retention(dtype, tokens, kind):
    h = hip()
    z, _, _, rot, gen = retention_setup(kind)
    proj = torch.randn(tokens, -(-(z.channels + 5) // 8) * 8, generator=gen) * 2
    positions = torch.randint(0, 100000, (tokens,), generator=gen)
    positions[0] = 99999
    freqs = torch.tensor([3000.0 ** (-2.0 * i / rot) for i in range(rot // 2)], dtype=F64) if rot else None
    got = h.retention_prepare(proj.to(DEV), None if freqs is None else freqs.to(DEV), positions.int().to(DEV), z, dtype)
    v, k, q = proj[:, :z.channels].to(F64).split([z.inner, z.heads * z.state, z.heads * z.state], 1)
    turned = [plain.rotate_halves(t.reshape(tokens, z.heads, z.state), positions, {"dims": rot, "base": 3000.0}).reshape(tokens, -1) for t in (k, q)]
    want = z.spread(torch.cat([v, *turned], 1).t().contiguous()).t()
    tol = dict(atol=2e-6, rtol=1e-6) if dtype == torch.float32 else dict(atol=2e-6, rtol=5e-3)
    torch.testing.assert_close(got.cpu().to(F64), want, **tol)
    assert torch.equal(got.cpu()[:, :z.heads * z.vp], want[:, :z.heads * z.vp].to(dtype)), "values pass"


@pytest.mark.parametrize("portions", sorted(PORTIONS))
@pytest.mark.parametrize("kind", sorted(RETENTION_SIZES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_retention_over_steps_and_slots(dtype, kind, portions):
    """Four requests of unequal length in packed steps of changing portions, each with its state in a slot of its own among
    slots that hold other requests' leftovers; decays from 0 (nothing is kept) to 1 (nothing is lost)."""
    h = hip()
    z, decay, dev, _, gen = retention_setup(kind)
    lengths, slots = [37, 1, 90, 280], [4, 0, 2, 5]
    rows = [z.spread(torch.randn(z.channels, n, generator=gen) * 0.8).t().contiguous().to(dtype) for n in lengths]
    state = torch.randn(6, z.matrix, device=DEV)
    before = state.clone()
    state[slots] = 0.0
    got = [[] for _ in lengths]
    for step, ctx in packed_steps(lengths, PORTIONS[portions], slots):
        y = h.ssd_scan(torch.cat([rows[i][a:a + n] for i, a, n in step]).to(DEV), dev["steps"], dev["logs"], None, state, ctx, z, keeps=dev["keeps"])
        at = 0
        for i, _, n in step:
            got[i].append(y[at:at + n])
            at += n
    for i, n in enumerate(lengths):
        m, at = rows[i].to(F64), z.heads * z.vp
        v = m[:, :at].view(n, z.heads, z.vp)[:, :, :z.vdim]
        k, q = (m[:, at + j * z.heads * z.np:at + (j + 1) * z.heads * z.np].view(n, z.heads, z.np)[:, :, :z.state] for j in range(2))
        want, S = plain.retention_rule(q, k * z.state ** -0.5, v, decay, torch.zeros(z.heads, z.state, z.vdim, dtype=F64))
        size = max(1.0, float(want.abs().max()))
        torch.testing.assert_close(torch.cat(got[i]).cpu().to(F64), want.reshape(n, -1), atol=3e-5 * size, rtol=3e-5)
        left = state[slots[i]].cpu().to(F64).view(z.heads, z.vp, z.np)
        torch.testing.assert_close(left[:, :z.vdim, :z.state], S.transpose(1, 2), atol=3e-5 * max(1.0, float(S.abs().max())), rtol=3e-5)
        assert float(left[:, z.vdim:].abs().sum()) == 0.0 and float(left[:, :, z.state:].abs().sum()) == 0.0, "places of no number stay zero"
    assert torch.equal(state[[1, 3]], before[[1, 3]])


def test_a_fixed_decay_is_multiplied_by_as_it_is():
    """Thousands of tokens that only decay: what is left of the state is decay^n, not a rounded logarithm's exponential."""
    h = hip()
    z = h.SsdSizes(2, 16, 2, 32, 1)
    decay = torch.tensor([1.0 - 2.0 ** -11, 0.9999], dtype=torch.float32)
    n = 3000
    rows = torch.zeros(n, z.row)
    rows[0, :2 * 16] = 1.0
    rows[0, 32:32 + 64] = 1.0                                                  # (k of both heads)
    state = torch.zeros(1, z.matrix, device=DEV)
    ctx = step_context([[0]], 1 << 20, [0], [n])
    h.ssd_scan(rows.to(DEV), torch.ones(2, device=DEV), torch.log(decay.double()).float().to(DEV), None, state, ctx, z, keeps=decay.to(DEV))
    got = state[0].view(2, 16, 32)[:, 0, 0].cpu().to(F64)
    torch.testing.assert_close(got, decay.to(F64) ** (n - 1), atol=0, rtol=3e-5)


@pytest.mark.parametrize("layer", ["P1", "Q0", "Q2", "R1", "S0", "T1", "T3"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_whole_retention_mixer(dtype, layer):
    from tinyserve_llm_amd.models.kufolorn import _encoding
    from tinyserve_llm_amd.parts.base import LayerMemory, make
    from tinyserve_llm_amd.parts.retention import Retention
    config = kufolorn_configs()[layer[0]][0]
    m = config.layers[int(layer[1])].mixer.right
    encodings = {}
    part = Retention(config.width, m.heads, m.dim, m.vdim, m.decay, config.norm_eps, position=_encoding(encodings, m.rot))
    z, gen = part.sizes, torch.Generator().manual_seed(9)
    params = {n: (torch.randn(s.shape, generator=gen) * s.shape[1] ** -0.5).to(dtype) for n, s in part.param_specs().items()}
    part.bind({n: t.to(DEV) for n, t in params.items()})
    keys = m.heads * m.dim
    v, k, q, g = params["proj"][:part.projected].to(F64).split([z.inner, keys, keys, z.inner])
    W = {"q": q, "k": k, "v": v, "g": g, "o": params["o"].to(F64)}
    x, x64 = rounded(torch.randn(150, config.width, generator=gen), dtype)
    mem = LayerMemory(state=torch.zeros(2, *part.state_spec().shape, device=DEV))
    encs = {n: make("position_encoding", ps) for n, ps in encodings.items()}
    for e in encs.values():
        e.prepare(DEV)
    raw = config.to_dict()["layers"][int(layer[1])]["mixer"]["right"]
    st, out, want = {}, [], []
    for a, b in ((0, 1), (1, 3), (3, 100), (100, 101), (101, 150)):
        ctx = step_context([[0]], 1 << 20, [a], [b - a], slots=[1])
        ctx.position_encodings = encs
        out.append(part.forward(x[a:b], ctx, mem))
        want.append(plain.retention(x64[a:b], torch.arange(a, b), W, raw, config.norm_eps, st))
    want = torch.cat(want)
    tol = 5e-5 if dtype == torch.float32 else 2e-2
    torch.testing.assert_close(torch.cat(out).cpu().to(F64), want, atol=tol * float(want.abs().max()), rtol=tol)


# ---- the gated delta rule: convolutions, unit factors, steps and decays; the recurrence; the whole mixer ---

DELTA_SIZES = {"odd": (3, 13, 1, 37, 6), "small": (4, 20, 2, 24, 4), "one": (1, 16, 1, 16, 2), "plain": (8, 64, 4, 64, 4), "long keys": (4, 64, 4, 128, 4),
               "large": (4, 80, 2, 160, 3), "no taps": (6, 8, 6, 32, 1), "tiny": (2, 1, 1, 1, 3), "many taps": (2, 24, 2, 40, 9), "tall": (2, 16, 1, 300, 4),
               "widest in chunks": (2, 48, 1, 256, 4)}                          # heads, vdim, groups, dim, taps


def delta_setup(kind, seed=1):
    h = hip()
    H, V, G, D, taps = DELTA_SIZES[kind]
    z = h.SsdSizes(H, V, G, D, taps)
    gen = torch.Generator().manual_seed(seed)
    W = {"conv": torch.randn(z.channels, taps, generator=gen) * 0.7, "dt_bias": torch.randn(H, generator=gen) - 1.0, "A_log": torch.randn(H, generator=gen) * 0.7}
    dev = dict(conv=z.spread(W["conv"]).t().contiguous().to(DEV), dt_bias=W["dt_bias"].to(DEV), a_log=W["A_log"].to(DEV))
    return z, {k: v.to(F64) for k, v in W.items()}, dev, gen


@pytest.mark.parametrize("portions", sorted(PORTIONS))
@pytest.mark.parametrize("kind", sorted(DELTA_SIZES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_convolutions_and_factors_over_steps_and_slots(dtype, kind, portions):
    h = hip()
    z, W, dev, gen = delta_setup(kind)
    lengths, slots = [37, 1, 90, 280], [4, 0, 2, 5]
    rows = [torch.randn(n, z.projected + z.heads + 3, generator=gen) * 1.5 for n in lengths]      # (columns behind: not its business)
    state = torch.randn(6, z.matrix + z.kept, device=DEV)
    before = state.clone()
    state[slots, z.matrix:] = 0.0
    got = [[] for _ in lengths]
    for step, ctx in packed_steps(lengths, PORTIONS[portions], slots):
        proj = torch.cat([rows[i][a:a + n] for i, a, n in step]).to(DEV)
        r = h.delta_prepare(proj, dev["conv"], dev["dt_bias"], dev["a_log"], state, ctx, z, dtype)
        at = 0
        for i, _, n in step:
            got[i].append([t[at:at + n] for t in (r.mixed, r.units, r.betas, r.logs)])
            at += n
    for i, n in enumerate(lengths):
        r = rows[i].to(F64)
        u = r[:, z.inner:z.inner + z.channels]
        want = plain.convolve(u, W["conv"], torch.zeros(z.taps - 1, z.channels, dtype=F64))
        mixed, units, betas, logs = (torch.cat(t).cpu().to(F64) for t in zip(*got[i]))
        torch.testing.assert_close(mixed, z.spread(want.t().contiguous()).t(), **(dict(atol=3e-6, rtol=3e-6) if dtype == torch.float32 else dict(atol=1e-6, rtol=5e-3)))
        # the factors make unit vectors of what stands in the rows, 32-bit whatever its type
        at, size = z.heads * z.vp, z.groups * z.np
        for j, scale in ((0, 1.0), (1, z.state ** -0.5)):
            x = mixed[:, at + j * size:at + (j + 1) * size].view(n, z.groups, z.np)[:, :, :z.state]
            unit = units[:, j * z.groups:(j + 1) * z.groups, None] * x
            torch.testing.assert_close(unit, plain.unit_vectors(x) * scale, atol=1e-6, rtol=3e-6)
        a, b = r[:, z.inner + z.channels:z.projected], r[:, z.projected:z.projected + z.heads]
        torch.testing.assert_close(betas, torch.sigmoid(b), atol=1e-7, rtol=1e-5)
        torch.testing.assert_close(logs, -torch.exp(W["A_log"]) * torch.nn.functional.softplus(a + W["dt_bias"], threshold=1e9), atol=1e-6, rtol=1e-5)
        kept = torch.cat([torch.zeros(z.taps - 1, z.channels, dtype=F64), u])[n:]
        left = state[slots[i], z.matrix:z.matrix + z.kept].cpu().to(F64).view(z.taps - 1, z.row)
        assert torch.equal(left, z.spread(kept.t().contiguous()).t() if z.taps > 1 else left), "the last inputs are what the slot keeps"
    assert torch.equal(state[[1, 3]], before[[1, 3]]) and torch.equal(state[:, :z.matrix], before[:, :z.matrix]), "nothing else is touched"


def delta_inputs(dtype, n, gen, z, slow):
    """Random operands as the engine hands them over (convolved rows in its type, factors, steps and decays 32-bit) and the
    oracle's view of the same numbers; `slow`: decays so weak, steps so small that a state outlives hundreds of tokens."""
    h = hip()
    mixed = z.spread(torch.randn(z.channels, n, generator=gen) * 0.8).t().contiguous().to(dtype)
    at, size = z.heads * z.vp, z.groups * z.np
    m = mixed.to(F64)
    v = m[:, :at].view(n, z.heads, z.vp)[:, :, :z.vdim]
    k, q = (m[:, at + j * size:at + (j + 1) * size].view(n, z.groups, z.np)[:, :, :z.state] for j in range(2))
    units = torch.cat([1 / torch.sqrt((k * k).sum(-1) + 1e-6), z.state ** -0.5 / torch.sqrt((q * q).sum(-1) + 1e-6)], 1).float()
    betas = torch.rand(n, z.heads, generator=gen) * (0.1 if slow else 1.0)
    logs = -torch.rand(n, z.heads, generator=gen) * (0.004 if slow else 2.0)
    own = torch.arange(z.heads) // (z.heads // z.groups)
    k = (k * units[:, :z.groups, None].to(F64))[:, own]
    q = (q * units[:, z.groups:, None].to(F64))[:, own]
    return h.DeltaRows(mixed, units, betas, logs), (q, k, v)


def delta_cut(h, rows, pieces):
    """The packed step's operands: `pieces` (request, first row, rows) of the requests' `rows`."""
    return h.DeltaRows(*(torch.cat([getattr(rows[i], name)[a:a + n] for i, a, n in pieces]).to(DEV) for name in ("mixed", "units", "betas", "logs")))


def plain_delta(z, rows, view, S=None):
    q, k, v = view
    return plain.delta_rule(q, k, v, torch.exp(rows.logs.to(F64)), rows.betas.to(F64), torch.zeros(z.heads, z.state, z.vdim, dtype=F64) if S is None else S)


@pytest.mark.parametrize("slow", [False, True])
@pytest.mark.parametrize("portions", sorted(PORTIONS))
@pytest.mark.parametrize("kind", sorted(DELTA_SIZES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_delta_rule_over_steps_and_slots(dtype, kind, portions, slow):
    """Four requests of unequal length in packed steps of changing portions, each with its state in a slot of its own among
    slots that hold other requests' leftovers. 32-bit rows and short portions walk token by token; long portions in bfloat16
    are worked in chunks (whole ones, a chunk's rest), beside walked requests in the same step."""
    h = hip()
    z, _, _, gen = delta_setup(kind)
    lengths, slots = [37, 1, 90, 280], [4, 0, 2, 5]
    inputs = [delta_inputs(dtype, n, gen, z, slow) for n in lengths]
    state = torch.randn(6, z.matrix + z.kept, device=DEV)
    before = state.clone()
    state[slots, :z.matrix] = 0.0
    got = [[] for _ in lengths]
    for step, ctx in packed_steps(lengths, PORTIONS[portions], slots):
        y = h.delta_scan(delta_cut(h, [r for r, _ in inputs], step), state, ctx, z)
        at = 0
        for i, _, n in step:
            got[i].append(y[at:at + n])
            at += n
    tol = 5e-5 if dtype == torch.bfloat16 else 1e-5                            # (of the largest number: two bfloat16 terms, or 32 bits)
    for i, n in enumerate(lengths):
        want, S = plain_delta(z, *inputs[i])
        torch.testing.assert_close(torch.cat(got[i]).cpu().to(F64), want.reshape(n, -1), atol=tol * float(want.abs().max()) + 1e-7, rtol=0)
        left = state[slots[i], :z.matrix].cpu().to(F64).view(z.heads, z.vp, z.np)
        torch.testing.assert_close(left[:, :z.vdim, :z.state], S.transpose(1, 2), atol=tol * float(S.abs().max()) + 1e-7, rtol=0)
        assert float(left[:, z.vdim:].abs().sum()) == 0.0 and float(left[:, :, z.state:].abs().sum()) == 0.0, "places of no number stay zero"
    assert torch.equal(state[[1, 3]], before[[1, 3]]) and torch.equal(state[:, z.matrix:], before[:, z.matrix:])


@pytest.mark.parametrize("portions", ["whole", "long beside single", "two"])
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["same key", "two keys in turn", "nearly the same key"])
def test_keys_that_are_written_over_and_over(dtype, kind, portions):
    """The hardest systems of a chunk: every token writes to the same key (or to two in turn) with steps near 1 and hardly
    any decay, so that each write takes back most of the one before."""
    h = hip()
    z, _, _, gen = delta_setup("plain")
    n = 200
    rows, _ = delta_inputs(dtype, n, gen, z, True)
    at, size = z.heads * z.vp, z.groups * z.np
    base = torch.randn(2, size, generator=gen)
    mixed = rows.mixed.float()
    mixed[:, at:at + size] = base[0] if kind != "two keys in turn" else base[torch.arange(n) % 2]
    if kind == "nearly the same key":
        mixed[:, at:at + size] += 0.01 * torch.randn(n, size, generator=gen)
    mixed = mixed.to(dtype)
    m = mixed.to(F64)
    k, q = (m[:, at + j * size:at + (j + 1) * size].view(n, z.groups, z.np)[:, :, :z.state] for j in range(2))
    units = torch.cat([1 / torch.sqrt((k * k).sum(-1) + 1e-6), z.state ** -0.5 / torch.sqrt((q * q).sum(-1) + 1e-6)], 1).float()
    rows = h.DeltaRows(mixed, units, torch.full((n, z.heads), 0.999), torch.full((n, z.heads), -1e-4))
    own = torch.arange(z.heads) // (z.heads // z.groups)
    view = ((q * units[:, z.groups:, None].to(F64))[:, own], (k * units[:, :z.groups, None].to(F64))[:, own],
            m[:, :at].view(n, z.heads, z.vp)[:, :, :z.vdim])
    want, S = plain_delta(z, rows, view)
    state, out = torch.zeros(1, z.matrix + z.kept, device=DEV), []
    for step, ctx in packed_steps([n], PORTIONS[portions], [0]):
        out.append(h.delta_scan(delta_cut(h, [rows], step), state, ctx, z))
    torch.testing.assert_close(torch.cat(out).cpu().to(F64), want.reshape(n, -1), atol=1e-4 * float(want.abs().max()), rtol=0)


@pytest.mark.parametrize("portions", ["whole", "two"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_tokens_that_forget_everything_between_tokens_that_forget_nothing(dtype, portions):
    """Log decays of -1e-4 beside ones of -30, -3,000 and -1e30: what lies between two forgetful tokens is carried as
    precisely as ever, and a forgetful token leaves nothing behind (and no NaN)."""
    h = hip()
    z, _, _, gen = delta_setup("plain")
    n = 280
    rows, view = delta_inputs(dtype, n, gen, z, True)
    rows.logs.fill_(-1e-4)
    for t, l in ((10, -3000.0), (11, -3000.0), (40, -30.0), (63, -3000.0), (64, -1e30), (100, -1e30), (101, -3000.0), (200, -1.0), (255, -1e30)):
        rows.logs[t] = l
    state, out = torch.zeros(1, z.matrix + z.kept, device=DEV), []
    for step, ctx in packed_steps([n], PORTIONS[portions], [0]):
        out.append(h.delta_scan(delta_cut(h, [rows], step), state, ctx, z))
    want, _ = plain_delta(z, rows, view)
    torch.testing.assert_close(torch.cat(out).cpu().to(F64), want.reshape(n, -1), atol=5e-5 * float(want.abs().max()), rtol=0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_token_is_read_out_hundreds_of_tokens_later(dtype):
    """One token writes to a place that no other key touches, and one far later query reads only that place: what comes back
    is that token's step times its value, decayed by the tokens between. A second write to the same place in between, with a
    step of 1, leaves nothing of the first. At chunks' borders on both sides, whole and in portions of two."""
    h = hip()
    z, _, _, gen = delta_setup("plain")
    n, at, size = 400, z.heads * z.vp, z.groups * z.np
    for src, over, dst in ((0, None, 399), (63, None, 64), (64, None, 127), (5, 70, 191), (128, 191, 192), (191, None, 193), (399, None, 399), (10, 63, 64), (10, 64, 64)):
        mixed = torch.randn(n, z.row, generator=gen) * 0.5
        k, q = (mixed[:, at + j * size:at + (j + 1) * size].view(n, z.groups, z.np) for j in range(2))
        k[:, :, 7] = q[:, :, 7] = 0.0
        for t in (src, over):
            if t is not None:
                k[t] = 0.0
                k[t, :, 7] = 1.0
        q[dst] = 0.0
        q[dst, :, 7] = 2.0
        mixed = mixed.to(dtype)
        kd, qd = (mixed.to(F64)[:, at + j * size:at + (j + 1) * size].view(n, z.groups, z.np) for j in range(2))
        units = torch.cat([1 / torch.sqrt((kd * kd).sum(-1) + 1e-6), z.state ** -0.5 / torch.sqrt((qd * qd).sum(-1) + 1e-6)], 1).float()
        betas = torch.full((n, z.heads), 0.5)
        if over is not None:
            betas[over] = 1.0
        rate = torch.linspace(5e-4, 4e-3, z.heads)
        rows = h.DeltaRows(mixed, units, betas, -rate.expand(n, -1).contiguous())
        last = src if over is None else over
        v = mixed[last, :at].to(F64).view(z.heads, z.vp)[:, :z.vdim]
        want = float(betas[last, 0]) * v * torch.exp(-(dst - last) * rate.to(F64))[:, None] * z.state ** -0.5
        for portions in ([400], [2]):
            state, out = torch.zeros(1, z.matrix + z.kept, device=DEV), []
            for step, ctx in packed_steps([n], portions, [0]):
                out.append(h.delta_scan(delta_cut(h, [rows], step), state, ctx, z))
            y = torch.cat(out)[dst].cpu().to(F64).view(z.heads, z.vdim)
            torch.testing.assert_close(y, want, atol=2e-5, rtol=1e-4, msg=lambda s: f"{src} read at {dst} in portions {portions}: {s}")


@pytest.mark.parametrize("layer", ["P0", "P2", "Q1", "Q3", "R0", "S1", "S2", "T0", "T2"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_whole_delta_mixer(dtype, layer):
    from tinyserve_llm_amd.parts.base import LayerMemory
    from tinyserve_llm_amd.parts.gated_delta import GatedDelta
    config = kufolorn_configs()[layer[0]][0]
    m = config.layers[int(layer[1])].mixer
    part = GatedDelta(config.width, m.heads, m.kv_heads, m.dim, m.vdim, m.conv, config.norm_eps)
    z, gen = part.sizes, torch.Generator().manual_seed(9)
    P = {}
    for name, spec in part.param_specs().items():
        t = torch.randn(spec.shape, generator=gen) * (spec.init[1] if name not in ("proj", "o") else spec.shape[1] ** -0.5) + spec.init[0]
        P[name] = t.to(torch.float32 if spec.storage == "float32" else dtype)
    part.bind({n: t.to(DEV) for n, t in P.items()})
    shared = m.kv_heads * m.dim
    g, v, k, q, a, b = P["proj"][:part.projected].to(F64).split([z.inner, z.inner, shared, shared, m.heads, m.heads])
    vc, kc, qc = P["conv"].to(F64).split([z.inner, shared, shared])
    W = {"q": q, "k": k, "v": v, "g": g, "a": a, "b": b, "q.conv": qc, "k.conv": kc, "v.conv": vc, "A_log": P["a_log"].to(F64),
         "dt_bias": P["dt_bias"].to(F64), "norm": P["norm"].to(F64), "o": P["o"].to(F64)}
    x, x64 = rounded(torch.randn(150, config.width, generator=gen), dtype)
    mem = LayerMemory(state=torch.zeros(2, *part.state_spec().shape, device=DEV))
    raw = config.to_dict()["layers"][int(layer[1])]["mixer"]
    st, out, want = {}, [], []
    for a, b in ((0, 1), (1, 3), (3, 100), (100, 101), (101, 150)):
        out.append(part.forward(x[a:b], step_context([[0]], 1 << 20, [a], [b - a], slots=[1]), mem))
        want.append(plain.delta_mixer(x64[a:b], W, raw, config.norm_eps, st))
    want = torch.cat(want)
    tol = 5e-5 if dtype == torch.float32 else 3e-2
    torch.testing.assert_close(torch.cat(out).cpu().to(F64), want, atol=tol * float(want.abs().max()), rtol=tol)


# ---- whole models through trace replay ---------------------------------------------------------------

LENGTHS = {"P": [1, 23, 97, 200], "Q": [1, 30, 75, 150], "R": [2, 19, 66, 131], "S": [1, 40, 140], "T": [1, 29, 110]}
TOL = {"float32": 5e-5, "bfloat16": 0.12}       # of the spread of the oracle's logits, for every row,
MEDIAN = {"float32": 2e-5, "bfloat16": 0.03}    # and for the middle one (a head whose read-out is nearly nothing is normed up, and its rounding with it)


def calm(oracle, seed, n, vocab):
    """(a prompt of n tokens, the plain model's logits for them): random tokens, drawn again where a router's choice would be
    a close call, which bfloat16 may turn round."""
    gen = torch.Generator().manual_seed(seed)
    oracle.reset()
    ids, rows = [], []
    for _ in range(n):
        for _ in range(30):
            before = ([dict(m) for m in oracle.memory], oracle.fed)
            token = int(torch.randint(0, vocab, (1,), generator=gen))
            row = oracle.forward([token])[0]
            if oracle.margin > 0.12:
                break
            oracle.memory, oracle.fed = before
        else:
            row = oracle.forward([token])[0]
        ids.append(token)
        rows.append(row)
    return ids, torch.stack(rows)


@pytest.fixture(scope="module", params=["P", "Q", "R", "S", "T"])
def case(request, tmp_path_factory):
    from tinyserve_llm_amd.weights.random_init import write_random_model
    name = request.param
    config, seed = kufolorn_configs()[name]
    folder = str(tmp_path_factory.mktemp(f"kufolorn_{name}"))
    write_random_model(folder, config, seed, torch.bfloat16)
    oracle = plain.PlainKufolorn.from_folder(folder)
    prompts, rows = zip(*(calm(oracle, 500 + i, n, config.vocab) for i, n in enumerate(LENGTHS[name])))
    return name, folder, config, list(prompts), oracle, list(rows)


@pytest.fixture(scope="module")
def further(case):
    """More prompts of the same model with the plain model's rows: nine unequal ones, one of 520 tokens, one of 305."""
    _, _, config, _, oracle, _ = case
    return {n: calm(oracle, 900 + i, n, config.vocab) for i, n in enumerate([129, 70, 40, 1, 65, 100, 128, 30, 150, 520, 305])}


def replayer(folder, dtype, max_tokens):
    from tinyserve_llm_amd.engine.replay import Replay
    return Replay(folder, dtype, max_tokens)


def check(got, oracle_rows, dtype):
    """Every row's root mean square difference within `TOL` of the logits' spread, and the middle row's within `MEDIAN`."""
    assert got, "nothing was compared"
    spread = float(torch.cat([o.flatten() for o in oracle_rows]).std())
    errors = {key: float((row.double().cpu() - oracle_rows[key[0]][key[1]]).pow(2).mean().sqrt()) / spread for key, row in got.items()}
    over = {key: e for key, e in errors.items() if not e <= TOL[dtype]}
    print(f"[{dtype}] worst row {max(errors.values()):.3e} of the logits' spread ({spread:.2f}) over {len(got)} rows")
    assert not over, f"(request, position): error {over}"
    middle = sorted(errors.values())[(len(errors) - 1) // 2]
    assert middle <= MEDIAN[dtype], f"half the rows are {middle:.3e} away or more"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_layer_streams_and_whole_requests(case, dtype):
    name, folder, config, prompts, oracle, rows = case
    rep = replayer(folder, dtype, 256)
    got = {}
    for r, p in enumerate(prompts):
        logits = rep.step([{"id": f"r{r}", "tokens": p, "want": list(range(len(p)))}], [f"r{r}"])
        assert logits.shape == (len(p), config.vocab) and logits.dtype == torch.float32
        for pos in range(len(p)):
            got[(r, pos)] = logits[pos]
    check(got, rows, dtype)
    assert rep.manager.num_available_blocks() == rep.manager.num_blocks, "every page came back"
    assert len(rep.manager.free_state_slots) == 4, "every state slot came back"
    if dtype == "float32":
        # the residual stream after every layer, one by one
        from tinyserve_llm_amd.engine.runner import StepEntry
        from tinyserve_llm_amd.parts import base
        from tinyserve_llm_amd.parts.stream import ResidualStream
        p = prompts[2]
        want = oracle.streams(p)
        assert len(want) == len(rep.model.spec.order)
        rep.manager.allocate(77, p)
        ctx, _, _ = rep.runner.prepare([StepEntry(77, p, 0, [])])
        ctx.position_encodings = rep.model.position_encodings
        hidden, residual = rep.model.embedding.forward(ctx), None
        for i, (run, mem) in enumerate(zip(rep.model.spec.order, rep.runner.memory)):
            layer = rep.model.layers[run.layer]
            hidden, residual = base.BLOCKS[layer.block](layer, hidden, residual, ctx, mem)
            now = ResidualStream(hidden.x.clone(), hidden.a, post=hidden.post).take()[0]
            scale = float(want[i].abs().max())
            torch.testing.assert_close(now.cpu().double(), want[i], atol=3e-5 * max(1.0, scale), rtol=1e-5, msg=lambda m: f"after layer {i}: {m}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompt_then_token_by_token(case, dtype):
    """The last tokens one by one: more of them than a page holds."""
    name, folder, config, prompts, oracle, rows = case
    rep = replayer(folder, dtype, 256)
    got = {}
    for r, p in enumerate(prompts):
        head = max(0, len(p) - 80)
        if head:
            got[(r, head - 1)] = rep.step([{"id": f"r{r}", "tokens": p[:head], "want": [head - 1]}], [])[0]
        for pos in range(head, len(p)):
            got[(r, pos)] = rep.step([{"id": f"r{r}", "tokens": [p[pos]], "want": [0]}], [f"r{r}"] if pos == len(p) - 1 else [])[0]
    check(got, rows, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_portions_down_to_two_tokens(case, dtype):
    name, folder, config, prompts, oracle, rows = case
    rep = replayer(folder, dtype, 256)
    sizes = [2, 7, 3, 16, 2, 5, 31, 2, 64, 9, 1, 33]
    got = {}
    for r, p in enumerate(prompts):
        pos, i = 0, r
        while pos < len(p):
            n = min(sizes[i % len(sizes)], len(p) - pos)
            i += 1
            want = sorted({0, n - 1})
            logits = rep.step([{"id": f"r{r}", "tokens": p[pos:pos + n], "want": want}], [f"r{r}"] if pos + n == len(p) else [])
            for j, w in enumerate(want):
                got[(r, pos + w)] = logits[j]
            pos += n
    check(got, rows, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_mixed_batches_on_pages_and_slots_used_again(case, further, dtype):
    """Nine unequal requests, at most four live, on a pool that holds the first four: later requests start on pages and in
    state slots that earlier ones have written and given back, beside others that are in the middle of theirs. A state that is not cleared, or a stale page, shows in the logits."""
    name, folder, config, _, oracle, _ = case
    lengths = [129, 70, 40, 1, 65, 100, 128, 30, 150]
    prompts, rows = zip(*(further[n] for n in lengths))
    pool = sum(-(-n // 64) for n in lengths[:4])
    rep = replayer(folder, dtype, 64 * pool)
    assert rep.manager.num_blocks == pool and len(rep.manager.free_state_slots) == 4
    chunk = [13, 2, 1, 7, 1, 1, 30, 1, 3, 1]
    cursors, pages = [0] * len(prompts), [-(-n // 64) for n in lengths]
    waiting, live, tick, got, slots_used = list(range(len(prompts))), [], 0, {}, []
    while waiting or live:
        while waiting and len(live) < 4 and sum(pages[r] for r in live) + pages[waiting[0]] <= pool:
            live.append(waiting.pop(0))
        batch, end, wanted = [], [], []
        new = [r for r in live if cursors[r] == 0]
        for r in live:
            n = min(lengths[r] - cursors[r], chunk[(tick + 3 * r) % len(chunk)])
            batch.append({"id": f"q{r}", "tokens": prompts[r][cursors[r]:cursors[r] + n], "want": [n - 1]})
            wanted.append((r, cursors[r] + n - 1))
            cursors[r] += n
            if cursors[r] == lengths[r]:
                end.append(r)
        logits = rep.step(batch, [])
        slots_used += [rep.manager.state_slot(rep.ids[f"q{r}"]) for r in new]
        for j, key in enumerate(wanted):
            got[key] = logits[j]
        rep.step([], [f"q{r}" for r in end])
        live = [r for r in live if r not in end]
        tick += 1
    assert len(slots_used) > len(set(slots_used)), "state slots were used again"
    check(got, rows, dtype)
    assert rep.manager.num_available_blocks() == rep.manager.num_blocks


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_prompts_whole_and_in_long_portions(case, further, dtype):
    """Steps of hundreds of tokens take kernels of their own: a prompt of 520 tokens whole, and cut where the second
    portion starts in the middle of a page and of a chunk of the recurrences, beside a short request."""
    name, folder, config, _, oracle, _ = case
    (long, long_rows), (short, short_rows) = further[520], further[40]
    rows = [long_rows, short_rows]
    rep = replayer(folder, dtype, 640)
    marks = [0, 1, 255, 256, 257, 300, 518, 519]
    got = {}
    logits = rep.step([{"id": "w", "tokens": long, "want": marks}], ["w"])
    for j, pos in enumerate(marks):
        got[(0, pos)] = logits[j]
    check(got, rows, dtype)
    got = {}
    logits = rep.step([{"id": "a", "tokens": long[:263], "want": [0, 262]}, {"id": "b", "tokens": short[:7], "want": [6]}], [])
    got[(0, 0)], got[(0, 262)], got[(1, 6)] = logits[0], logits[1], logits[2]
    logits = rep.step([{"id": "b", "tokens": short[7:], "want": [0, 32]}, {"id": "a", "tokens": long[263:], "want": [0, 1, 37, 256]}], ["a", "b"])
    got[(1, 7)], got[(1, 39)] = logits[0], logits[1]
    for j, pos in enumerate([263, 264, 300, 519]):
        got[(0, pos)] = logits[2 + j]
    check(got, rows, dtype)
    assert rep.manager.num_available_blocks() == rep.manager.num_blocks


def test_a_batch_equals_each_request_alone_in_float32(case):
    """float32: the logits of a request do not depend on what else is in the batch, beyond rounding."""
    name, folder, config, prompts, oracle, rows = case
    rep = replayer(folder, "float32", 1024)
    alone = [rep.step([{"id": f"a{r}", "tokens": p, "want": [len(p) - 1]}], [f"a{r}"])[0] for r, p in enumerate(prompts)]
    together = rep.step([{"id": f"b{r}", "tokens": p, "want": [len(p) - 1]} for r, p in enumerate(prompts)],
                        [f"b{r}" for r in range(len(prompts))])
    for r in range(len(prompts)):
        torch.testing.assert_close(together[r], alone[r], atol=2e-6, rtol=1e-6)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(case, further, dtype):
    """300 tokens fed one by one after a prompt of five: states are carried through every step, keys fill page after page."""
    name, folder, config, _, oracle, _ = case
    p, rows = further[305]
    rep = replayer(folder, dtype, 320)
    rep.step([{"id": "d", "tokens": p[:5], "want": []}], [])
    got = {}
    for pos in range(5, len(p)):
        logits = rep.step([{"id": "d", "tokens": [p[pos]], "want": [0]}], [])
        if pos % 7 == 0 or pos >= 300:
            got[(0, pos)] = logits[0]
    check(got, [rows], dtype)


# ---- generation through the engine's entry point -----------------------------------------------------

def test_greedy_generation_through_the_scheduler(case):
    from tinyserve_llm_amd.engine.llm import LLM, CacheConfig
    from tinyserve_llm_amd.engine.scheduler import SchedulerConfig
    from tinyserve_llm_amd.engine.sequence import SamplingParams
    name, folder, config, prompts, oracle, _ = case
    prompts = [p for p in prompts if len(p) <= 75] + [prompt(42, 90, config.vocab)]
    want = [oracle.greedy(p, 12) for p in prompts]
    sc = SchedulerConfig(max_model_len=256, max_num_seqs=4, max_num_batched_tokens=48, max_prefill_chunk=32)
    llm = LLM(folder, sc, CacheConfig(block_size=32), dtype=torch.float32, num_blocks=24)
    got = llm.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    assert [r.token_ids[0] for r in got] == want
    # bfloat16 may flip a near-tie: its tokens are judged by the plain model's logits for the same history
    llm16 = LLM(folder, sc, CacheConfig(block_size=32), dtype=torch.bfloat16, num_blocks=24)
    got16 = llm16.generate(prompts[:2], SamplingParams(max_tokens=8, temperature=0.0, ignore_eos=True))
    spread = float(oracle.logits(prompts[1]).std())
    for p, r in zip(prompts, got16):
        ids = list(p)
        for tok in r.token_ids[0]:
            row = oracle.logits(ids)[-1]
            assert float(row.max() - row[tok]) <= 0.15 * spread, "a bfloat16 token far from the plain model's best"
            ids.append(tok)


def test_forked_continuations_and_preemption(case):
    """n = 3 at temperature 0: the continuations part after the prompt, each with a copy of the states and the
    prompt's pages shared; all three must be the oracle's greedy continuation. And a pool so small that requests are
    preempted and fed again from their first token."""
    from tinyserve_llm_amd.engine.llm import LLM, CacheConfig
    from tinyserve_llm_amd.engine.scheduler import SchedulerConfig
    from tinyserve_llm_amd.engine.sequence import SamplingParams
    name, folder, config, prompts, oracle, _ = case
    p = prompt(11, 45, config.vocab)
    want = oracle.greedy(p, 10)
    sc = SchedulerConfig(max_model_len=128, max_num_seqs=4, max_num_batched_tokens=64, max_prefill_chunk=16)
    llm = LLM(folder, sc, CacheConfig(block_size=16), dtype=torch.float32, num_blocks=24)
    got = llm.generate([p], SamplingParams(max_tokens=10, temperature=0.0, n=3, ignore_eos=True))
    assert got[0].token_ids == [want, want, want]
    many = [prompt(20 + i, 60 + 3 * i, config.vocab) for i in range(4)]
    wants = [oracle.greedy(q, 30) for q in many]
    small = LLM(folder, sc, CacheConfig(block_size=16, caching=False), dtype=torch.float32, num_blocks=14)
    out = small.generate(many, SamplingParams(max_tokens=30, temperature=0.0, ignore_eos=True))
    assert [r.token_ids[0] for r in out] == wants


def test_command_line_generates_from_a_model_folder(case, tmp_path):
    import json
    import os
    import subprocess
    import sys
    name, folder, config, prompts, oracle, _ = case
    if name != "P":
        pytest.skip("one configuration through the command line is enough")
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    p = prompts[2]
    out = tmp_path / "record.json"
    cmd = [sys.executable, "-m", "tinyserve_llm_amd.generate", "--model", folder, "--prompt-ids", ",".join(map(str, p)),
           "--max-tokens", "6", "--temperature", "0", "--ignore-eos", "--dtype", "float32", "--block-size", "32",
           "--num-blocks", "16", "--max-model-len", "256", "--max-num-seqs", "4", "--out", str(out)]
    r = subprocess.run(cmd, cwd=root, capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr[-2000:]
    record = json.loads(out.read_text())
    text = json.dumps(record)
    assert json.dumps(oracle.greedy(p, 6)).replace(" ", "") in text.replace(" ", ""), text[:500]
