"""The Morulix decoder on the GPU against the plain implementation in tests/plain/morulix.py: each mechanism's kernel
alone (with inputs made so that a fault shows: a far key whose score stands out, keys just inside and just outside a
window, at page borders, the first tokens where a sink weighs most, a state that is to be read out hundreds of tokens
after it was written, states and convolution inputs carried over steps and slots), then whole models of five small
configurations through trace replay (layer by layer, whole, token by token, in portions down to two tokens, mixed
batches on pages and state slots that are used again, long decoding), and greedy generation through `LLM.generate` and
the scheduler. float32 and bfloat16."""

from __future__ import annotations

import pytest
import torch

from tests.helpers import morulix_configs, prompt
from tests.plain import morulix as plain
from tests.test_gpu_fanotar import paged, rounded, step_context, tolerance

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F64 = torch.float64
DTYPES = [torch.float32, torch.bfloat16]


def hip():
    from tinyserve_llm_amd.ops import hip as h
    return h


# ---- the stream: one norm for two branches, a row added to every token, the input of a pass -----------

@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width", [80, 99, 256, 2048, 4100])
def test_a_row_added_to_every_token_rides_on_the_norm(dtype, width):
    from tinyserve_llm_amd.parts.norm import RMSNorm
    from tinyserve_llm_amd.parts.stream import ResidualStream
    n, eps = 7, 1e-5
    x, row = torch.randn(n, width) * 3, torch.randn(3, width)
    step, step64 = rounded(row, dtype)
    w, w64 = rounded(torch.randn(width) * 0.2, dtype)
    norm = RMSNorm(width, eps, one_plus=True)
    norm.bind({"weight": w})
    stream = ResidualStream(x.to(DEV), bias=step[1])
    assert stream.pending
    got, h = stream.take(norm)
    want = x.to(F64) + step64[1]
    torch.testing.assert_close(got.cpu().to(F64), want, atol=2e-6, rtol=1e-6)
    torch.testing.assert_close(h.cpu().to(F64), plain.layer_norm(want, w64, eps), **tolerance(dtype))
    assert not stream.pending
    # two branches' rows pending, then the norm of picked rows
    a, b = torch.randn(n, width), torch.randn(n, width)
    stream = ResidualStream(x.to(DEV), a.to(DEV), b.to(DEV))
    rows = torch.tensor([5, 0], dtype=torch.int32, device=DEV)
    picked, _ = norm(stream, None, rows)
    want = (x + a).to(F64) + b.to(F64)
    torch.testing.assert_close(picked.cpu().to(F64), plain.layer_norm(want, w64, eps)[[5, 0]], **tolerance(dtype))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("tokens, width", [(1, 80), (7, 99), (5, 512), (70, 256), (300, 80)])
def test_the_input_of_a_pass(dtype, tokens, width):
    """W [x; x0] + step[n], x with both branches' rows pending and with none; the stream that comes in is not what goes on."""
    from tinyserve_llm_amd.parts.pass_input import ProjectedPassInput
    from tinyserve_llm_amd.parts.stream import ResidualStream
    part = ProjectedPassInput(width, 3)
    w, w64 = rounded(torch.randn(width, 2 * width) * (2 * width) ** -0.5, dtype)
    step, step64 = rounded(torch.randn(3, width), dtype)
    part.bind({"weight": w, "step": step})
    x, x0, a, b = (torch.randn(tokens, width) for _ in range(4))
    tol = dict(atol=3e-5, rtol=1e-5) if dtype == torch.float32 else dict(atol=3e-2, rtol=1e-2)
    start = x0.to(DEV)
    for n, pending in ((0, (None, None)), (2, (a, b)), (1, (a, None))):
        before = x.to(DEV)
        stream = ResidualStream(before, *(None if t is None else t.to(DEV) for t in pending))
        out = part.forward(stream, start, None, n).settle()[0]
        now = x.to(F64) + sum(t.to(F64) for t in pending if t is not None)
        torch.testing.assert_close(out.cpu().to(F64), plain.pass_input(now, x0.to(F64), w64, step64[n]), **tol)
        assert torch.equal(start.cpu(), x0), "the embedding's rows stay for the passes to come"
    joined = ResidualStream(x.to(DEV), a.to(DEV), b.to(DEV)).joined_with(start, dtype)
    exact = torch.cat([x + (a + b), x0], 1)
    assert torch.equal(joined.cpu(), exact.to(dtype))


# ---- windowed attention: edges, far keys, page borders -------------------------------------------------

FORMS = {"decoded": None, "prompt": 0, "portion": 130}       # (a portion that starts inside a page)


def decides(want_row, value_row) -> bool:
    return float((want_row - value_row).abs().max()) < 0.2 * float(value_row.abs().max())


def marked(length, queries, stand_out, H, G, D, gen, scale):
    """Queries and keys of unit size, where a query's score for the key it is to find stands out at 11."""
    k64 = plain.unit_rms(torch.randn(length, G, D, generator=gen, dtype=F64), 0.0)
    q64 = plain.unit_rms(torch.randn(len(queries), H, D, generator=gen, dtype=F64), 0.0)
    for i, p in enumerate(queries):
        if p in stand_out:
            g_dir = plain.unit_rms(torch.randn(G, D, generator=gen, dtype=F64), 0.0)
            for hh in range(H):
                q64[i, hh] = g_dir[hh // (H // G)]
            k64[stand_out[p]] = 11.0 / (D * scale) * g_dir
    return q64, k64


def window_case(dtype, H, G, D, V, page, length, queries, stand_out, window, portion_from):
    """One request of `length` tokens on shuffled pages; queries as decoded tokens over the same pages, or every position
    from `portion_from` on as one portion of a prompt. Returns (kernel output, oracle output, values, query positions)."""
    h = hip()
    if portion_from is not None:
        queries = list(range(portion_from, length))
        stand_out = {q: key for q, key in stand_out.items() if q >= portion_from}
    gen = torch.Generator().manual_seed(5)
    scale = D ** -0.5
    q64, k64 = marked(length, queries, stand_out, H, G, D, gen, scale)
    v64 = torch.randn(length, G, V, generator=gen, dtype=F64)
    pages = -(-length // page)
    table = torch.randperm(pages + 3, generator=gen)[:pages].tolist()
    k, v = paged(pages + 3, page, G, D, V, dtype)
    kr, vr = k64.to(dtype), v64.to(dtype)
    at = torch.arange(length)
    pg, off = torch.tensor(table)[at // page].to(DEV), (at % page).to(DEV)
    k[pg, off], v[pg, off] = kr.to(DEV), vr.to(DEV)
    q = q64.to(dtype).to(DEV)
    ctx = step_context([table] * len(queries), page, queries, [1] * len(queries)) if portion_from is None else \
        step_context([table], page, [portion_from], [len(queries)])
    out = h.paged_attention(q, k, v, ctx, 0, scale, window)
    want = plain.softmax_attention(q.cpu().to(F64), kr.to(F64), vr.to(F64), torch.tensor(queries), scale, window)
    return out.cpu().to(F64).view(len(queries), H, V), want, vr.to(F64), queries


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("window, sizes", [(1, (2, 2, 16, 16)), (16, (4, 2, 32, 48)), (24, (4, 2, 32, 48)), (33, (8, 2, 64, 64)), (64, (4, 4, 64, 64)),
                                           (70, (3, 1, 20, 12)), (130, (8, 2, 64, 64)), (257, (4, 1, 96, 96)), (100, (2, 2, 128, 128))])
def test_window_edges(dtype, window, sizes, form):
    """The key that stands out is the farthest a query sees for some queries and the first it does not see for others."""
    H, G, D, V = sizes
    length = max(600, 4 * window + 15)
    inside = {q: q - window + 1 for q in (window - 1, 3 * window + 9)}
    outside = {q: q - window for q in (2 * window + 4, length - 1)}
    queries = sorted({0, 127, 128, 129, *inside, *outside})
    out, want, v, queries = window_case(dtype, H, G, D, V, 32 if window % 2 else 16, length, queries, {**inside, **outside}, window, FORMS[form])
    torch.testing.assert_close(out, want, **tolerance(dtype))
    for q, key in inside.items():
        if q in queries:
            assert decides(want[queries.index(q), 0], v[key, 0]), (q, key)
    for q, key in outside.items():
        if q in queries and window > 1:
            assert not decides(want[queries.index(q), 0], v[key, 0]), (q, key)


# ---- attention through a latent, with sinks and a gate per head ----------------------------------------

def latent_case(dtype, H, rank, page, length, queries, stand_out, portion_from, sinks, gate, seed=3):
    h = hip()
    if portion_from is not None:
        queries = list(range(portion_from, length))
        stand_out = {q: key for q, key in stand_out.items() if q >= portion_from}
    gen = torch.Generator().manual_seed(seed)
    scale = rank ** -0.5
    q64, k64 = marked(length, queries, stand_out, H, 1, rank, gen, scale)
    rows = k64[:, 0].to(dtype)
    pages = -(-length // page)
    table = torch.randperm(pages + 3, generator=gen)[:pages].tolist()
    cache = torch.zeros(pages + 3, page, 1, rank, dtype=dtype, device=DEV)
    values = torch.zeros(pages + 3, 1, rank, page, dtype=dtype, device=DEV).permute(0, 3, 1, 2)
    at = torch.arange(length)
    pg, off = torch.tensor(table)[at // page].to(DEV), (at % page).to(DEV)
    cache[pg, off, 0] = rows.to(DEV)
    values[pg, off, 0] = rows.to(DEV)
    q = q64.float().to(DEV)
    wide = torch.randn(len(queries), H + 5, generator=gen) * 2                # (the gate's numbers are columns of wider rows)
    ctx = step_context([table] * len(queries), page, queries, [1] * len(queries)) if portion_from is None else \
        step_context([table], page, [portion_from], [len(queries)])
    s = None if sinks is None else sinks.float().to(DEV)
    g = wide.to(DEV)[:, 2:2 + H] if gate else None
    out = h.paged_attention_latent(q, cache, rank, ctx, 0, scale, out_dtype=dtype, v_cache=values, sinks=s, head_gate=g)
    keys = rows.to(F64)[:, None, :]
    want = plain.softmax_attention(q.cpu().to(F64), keys, keys, torch.tensor(queries), scale, sinks=None if sinks is None else sinks.to(F64))
    if gate:
        want = want * torch.sigmoid(wide[:, 2:2 + H].to(F64))[:, :, None]
    used = h.latent_mfma_takes(q, cache, values, rank)
    return out.cpu().to(F64), want, keys[:, 0], queries, used


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("page", [16, 32])
@pytest.mark.parametrize("sizes", [(3, 40), (2, 16), (8, 256), (5, 34), (20, 128), (6, 64), (40, 512), (33, 496)])
def test_latent_attention_with_sinks_and_gates(dtype, sizes, form, page):
    """Far keys and keys at page borders stand out for their queries and decide their rows, beside a sink per head that
    differs from head to head; decoded tokens' keys are cut into stretches whose parts a second kernel adds up."""
    H, rank = sizes
    stand_out = {699: 3, 650: 15, 651: 16, 652: 17, 653: 653, 500: 255, 501: 256, 31: 0, 32: 31, 33: 32}
    queries = [0, 1, 2, 3, 15, 16, 17, 31, 32, 33, 500, 501, 650, 651, 652, 653, 699]
    sinks = torch.linspace(-3.0, 4.0, H)
    out, want, v, qs, used = latent_case(dtype, H, rank, page, 700, queries, stand_out, FORMS[form], sinks, True)
    assert used == (dtype == torch.bfloat16 and page == 32 and rank % 16 == 0)
    torch.testing.assert_close(out, want, **tolerance(dtype))
    plain_out, plain_want, v, qs, _ = latent_case(dtype, H, rank, page, 700, queries, stand_out, FORMS[form], None, False)
    torch.testing.assert_close(plain_out, plain_want, **tolerance(dtype))
    assert decides(plain_want[qs.index(699), 0], v[3]), "the far key decides the row"


@pytest.mark.parametrize("form", sorted(FORMS))
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_sink_takes_its_share_and_no_more(dtype, form):
    """A sink far above every score takes nearly everything, one far below nothing, whatever their distance (no overflow);
    one that equals the only score takes half at the first token."""
    H, rank = 4, 64
    for value in (300.0, 6.0, 0.0, -40.0, -300.0):
        sinks = torch.full((H,), value)
        out, want, v, qs, _ = latent_case(dtype, H, rank, 32, 300, [0, 1, 2, 31, 32, 299], {}, FORMS[form], sinks, False)
        torch.testing.assert_close(out, want, **tolerance(dtype))
        if value >= 300:
            assert float(out.abs().max()) < 1e-6
        if value <= -300 and qs[0] == 0:
            torch.testing.assert_close(out[0, 0], v[0], **tolerance(dtype))


# ---- the state-space mixer: convolution and step sizes, the recurrence, the gated norm -----------------

SSD_SIZES = {"odd": (3, 13, 3, 37, 6), "small": (4, 20, 2, 24, 4), "one": (1, 16, 1, 16, 2), "plain": (8, 64, 2, 128, 4), "large": (4, 80, 2, 160, 3),
             "no taps": (6, 8, 6, 32, 1), "tiny": (2, 1, 1, 1, 3), "many taps": (2, 24, 2, 40, 9), "tall": (2, 16, 1, 300, 4)}


def ssd_setup(kind, dtype, seed=1):
    """Sizes and random parameters, rounded where the engine's are; the plain mixer's weights by name, with projections that
    pick coordinates of the input, so that a projected row itself can be fed to it."""
    h = hip()
    H, V, G, N, taps = SSD_SIZES[kind]
    z = h.SsdSizes(H, V, G, N, taps)
    gen = torch.Generator().manual_seed(seed)
    W = {"conv": torch.randn(z.channels, taps, generator=gen) * 0.7, "conv.b": torch.randn(z.channels, generator=gen) * 0.3,
         "dt_bias": torch.randn(H, generator=gen) - 1.0, "A_log": torch.randn(H, generator=gen) * 0.7, "D": 1 + torch.randn(H, generator=gen) * 0.5}
    W = {k: v.to(F64) for k, v in W.items()}
    dev = dict(conv=z.spread(W["conv"].float()).t().contiguous().to(DEV), bias=z.spread(W["conv.b"].float()).to(DEV),
               dt_bias=W["dt_bias"].float().to(DEV), a_log=W["A_log"].float().to(DEV), skip=W["D"].float().to(DEV))
    return z, W, dev, gen


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


@pytest.mark.parametrize("portions", sorted(PORTIONS))
@pytest.mark.parametrize("kind", sorted(SSD_SIZES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_convolution_and_step_sizes_over_steps_and_slots(dtype, kind, portions):
    h = hip()
    z, W, dev, gen = ssd_setup(kind, dtype)
    lengths, slots = [37, 1, 90, 280], [4, 0, 2, 5]
    rows = [torch.randn(n, z.projected + 3, generator=gen) * 1.5 for n in lengths]           # (columns behind: not its business)
    state = torch.randn(6, z.matrix + z.kept, device=DEV)
    before = state.clone()
    state[slots, z.matrix:] = 0.0
    got = [[] for _ in lengths]
    for step, ctx in packed_steps(lengths, PORTIONS[portions], slots):
        proj = torch.cat([rows[i][a:a + n] for i, a, n in step]).to(DEV)
        mixed, steps, logs = h.ssd_prepare(proj, dev["conv"], dev["bias"], dev["dt_bias"], dev["a_log"], state, ctx, z, dtype)
        at = 0
        for i, _, n in step:
            got[i].append((mixed[at:at + n], steps[at:at + n], logs[at:at + n]))
            at += n
    tol = dict(atol=3e-6, rtol=3e-6) if dtype == torch.float32 else dict(atol=1e-6, rtol=5e-3)
    for i, n in enumerate(lengths):
        r = rows[i].to(F64)
        u = r[:, z.inner:z.inner + z.channels]
        want = plain.convolve(u, W["conv"], W["conv.b"], torch.zeros(z.taps - 1, z.channels, dtype=F64))
        mixed, steps, logs = (torch.cat(t).cpu().to(F64) for t in zip(*got[i]))
        torch.testing.assert_close(mixed, z.spread(want.t().contiguous()).t(), **tol)
        d = torch.nn.functional.softplus(r[:, z.inner + z.channels:z.projected] + W["dt_bias"], threshold=1e9)
        torch.testing.assert_close(steps, d, atol=1e-6, rtol=1e-5)
        torch.testing.assert_close(logs, -torch.exp(W["A_log"]) * d, atol=1e-6, rtol=1e-5)
        kept = torch.cat([torch.zeros(z.taps - 1, z.channels, dtype=F64), u])[n:]
        left = state[slots[i], z.matrix:z.matrix + z.kept].cpu().to(F64).view(z.taps - 1, z.row)
        assert torch.equal(left, z.spread(kept.t().contiguous()).t() if z.taps > 1 else left), "the last inputs are what the slot keeps"
    assert torch.equal(state[[1, 3]], before[[1, 3]]) and torch.equal(state[:, :z.matrix], before[:, :z.matrix]), "nothing else is touched"


def test_step_sizes_far_out_and_a_log_rate_of_either_sign():
    h = hip()
    z, W, dev, gen = ssd_setup("one", torch.float32)
    proj = torch.zeros(5, z.projected)
    proj[:, -1] = torch.tensor([-90.0, -20.0, 0.0, 30.0, 500.0])
    ctx = step_context([[0]], 1 << 20, [0], [5])
    state = torch.zeros(1, z.matrix + z.kept, device=DEV)
    _, steps, logs = h.ssd_prepare(proj.to(DEV), dev["conv"], dev["bias"], torch.zeros(1, device=DEV), torch.full((1,), 1.5, device=DEV), state, ctx, z, torch.float32)
    want = torch.nn.functional.softplus(proj[:, -1].to(F64), threshold=1e9)
    torch.testing.assert_close(steps[:, 0].cpu().to(F64), want, atol=0, rtol=1e-6)
    torch.testing.assert_close(logs[:, 0].cpu().to(F64), -want * torch.exp(torch.tensor(1.5, dtype=F64)), atol=0, rtol=1e-6)
    assert float(steps.min()) > 0.0 and float(steps[4, 0]) == 500.0, "no clamp on either side"


def scan_inputs(kind, dtype, lengths, gen, z, slow=False):
    """Random mixed rows (of the engine's type; places that hold no channel are zero), step sizes and log decays; `slow`:
    decays so weak that a state outlives hundreds of tokens."""
    out = []
    for n in lengths:
        m = z.spread((torch.randn(z.channels, n, generator=gen) * 0.8)).t().contiguous().to(dtype)
        d = torch.rand(n, z.heads, generator=gen) * (0.02 if slow else 1.0) + 1e-3
        rate = torch.rand(z.heads, generator=gen) * (0.05 if slow else 3.0) + 0.01
        out.append((m, d, -rate * d, rate))
    return out


def plain_scan(z, m, d, rate, skip, S=None):
    m = m.to(F64)
    n, at = m.shape[0], z.heads * z.vp
    x = m[:, :at].view(n, z.heads, z.vp)[:, :, :z.vdim]
    B, C = (m[:, at + j * z.groups * z.np:at + (j + 1) * z.groups * z.np].view(n, z.groups, z.np)[:, :, :z.state] for j in range(2))
    S = torch.zeros(z.heads, z.state, z.vdim, dtype=F64) if S is None else S
    return plain.state_space(x, B, C, d.to(F64), torch.log(rate.to(F64)), skip.to(F64), S)


@pytest.mark.parametrize("slow", [False, True])
@pytest.mark.parametrize("portions", sorted(PORTIONS))
@pytest.mark.parametrize("kind", sorted(SSD_SIZES))
@pytest.mark.parametrize("dtype", DTYPES)
def test_recurrence_over_steps_and_slots(dtype, kind, portions, slow):
    """Four requests of unequal length in packed steps of changing portions, each with its state in a slot of its own among
    slots that hold other requests' leftovers. 32-bit rows and short portions walk token by token; long portions in bfloat16
    are worked in chunks (whole ones, a chunk's rest), beside walked requests in the same step. The operands are given as
    they are, so both types are held to the same bounds."""
    h = hip()
    z, W, dev, gen = ssd_setup(kind, dtype)
    lengths, slots = [37, 1, 90, 280], [4, 0, 2, 5]
    inputs = scan_inputs(kind, dtype, lengths, gen, z, slow)
    state = torch.randn(6, z.matrix + z.kept, device=DEV)
    before = state.clone()
    state[slots, :z.matrix] = 0.0
    got = [[] for _ in lengths]
    for step, ctx in packed_steps(lengths, PORTIONS[portions], slots):
        m, d, l = (torch.cat([inputs[i][j][a:a + n] for i, a, n in step]).to(DEV) for j in range(3))
        y = h.ssd_scan(m, d, l, dev["skip"], state, ctx, z)
        at = 0
        for i, _, n in step:
            got[i].append(y[at:at + n])
            at += n
    for i, n in enumerate(lengths):
        m, d, _, rate = inputs[i]
        want, S = plain_scan(z, m, d, rate, dev["skip"].cpu())
        size = max(1.0, float(want.abs().max()))
        torch.testing.assert_close(torch.cat(got[i]).cpu().to(F64), want.reshape(n, -1), atol=3e-5 * size, rtol=3e-5)
        left = state[slots[i], :z.matrix].cpu().to(F64).view(z.heads, z.vp, z.np)
        torch.testing.assert_close(left[:, :z.vdim, :z.state], S.transpose(1, 2), atol=3e-5 * max(1.0, float(S.abs().max())), rtol=3e-5)
        assert float(left[:, z.vdim:].abs().sum()) == 0.0 and float(left[:, :, z.state:].abs().sum()) == 0.0, "places of no number stay zero"
    assert torch.equal(state[[1, 3]], before[[1, 3]]) and torch.equal(state[:, z.matrix:], before[:, z.matrix:])


@pytest.mark.parametrize("portions", ["whole", "two"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_tokens_that_forget_everything_between_tokens_that_forget_nothing(dtype, portions):
    """Log decays of -1e-4 beside ones of -30, -3,000 and -1e30: what lies between two forgetful tokens is carried as
    precisely as ever, and a forgetful token leaves nothing behind (and no NaN)."""
    h = hip()
    z, W, dev, gen = ssd_setup("plain", dtype)
    n = 280
    m, d, _, _ = scan_inputs("plain", dtype, [n], gen, z, True)[0]
    logs = torch.full((n, z.heads), -1e-4)
    for t, l in ((10, -3000.0), (11, -3000.0), (40, -30.0), (63, -3000.0), (64, -1e30), (100, -1e30), (101, -3000.0), (200, -1.0), (255, -1e30)):
        logs[t] = l
    state, out = torch.zeros(1, z.matrix + z.kept, device=DEV), []
    for step, ctx in packed_steps([n], PORTIONS[portions], [0]):
        (_, a, k), = step
        out.append(h.ssd_scan(m[a:a + k].to(DEV), d[a:a + k].to(DEV), logs[a:a + k].to(DEV), dev["skip"], state, ctx, z))
    got = torch.cat(out).cpu().to(F64)
    S, want = torch.zeros(z.heads, z.state, z.vdim, dtype=F64), []
    for t in range(n):                                       # (a rate per token that makes exp(-rate d) the decay it is to have)
        y, S = plain_scan(z, m[t:t + 1], d[t:t + 1], -(logs[t].to(F64) / d[t].to(F64)), dev["skip"].cpu(), S)
        want.append(y.reshape(-1))
    want = torch.stack(want)
    size = max(1.0, float(want.abs().max()))
    torch.testing.assert_close(got, want, atol=3e-5 * size, rtol=3e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_a_token_is_read_out_hundreds_of_tokens_later(dtype):
    """One token writes to rows of the state that no other token writes to, and one far later query reads only those rows:
    what comes back is that token's x alone, decayed by the steps between. At chunks' borders on both sides, whole and in
    portions of two."""
    h = hip()
    z, W, dev, gen = ssd_setup("plain", dtype)
    n, at = 400, z.heads * z.vp
    for src, dst in ((0, 399), (63, 64), (64, 127), (5, 191), (128, 192), (191, 193), (399, 399)):
        m = (torch.randn(n, z.row, generator=gen) * 0.5)
        B, C = (m[:, at + j * z.groups * z.np:at + (j + 1) * z.groups * z.np].view(n, z.groups, z.np) for j in range(2))
        B[:, :, 7] = C[:, :, 7] = 0.0
        B[src, :, 7] = 1.0
        C[dst] = 0.0
        C[dst, :, 7] = 2.0
        d = torch.full((n, z.heads), 0.5)
        rate = torch.linspace(1e-3, 8e-3, z.heads)
        logs = -rate * d
        for portions in ([400], [2]):
            state = torch.zeros(1, z.matrix + z.kept, device=DEV)
            out = []
            for step, ctx in packed_steps([n], portions, [0]):
                (_, a, k), = step
                out.append(h.ssd_scan(m[a:a + k].to(dtype).to(DEV), d[a:a + k].to(DEV), logs[a:a + k].to(DEV), torch.zeros(z.heads, device=DEV), state, ctx, z))
            y = torch.cat(out)[dst].cpu().to(F64).view(z.heads, z.vdim)
            x = m[src, :at].to(dtype).to(F64).view(z.heads, z.vp)[:, :z.vdim]
            want = 2.0 * 0.5 * x * torch.exp(-(dst - src) * 0.5 * rate.to(F64))[:, None]
            torch.testing.assert_close(y, want, atol=2e-5, rtol=1e-4, msg=lambda s: f"{src} read at {dst} in portions {portions}: {s}")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("width, parts", [(80, 5), (39, 3), (48, 6), (48, 48), (512, 4), (2048, 8), (4096, 8), (1024, 1), (4096, 1), (8192, 1), (10000, 1), (320, 2)])
def test_gate_before_a_norm_in_parts(dtype, width, parts):
    h = hip()
    T = 9
    y, g, w = torch.randn(T, width) * 2, torch.randn(T, width + 8) * 3, 1 + torch.randn(width) * 0.2
    y[3] *= 1e-4                                                              # (a row where eps counts)
    out = h.gated_group_norm(y.to(DEV), g.to(DEV)[:, 4:4 + width], w.to(DEV), parts, 1e-5, dtype)
    want = plain.gated_group_norm(y.to(F64), g[:, 4:4 + width].to(F64), w.to(F64), parts, 1e-5)
    torch.testing.assert_close(out.cpu().to(F64), want, **(dict(atol=2e-5, rtol=1e-5) if dtype == torch.float32 else dict(atol=1e-3, rtol=5e-3)))


@pytest.mark.parametrize("layer", ["P0", "R0", "S1", "T1"])
@pytest.mark.parametrize("dtype", DTYPES)
def test_a_whole_state_space_mixer(dtype, layer):
    from tinyserve_llm_amd.parts.base import LayerMemory
    from tinyserve_llm_amd.parts.mamba2 import Mamba2
    config = morulix_configs()[layer[0]][0]
    m = config.layers[int(layer[1])].mixer
    part = Mamba2(config.width, m.heads, m.vdim, m.state, m.groups, m.conv, m.norm_groups, config.norm_eps)
    z, gen = part.sizes, torch.Generator().manual_seed(9)
    W, params = {}, {}
    for name, spec in part.param_specs().items():
        t = torch.randn(spec.shape, generator=gen) * (spec.init[1] if name not in ("proj", "o") else spec.shape[1] ** -0.5) + spec.init[0]
        stored = t.to(torch.float32 if spec.storage == "float32" else dtype)
        params[name] = stored.to(DEV)
        W[{"proj": "in", "conv_bias": "conv.b", "a_log": "A_log", "skip": "D"}.get(name, name)] = stored.to(F64)
    W["in"] = W["in"][:z.projected]
    part.bind(params)
    x, x64 = rounded(torch.randn(150, config.width, generator=gen), dtype)
    mem = LayerMemory(state=torch.zeros(2, *part.state_spec().shape, device=DEV))
    st, out, want = {}, [], []
    for a, b in ((0, 1), (1, 3), (3, 100), (100, 101), (101, 150)):
        out.append(part.forward(x[a:b], step_context([[0]], 1 << 20, [a], [b - a], slots=[1]), mem))
        want.append(plain.mamba2(x64[a:b], W, dict(heads=m.heads, vdim=m.vdim, state=m.state, groups=m.groups, norm_groups=m.norm_groups), config.norm_eps, st))
    want = torch.cat(want)
    tol = 3e-5 if dtype == torch.float32 else 2e-2
    torch.testing.assert_close(torch.cat(out).cpu().to(F64), want, atol=tol * float(want.abs().max()), rtol=tol)
    with pytest.raises(ValueError):
        Mamba2(config.width, 4, 10, 16, 2, 4, 7, 1e-5)


# ---- whole models through trace replay ---------------------------------------------------------------

LENGTHS = {"P": [1, 23, 97, 200], "Q": [1, 30, 75, 150], "R": [2, 19, 66, 131], "S": [1, 40, 140], "T": [1, 29, 110]}
TOL = {"float32": 2e-4, "bfloat16": 6e-2}       # of the spread of the oracle's logits


@pytest.fixture(scope="module", params=["P", "Q", "R", "S", "T"])
def case(request, tmp_path_factory):
    from tinyserve_llm_amd.weights.random_init import write_random_model
    name = request.param
    config, seed = morulix_configs()[name]
    folder = str(tmp_path_factory.mktemp(f"morulix_{name}"))
    write_random_model(folder, config, seed, torch.bfloat16)
    oracle = plain.PlainMorulix.from_folder(folder)
    prompts = [prompt(500 + i, n, config.vocab) for i, n in enumerate(LENGTHS[name])]
    return name, folder, config, prompts, oracle, [oracle.logits(p) for p in prompts]


def replayer(folder, dtype, max_tokens):
    from tinyserve_llm_amd.engine.replay import Replay
    return Replay(folder, dtype, max_tokens)


def check(got, oracle_rows, dtype):
    assert got, "nothing was compared"
    spread = float(torch.cat([o.flatten() for o in oracle_rows]).std())
    worst = 0.0
    for (r, pos), row in got.items():
        want = oracle_rows[r][pos]
        torch.testing.assert_close(row.double().cpu(), want, atol=TOL[dtype] * spread, rtol=0.0,
                                   msg=lambda m: f"request {r} position {pos}: {m}")
        worst = max(worst, float((row.double().cpu() - want).abs().max()))
    print(f"[{dtype}] worst logit error {worst / spread:.3e} of the logits' spread ({spread:.2f}) over {len(got)} rows")


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
        # the residual stream after every run of a layer, one by one (a looped layer counts every time)
        from tinyserve_llm_amd.engine.runner import StepEntry
        from tinyserve_llm_amd.parts import base
        from tinyserve_llm_amd.parts.stream import ResidualStream
        p = prompts[2]
        want = oracle.streams(p)
        assert len(want) == len(rep.model.spec.order)
        rep.manager.allocate(77, p)
        ctx, _, _ = rep.runner.prepare([StepEntry(77, p, 0, [])])
        ctx.position_encodings = rep.model.position_encodings
        hidden, residual, start = rep.model.embedding.forward(ctx), None, rep.model.embedding.forward(ctx).x
        for i, (run, mem) in enumerate(zip(rep.model.spec.order, rep.runner.memory)):
            layer = rep.model.layers[run.layer]
            if run.begins is not None:
                hidden = rep.model.pass_inputs[run.begins[0]].forward(hidden, start, ctx, run.begins[1])
            hidden, residual = base.BLOCKS[layer.block](layer, hidden, residual, ctx, mem)
            now = ResidualStream(hidden.x.clone(), hidden.a, hidden.b).take()[0]
            scale = float(want[i].abs().max())
            torch.testing.assert_close(now.cpu().double(), want[i], atol=2e-5 * max(1.0, scale), rtol=1e-5, msg=lambda m: f"after layer {i}: {m}")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_prompt_then_token_by_token(case, dtype):
    """The last tokens one by one: more of them than a page, most windows hold."""
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
def test_mixed_batches_on_pages_and_slots_used_again(case, dtype):
    """Nine unequal requests, at most four live, on a pool that holds the first four: later requests start on pages and in
    state slots that earlier ones have written and given back, beside others that are in the middle of theirs. A state that is not cleared, or a stale page, shows in the logits."""
    name, folder, config, _, oracle, _ = case
    lengths = [129, 70, 40, 1, 65, 100, 128, 30, 150]
    prompts = [prompt(900 + i, n, config.vocab) for i, n in enumerate(lengths)]
    rows = [oracle.logits(p) for p in prompts]
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
def test_long_prompts_whole_and_in_long_portions(case, dtype):
    """Steps of hundreds of tokens take kernels of their own: a prompt of 520 tokens whole, and cut where the second
    portion starts in the middle of a page, of a chunk of the recurrence and of a window, beside a short request."""
    name, folder, config, _, oracle, _ = case
    long, short = prompt(321, 520, config.vocab), prompt(322, 40, config.vocab)
    rows = [oracle.logits(long), oracle.logits(short)]
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
def test_long_decoding(case, dtype):
    """300 tokens fed one by one after a prompt of five: states are carried through every step, windows
    pass over decoded tokens, latents and keys fill page after page."""
    name, folder, config, _, oracle, _ = case
    p = prompt(77, 305, config.vocab)
    rows = oracle.logits(p)
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
