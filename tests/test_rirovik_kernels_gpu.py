"""The kernel forms that came with Rirovik's mechanisms, each alone against float64: attention in a window or in chunks
that keeps the first positions, in every attention kernel, with one key that stands out just inside and just outside every
edge; head norms without scales; the query latent's norm alone; a gate per head behind the value projection; the router that
chooses by its logits; the square of relu as an experts' unit."""

import math

import pytest
import torch

pytestmark = pytest.mark.gpu

import plain_rirovik as plain  # noqa: E402
from burn_transformers_amd.kernels import library as K  # noqa: E402
from kernel_helpers import PagedCase  # noqa: E402

DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64
BOUND = {"float32": 1e-5, "bfloat16": 1.5e-2}


def rel_err(got, want):
    got = got.detach().cpu().double()
    return float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))


def seen_by(pos, window, chunk, keep):
    """The positions a query at ``pos`` sees."""
    first = max(pos - window + 1 if window else 0, pos - pos % chunk if chunk else 0, 0)
    return [p for p in range(pos + 1) if p >= first or p < keep]


def reference(case, q, q_heads, scale, window, chunk, keep, gate=None):
    hd, group = case.head_dim, q_heads // case.kv_heads
    out = torch.zeros(case.n_tokens, q_heads, hd, dtype=F64)
    row = 0
    for s, (total, count) in enumerate(zip(case.totals, case.counts)):
        k = case.k_rows[s].double().view(total, case.kv_heads, hd)
        v = case.v_rows[s].double().view(total, case.kv_heads, hd)
        for i in range(count):
            keys = seen_by(total - count + i, window, chunk, keep)
            for h in range(q_heads):
                scores = (k[keys, h // group] @ q[row, h * hd:(h + 1) * hd].double()) * scale
                out[row, h] = torch.softmax(scores, 0) @ v[keys, h // group]
            row += 1
    out = out.reshape(case.n_tokens, -1)
    return out if gate is None else out * plain.sigmoid(gate.double())


def run(case, q, q_heads, scale, window, chunk, keep, dtype, decode, impl, gate=None, runs=1):
    out = torch.full((case.n_tokens, q_heads * case.head_dim), float("nan"), dtype=DTYPES[dtype], device=DEV)
    partial = torch.full((len(case.totals) * q_heads * runs, case.head_dim + 2), float("nan"), device=DEV) if runs > 1 else None
    args = K.attention_args(q.to(DEV), out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, q_heads,
                            len(case.totals), max(case.counts), scale, window, partial, chunk=chunk, keep=keep,
                            gate=gate.to(DEV) if gate is not None else None, gate_dim=case.head_dim if gate is not None else 0)
    K.attention(args, DTYPES[dtype], decode, impl=impl)
    return out


MASKS = [(40, 0, 5), (70, 0, 66), (100, 0, 130), (1, 0, 1), (0, 50, 3), (96, 80, 64), (33, 0, 1000), (0, 0, 9)]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("q_heads,kv_heads,hd", [(4, 2, 16), (2, 1, 64), (3, 3, 48), (4, 1, 80), (2, 2, 128), (3, 1, 112)])
@pytest.mark.parametrize("window,chunk,keep", MASKS)
def test_attention_that_keeps_the_first_positions(dtype, q_heads, kv_heads, hd, window, chunk, keep):
    """Prompts behind contexts of several lengths and decode steps, whole and in runs, in the tiled and the plain kernels,
    on a cache of NaN wherever no token lies."""
    gen = torch.Generator().manual_seed(hd + window)
    for totals, counts in (([260, 9, 131], [150, 9, 40]), ([300, 70, 1, 129], [1, 1, 1, 1])):
        decode = max(counts) == 1
        case = PagedCase(totals, counts, kv_heads, hd, DTYPES[dtype], DEV, seed=hd, poison=True)
        q = torch.randn(case.n_tokens, q_heads * hd, generator=gen).to(DTYPES[dtype])
        want = reference(case, q, q_heads, 1.5 / math.sqrt(hd), window, chunk, keep)
        for impl, runs in (("auto", 1), ("plain", 1)) + ((("auto", 3),) if decode else ()):
            got = run(case, q, q_heads, 1.5 / math.sqrt(hd), window, chunk, keep, dtype, decode, impl, runs=runs)
            assert rel_err(got, want) < BOUND[dtype], (totals, impl, runs)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("hd", [32, 64, 96])
def test_kept_positions_with_a_gate_per_channel(dtype, decode, hd):
    """The modules with an output stage."""
    totals, counts = ([210, 5, 130], [1, 1, 1]) if decode else ([210, 5, 130], [100, 5, 130])
    case = PagedCase(totals, counts, 2, hd, DTYPES[dtype], DEV, seed=hd, poison=True)
    gen = torch.Generator().manual_seed(3)
    q = torch.randn(case.n_tokens, 4 * hd, generator=gen).to(DTYPES[dtype])
    gate = torch.randn(case.n_tokens, 4 * hd, generator=gen)
    got = run(case, q, 4, 0.2, 50, 0, 7, dtype, decode, "auto", gate=gate)
    assert rel_err(got, reference(case, q, 4, 0.2, 50, 0, 7, gate=gate)) < BOUND[dtype]


def test_pairs_of_query_tiles_in_a_window_that_keeps_the_first_positions():
    """Enough tiles that late and early ones share a work-group (heads up to 64, bfloat16)."""
    case = PagedCase([700, 300], [700, 300], 4, 32, torch.bfloat16, DEV, seed=5, poison=True)
    q = torch.randn(case.n_tokens, 64 * 32, generator=torch.Generator().manual_seed(1)).to(torch.bfloat16)
    got = run(case, q, 64, 0.3, 90, 0, 40, "bfloat16", False, "auto").view(case.n_tokens, 64, 32)
    for head in (0, 17, 63):            # (each head is a case of its own: its key/value head is head // 16)
        k, v = torch.cat(case.k_rows).view(-1, 4, 32)[:, head // 16].double(), torch.cat(case.v_rows).view(-1, 4, 32)[:, head // 16].double()
        for row, start in ((5, 0), (39, 0), (129, 0), (130, 0), (699, 0), (700 + 299, 700)):
            keys = [start + p for p in seen_by(row - start, 90, 0, 40)]
            w = torch.softmax((k[keys] @ q[row, head * 32:(head + 1) * 32].double()) * 0.3, 0)
            assert rel_err(got[row, head], w @ v[keys]) < 2e-2, (head, row)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("hd,impl", [(32, "auto"), (64, "auto"), (128, "auto"), (64, "plain"), (160, "plain")])
@pytest.mark.parametrize("window,keep", [(70, 10), (64, 64), (100, 65), (40, 130)])
def test_one_key_that_stands_out_at_every_edge(dtype, decode, hd, impl, window, keep):
    """One key a query's score is large for, at the start, just inside and just outside the kept positions and the window,
    at block borders and at the query itself: seen, the output is (nearly) its value; not seen, it has no part."""
    total = 321
    edge = total - window
    for place in sorted({0, keep - 1, keep, 63, 64, 127, 128, edge - 1, edge, 255, 256, total - 1}):
        case = PagedCase([total], [1 if decode else 60], 1, hd, DTYPES[dtype], DEV, seed=place)
        q = torch.zeros(case.n_tokens, hd)
        q[-1] = case.k_rows[0][place].float() * (40.0 / hd * 4)
        q = q.to(DTYPES[dtype])
        want = reference(case, q, 1, 0.5, window, 0, keep)[-1:]
        value = case.v_rows[0][place].double()
        near = float((want[0] - value).abs().max()) < 0.2 * float(value.abs().max())
        assert near == (place >= edge or place < keep), f"the premise for the key at {place}"
        got = run(case, q, 1, 0.5, window, 0, keep, dtype, decode, impl)[-1:]
        assert rel_err(got, want) < BOUND[dtype], f"the key at {place}"


def test_what_kept_positions_refuse():
    for dtype, impl in ((torch.float32, "auto"), (torch.float32, "plain"), (torch.bfloat16, "auto")):
        case = PagedCase([8], [8], 1, 64, dtype, DEV)
        q, out = torch.zeros(8, 64, device=DEV, dtype=dtype), torch.zeros(8, 64, device=DEV, dtype=dtype)
        args = K.attention_args(q, out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, 1, 1, 8, 0.1, window=3, keep=-1)
        with pytest.raises(K.KernelError, match="kept"):
            K.attention(args, dtype, False, impl=impl)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("span", ["channel", "head"])
@pytest.mark.parametrize("tokens", [1, 17, 32, 33, 100])
@pytest.mark.parametrize("heads,vdim,rank,pitch", [(3, 24, 40, 48), (5, 130, 70, 80), (1, 1, 1, 16)])
def test_value_projection_with_a_gate_per_head_or_output(dtype, span, tokens, heads, vdim, rank, pitch):
    gen = torch.Generator().manual_seed(tokens)
    ctx = torch.randn(tokens, heads * pitch, generator=gen).to(DTYPES[dtype])
    weight = (torch.randn(heads * vdim, rank, generator=gen) / math.sqrt(rank)).to(DTYPES[dtype])
    gate = torch.randn(tokens, heads * vdim + 3 if span == "channel" else heads + 2, generator=gen) * 2.0
    out = torch.full((tokens, heads * vdim + 5), float("nan"), dtype=DTYPES[dtype], device=DEV)
    K.head_project(ctx.to(DEV), weight.to(DEV), heads, vdim, rank, pitch, out, gate=gate.to(DEV), gate_span=span)
    want = torch.einsum("thr,hvr->thv", ctx.double().view(tokens, heads, pitch)[..., :rank], weight.double().view(heads, vdim, rank))
    factor = plain.sigmoid(gate.double())
    factor = factor[:, :heads * vdim].view(tokens, heads, vdim) if span == "channel" else factor[:, :heads, None]
    assert rel_err(out[:, :heads * vdim], (want * factor).reshape(tokens, -1)) < (1e-5 if dtype == "float32" else 1e-2)
    assert float(out[:, heads * vdim:].float().abs().max()) == 0.0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("q_rank", [7, 24, 300])
def test_the_query_latents_norm_alone(dtype, q_rank):
    """A layer that borrows another's latent: nothing goes to the cache."""
    case = PagedCase([5], [5], 1, 32, DTYPES[dtype], DEV, seed=1)
    before = case.keys.clone(), case.values.clone()
    gen = torch.Generator().manual_seed(q_rank)
    fused, gamma = torch.randn(5, q_rank + 6, generator=gen), torch.randn(q_rank, generator=gen)
    out = torch.full((5, q_rank + 3), float("nan"), dtype=DTYPES[dtype], device=DEV)
    K.latent_norm(fused.to(DEV), q_rank, (q_rank + 3) // 4 * 4, 0, gamma.to(DEV), None, 1e-4, out, case.tok_seq, case.tok_pos, case.view(), DTYPES[dtype])
    assert rel_err(out[:, :q_rank], plain.unit_rms(fused.double()[:, :q_rank], 1e-4) * gamma.double()) < (1e-5 if dtype == "float32" else 1e-2)
    assert float(out[:, q_rank:].float().abs().max()) == 0.0
    assert torch.equal(case.keys, before[0]) and torch.equal(case.values, before[1])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("experts,top,width,tokens", [(5, 2, 40, 9), (11, 4, 304, 33), (1, 1, 24, 3), (200, 7, 130, 300), (64, 64, 64, 5)])
@pytest.mark.parametrize("spread", [1.0, 60.0])
def test_router_that_weighs_by_the_softmax_over_the_chosen(dtype, experts, top, width, tokens, spread):
    """Logits with a bias; also so far apart that a softmax over all of them would leave only zeros behind the first."""
    gen = torch.Generator().manual_seed(experts)
    h = torch.randn(tokens, width, generator=gen).to(DTYPES[dtype])
    W = torch.randn(experts, width, generator=gen) * spread / math.sqrt(width)
    bias = torch.randn(experts, generator=gen) * 2.0
    weights = torch.full((tokens, experts), float("nan"), device=DEV)
    K.route(h.to(DEV), W.to(DEV), None, top, 1, 1, weights, score="chosen", bias=bias.to(DEV))
    z = h.double() @ W.double().T + bias.double()
    got = weights.cpu().double()
    for t in range(tokens):
        chosen, w = plain.choice(z[t], top)
        want = torch.zeros(experts, dtype=F64)
        want[chosen] = w
        ranked = z[t].sort(descending=True).values
        if top < experts and float(ranked[top - 1] - ranked[top]) < 1e-4 * spread:      # a close call
            continue
        assert float((got[t] - want).abs().max()) < 2e-5 * spread, t
    assert torch.allclose(got.sum(1), torch.ones(tokens, dtype=F64), atol=1e-5)


def test_router_bias_goes_with_every_score():
    gen = torch.Generator().manual_seed(9)
    h, W, bias = torch.randn(7, 32, generator=gen), torch.randn(6, 32, generator=gen), torch.randn(6, generator=gen)
    z = h.double() @ W.double().T + bias.double()
    for score, s in (("softmax", torch.softmax(z, 1)), ("sigmoid", plain.sigmoid(z))):
        weights = torch.zeros(7, 6, device=DEV)
        K.route(h.to(DEV), W.to(DEV), None, 6, 1, 1, weights, score=score, bias=bias.to(DEV), normalize=False)
        assert rel_err(weights, s) < 1e-5
    with pytest.raises(K.KernelError):
        K.route(h.to(DEV), W.to(DEV), None, 2, 1, 1, torch.zeros(7, 6, device=DEV), score="chosen", normalize=False)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("experts,ff,shared", [(4, 12, 20), (3, 5, 0), (1, 8, 8), (1, 1, 1)])
def test_squared_relu_as_an_experts_unit(dtype, experts, ff, shared):
    gen = torch.Generator().manual_seed(experts)
    tokens, inner = 19, experts * ff + shared
    up = torch.randn(tokens, inner + 3, generator=gen).to(DTYPES[dtype])
    weights = torch.rand(tokens, experts, generator=gen)
    weights[weights < 0.4] = 0.0
    hidden = torch.full((tokens, inner + 2), float("nan"), dtype=DTYPES[dtype], device=DEV)
    K.gated_experts(up.to(DEV), weights.to(DEV), None, experts, ff, shared, 0, hidden, unit="squared_relu")
    want = plain.squared_relu(up.double()[:, :inner])
    want[:, :experts * ff] *= weights.double().repeat_interleave(ff, dim=1)
    assert rel_err(hidden[:, :inner], want) < (1e-6 if dtype == "float32" else 1e-2)
    assert float(hidden[:, inner:].float().abs().max()) == 0.0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("m", [1, 8, 16, 17, 33, 64])
@pytest.mark.parametrize("heads,pitch,at,dims,k", [(3, 48, 32, 16, 40), (5, 16, 10, 6, 96), (2, 128, 0, 128, 24), (1, 4, 2, 2, 8), (16, 128, 96, 32, 384)])
def test_a_product_that_turns_columns_by_the_rows_positions(dtype, m, heads, pitch, at, dims, k):
    """Plain and packed weights; turned ranges that begin inside four columns; positions up to some thousands."""
    gen = torch.Generator().manual_seed(m + pitch)
    n, amplitude = heads * pitch, 1.25
    a, w = torch.randn(m, k, generator=gen).to(DTYPES[dtype]), (torch.randn(n, k, generator=gen) / math.sqrt(k)).to(DTYPES[dtype])
    positions = torch.randint(0, 3000, (m,), generator=gen)
    positions[0] = 0
    rot = {"dims": dims, "base": 700.0}
    want = (a.double() @ w.double().T).view(m, heads, pitch)
    want[..., at:at + dims] = amplitude * plain.turn(want[..., at:at + dims], positions, rot)
    freq = torch.tensor([700.0 ** (-2.0 * i / dims) for i in range(dims // 2)]).to(DEV)
    bound = 1e-3 if dtype == "float32" else 1e-2        # (angles are 32-bit products: at position 3,000 they are off by 2e-4)
    out = torch.full((m, n + 4), float("nan"), dtype=DTYPES[dtype], device=DEV)[:, :n]
    on_gpu = positions.to(torch.int32).to(DEV)          # (an epilogue holds addresses: what they name stays here)
    epilogue = K.epilogue_turn(out, pitch, at, dims, freq, on_gpu, amplitude)
    K.gemm(a.to(DEV), w.to(DEV), epilogue)
    assert rel_err(out, want.reshape(m, n)) < bound
    first = out.clone()
    K.gemm(a.to(DEV), w.to(DEV), epilogue, packed=(K.pack_columns(w.to(DEV), 16), 16))
    assert torch.equal(first, out)


@pytest.mark.parametrize("m", [1, 7, 16])
def test_a_turning_product_that_normalises_its_rows_itself(m):
    gen = torch.Generator().manual_seed(m)
    k, heads, pitch, at, dims, eps = 72, 4, 32, 20, 12, 1e-4
    fused, gamma = torch.randn(m, k + 8, generator=gen), torch.randn(k, generator=gen)
    w = (torch.randn(heads * pitch, k, generator=gen) / 8).to(torch.bfloat16)
    positions = torch.arange(m) * 5 + 3
    c = (plain.unit_rms(fused[:, :k].double(), eps) * gamma.double()).to(torch.bfloat16).double()
    want = (c @ w.double().T).view(m, heads, pitch)
    want[..., at:at + dims] = plain.turn(want[..., at:at + dims], positions, {"dims": dims, "base": 50.0})
    freq = torch.tensor([50.0 ** (-2.0 * i / dims) for i in range(dims // 2)]).to(DEV)
    out = torch.zeros(m, heads * pitch, dtype=torch.bfloat16, device=DEV)
    held = fused.to(DEV), gamma.to(DEV), positions.to(torch.int32).to(DEV)
    K.gemm(K.Normalized(held[0][:, :k], held[1], None, eps, "rms_norm"), w.to(DEV), K.epilogue_turn(out, pitch, at, dims, freq, held[2]))
    assert rel_err(out, want.reshape(m, -1)) < 1.5e-2


def test_what_a_turning_product_refuses():
    a, w, out = torch.zeros(4, 16, device=DEV), torch.zeros(32, 16, device=DEV), torch.zeros(4, 32, device=DEV)
    freq, pos = torch.ones(8, device=DEV), torch.zeros(4, dtype=torch.int32, device=DEV)
    for pitch, at, dims in ((16, 1, 4), (16, 0, 3), (16, 14, 4), (6, 0, 2), (20, 0, 4)):
        with pytest.raises(K.KernelError):
            K.gemm(a, w, K.epilogue_turn(out, pitch, at, dims, freq, pos))
    with pytest.raises(K.KernelError):
        K.gemm(a, w, K.epilogue_turn(out, 16, 0, 4, freq, pos), impl="tile")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("experts,ff,shared,top,tokens", [(8, 1024, 64, 2, 8), (5, 7, 0, 3, 64), (3, 16, 9, 1, 1), (130, 8, 8, 6, 20), (1, 1, 1, 1, 2)])
@pytest.mark.parametrize("score", ["chosen", "softmax", "sigmoid"])
def test_units_weighed_by_logits_that_came_with_them(dtype, experts, ff, shared, top, tokens, score):
    """The same weights as the router kernel's, on the units in place; columns behind the experts stay; an unchosen
    expert's units are zero whatever they were."""
    gen = torch.Generator().manual_seed(experts + tokens)
    logits = torch.randn(tokens, experts + 3, generator=gen) * 3.0
    bias = torch.randn(experts, generator=gen)
    z = (logits[:, :experts] + bias).double()
    weights = torch.zeros(tokens, experts, dtype=F64)
    s = {"chosen": torch.exp(z - z.max(1, keepdim=True).values), "softmax": torch.softmax(z, 1), "sigmoid": plain.sigmoid(z)}[score]
    for t in range(tokens):
        chosen = z[t].argsort(descending=True)[:top]
        weights[t, chosen] = s[t, chosen] / s[t, chosen].sum()
    hidden = torch.randn(tokens, experts * ff + shared + 5, generator=gen).to(DTYPES[dtype])
    want = hidden.double()
    want[:, :experts * ff] *= weights.repeat_interleave(ff, dim=1)
    if top < experts:
        hidden[0, int(z[0].argmin()) * ff] = float("inf")
    rows = hidden.to(DEV)
    K.weigh_experts(logits.to(DEV), bias.to(DEV), None, top, 1, 1, rows, experts, ff, score=score)
    assert rel_err(rows, want) < (1e-5 if dtype == "float32" else 1e-2)
    assert torch.equal(rows[:, experts * ff:].cpu(), hidden[:, experts * ff:])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("unit", ["squared_relu", "gelu_erf", "silu"])
def test_units_taken_sixteen_bytes_at_a_time(dtype, unit):
    gen = torch.Generator().manual_seed(2)
    tokens, experts, ff, shared = 70, 3, 1032, 24
    inner = experts * ff + shared
    up = torch.randn(tokens, inner + 8, generator=gen).to(DTYPES[dtype])
    weights = torch.rand(tokens, experts, generator=gen)
    weights[weights < 0.4] = 0.0
    hidden = torch.full((tokens, inner + 8), float("nan"), dtype=DTYPES[dtype], device=DEV)
    K.gated_experts(up.to(DEV), weights.to(DEV), None, experts, ff, shared, 0, hidden, unit=unit)
    act = {"squared_relu": plain.squared_relu, "silu": lambda z: z * plain.sigmoid(z),
           "gelu_erf": lambda z: 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))}[unit]
    want = act(up.double()[:, :inner])
    want[:, :experts * ff] *= weights.double().repeat_interleave(ff, dim=1)
    assert rel_err(hidden[:, :inner], want) < (1e-6 if dtype == "float32" else 1e-2)
    assert float(hidden[:, inner:].float().abs().max()) == 0.0


SHARED = [(1, 144), (3, 64), (16, 128), (16, 576), (20, 96), (33, 320), (5, 512), (128, 192), (2, 640), (17, 768)]


@pytest.mark.parametrize("heads,hd", SHARED)
@pytest.mark.parametrize("window,keep", [(0, 0), (70, 0), (100, 66), (1, 1)])
def test_attention_on_one_shared_head(heads, hd, window, keep):
    """Prompts behind contexts, portions of a few tokens and decode steps, whole and in runs (more of them than some
    sequences have blocks), with and without a last part of the value that is not read, on a cache of NaN wherever no token
    lies."""
    gen = torch.Generator().manual_seed(hd + heads)
    for totals, counts in (([200, 9, 131], [40, 9, 3]), ([330, 70, 1, 129], [1, 1, 1, 1])):
        case = PagedCase(totals, counts, 1, hd, torch.bfloat16, DEV, seed=hd, poison=True)
        q = (torch.randn(case.n_tokens, heads * hd, generator=gen) * 2.0 / math.sqrt(hd)).to(torch.bfloat16)
        whole = reference(case, q, heads, 1.0, window, 0, keep).view(case.n_tokens, heads, hd)
        for value_dim, runs in ((0, 1), (hd - hd // 5 // 4 * 4, 1), (hd - 16, 3), (0, 8)):
            out = torch.full((case.n_tokens, heads * hd), float("nan"), dtype=torch.bfloat16, device=DEV)
            partial = torch.full((case.n_tokens * heads * runs, hd + 2), float("nan"), device=DEV) if runs > 1 else None
            args = K.attention_args(q.to(DEV), out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, heads,
                                    len(totals), max(counts), 1.0, window, partial, runs=runs if runs > 1 else None, keep=keep, value_dim=value_dim)
            K.attention(args, torch.bfloat16, max(counts) == 1, impl="shared")
            want = whole.clone()
            if value_dim:
                want[..., value_dim:] = 0.0
            assert rel_err(out, want.reshape(case.n_tokens, -1)) < 1.5e-2, (totals, value_dim, runs)
            assert not value_dim or float(out.view(case.n_tokens, heads, hd)[..., value_dim:].float().abs().max()) == 0.0


@pytest.mark.parametrize("hd", [96, 320, 576])
@pytest.mark.parametrize("runs", [1, 4])
@pytest.mark.parametrize("span", ["head", "channel", None])
def test_shared_head_with_a_gate_a_sink_and_chunk_major_rows(hd, runs, span):
    totals, heads = [150, 300, 7, 64, 65, 1, 129, 200, 30, 90], 18
    case = PagedCase(totals, [1] * len(totals), 1, hd, torch.bfloat16, DEV, seed=hd, poison=True)
    gen = torch.Generator().manual_seed(hd)
    q = (torch.randn(case.n_tokens, heads * hd, generator=gen) / math.sqrt(hd)).to(torch.bfloat16)
    sink = torch.randn(heads, generator=gen) + 2.0
    gate = {"head": torch.randn(case.n_tokens, heads + 2, generator=gen), "channel": torch.randn(case.n_tokens, heads * hd, generator=gen), None: None}[span]
    want = torch.zeros(case.n_tokens, heads, hd, dtype=F64)
    for s, total in enumerate(totals):
        k, v = case.k_rows[s].double(), case.v_rows[s].double()
        for h in range(heads):
            scores = torch.cat([k @ q[s, h * hd:(h + 1) * hd].double() * 2.0, sink[h:h + 1].double()])
            want[s, h] = torch.softmax(scores, 0)[:-1] @ v
    if span == "head":
        want *= plain.sigmoid(gate.double())[:, :heads, None]
    want = want.reshape(case.n_tokens, -1) * (plain.sigmoid(gate.double()) if span == "channel" else 1.0)
    columns = heads * hd
    chunked = K.Chunked(torch.zeros(case.n_tokens, (columns + 31) // 32 * 32, dtype=torch.bfloat16, device=DEV), case.n_tokens, columns)
    row_major = torch.zeros(case.n_tokens, columns, dtype=torch.bfloat16, device=DEV)
    partial = torch.full((case.n_tokens * heads * runs, hd + 2), float("nan"), device=DEV) if runs > 1 else None
    held = q.to(DEV), sink.to(DEV), gate.to(DEV) if gate is not None else None
    for out in (chunked, row_major):
        args = K.attention_args(held[0], out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, heads, len(totals), 1,
                                2.0, 0, partial, sink=held[1], gate=held[2], gate_dim=hd if span == "channel" else 0)
        K.attention(args, torch.bfloat16, True, impl="shared")
    assert rel_err(row_major, want) < 1.5e-2
    assert torch.equal(chunked.to_rows(), row_major)


@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("window,keep", [(70, 10), (64, 64), (100, 65)])
def test_one_key_that_stands_out_on_a_shared_head(decode, window, keep):
    hd, total, heads = 320, 321, 3
    edge = total - window
    for place in sorted({0, keep - 1, keep, 63, 64, 127, 128, edge - 1, edge, 255, 256, total - 1}):
        case = PagedCase([total], [1 if decode else 60], 1, hd, torch.bfloat16, DEV, seed=place)
        q = torch.zeros(case.n_tokens, heads * hd)
        q[-1] = case.k_rows[0][place].float().repeat(heads) * 0.5
        q = q.to(torch.bfloat16)
        want = reference(case, q, heads, 0.5, window, 0, keep)[-1:]
        value = case.v_rows[0][place].double().repeat(heads)
        assert (float((want[0] - value).abs().max()) < 0.2 * float(value.abs().max())) == (place >= edge or place < keep), f"the premise for the key at {place}"
        got = run(case, q, heads, 0.5, window, 0, keep, "bfloat16", decode, "shared")[-1:]
        assert rel_err(got, want) < 1.5e-2, f"the key at {place}"


def test_what_the_shared_head_refuses():
    case = PagedCase([8], [8], 2, 64, torch.bfloat16, DEV)
    one = PagedCase([8], [8], 1, 64, torch.bfloat16, DEV)
    q, out = torch.zeros(8, 128, device=DEV, dtype=torch.bfloat16), torch.zeros(8, 128, device=DEV, dtype=torch.bfloat16)
    for c, options in ((case, {}), (one, {"softcap": 1.0}), (one, {"value_dim": 66}), (one, {"value_dim": 80})):
        args = K.attention_args(q, out, c.view(), c.tok_seq, c.tok_pos, c.seq_off, c.seq_start, 2, 1, 8, 0.1, **options)
        with pytest.raises(K.KernelError):
            K.attention(args, torch.bfloat16, False, impl="shared")
