"""The kernel forms that came with Loselix's mechanisms, each alone against float64: attention with capped scores, with
sigmoid weights and with an output stage (plain, tiled and decode kernels, in runs too), queries and keys in two maps,
values taken from the keys, a temperature, the difference of two maps, a product that leaves 32-bit and activated
columns, the square of relu."""

import math

import pytest
import torch

pytestmark = pytest.mark.gpu

import plain_loselix as plain  # noqa: E402
from burn_transformers_amd.kernels import library as K  # noqa: E402
from burn_transformers_amd.parts.rotary_attention import rotary_frequencies  # noqa: E402
from kernel_helpers import PagedCase  # noqa: E402

DEV = "cuda:0"
DTYPES = {"float32": torch.float32, "bfloat16": torch.bfloat16}
F64 = torch.float64


def rel_err(got, want):
    got = got.detach().cpu().double()
    assert torch.isfinite(got).all()
    return float((got - want).abs().max() / want.abs().max().clamp_min(1e-30))


def reference(case, q, q_heads, scale, form, cap, bias, gate, gate_dim):
    """float64 attention of the step's queries with a form of the scores and a gate."""
    hd, group = case.head_dim, q_heads // case.kv_heads
    out = torch.zeros(case.n_tokens, q_heads, hd, dtype=F64)
    row = 0
    for s, (total, count) in enumerate(zip(case.totals, case.counts)):
        k = case.k_rows[s].double().view(total, case.kv_heads, hd)
        v = case.v_rows[s].double().view(total, case.kv_heads, hd)
        for i in range(count):
            seen = total - count + i + 1
            for h in range(q_heads):
                scores = (k[:seen, h // group] @ q[row, h * hd:(h + 1) * hd].double()) * scale
                if form == "capped":
                    scores = plain.softcap(scores, cap)
                weights = plain.sigmoid(scores + bias[h]) if form == "sigmoid" else torch.softmax(scores, 0)
                out[row, h] = weights @ v[:seen, h // group]
            row += 1
    if gate is not None:
        g = plain.sigmoid(gate.double())
        if gate_dim:
            factor = torch.ones(case.n_tokens, q_heads, hd, dtype=F64)
            factor[..., :gate_dim] = g[:, :q_heads * gate_dim].view(case.n_tokens, q_heads, gate_dim)
            out = out * factor
        else:
            out = out * g[:, :q_heads, None]
    return out.reshape(case.n_tokens, -1)


def run_case(dtype, form, gate_kind, totals, counts, q_heads, kv_heads, hd, impl="auto", runs=None, f32_out=False, seed=0, far=None):
    case = PagedCase(totals, counts, kv_heads, hd, DTYPES[dtype], DEV, seed=seed, poison=True)
    gen = torch.Generator().manual_seed(seed + 1)
    q = (torch.randn(case.n_tokens, q_heads * hd, generator=gen) * 0.6).to(DTYPES[dtype])
    scale, cap = 1.0 / math.sqrt(hd), 4.0
    bias = torch.randn(q_heads, generator=gen) - 2.0 if form == "sigmoid" else None
    gate_dim = {None: 0, "head": 0, "channel": hd - 3}[gate_kind]
    gate = None if gate_kind is None else torch.randn(case.n_tokens, (q_heads * gate_dim if gate_dim else q_heads) + 5, generator=gen)
    decode = max(counts) == 1
    out = torch.full((case.n_tokens, q_heads * hd), float("nan"), dtype=torch.float32 if f32_out else DTYPES[dtype], device=DEV)
    partial = torch.full((len(totals) * q_heads * runs, hd + 2), float("nan"), device=DEV) if runs else None
    args = K.attention_args(q.to(DEV), out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, q_heads, len(totals),
                            max(counts), scale, 0, partial, softcap=cap if form == "capped" else 0.0, sigmoid=form == "sigmoid",
                            score_bias=bias.to(DEV) if bias is not None else None, gate=gate.to(DEV) if gate is not None else None,
                            gate_dim=gate_dim)
    K.attention(args, DTYPES[dtype], decode, impl=impl)
    torch.cuda.synchronize()
    want = reference(case, q, q_heads, scale, form, cap, bias, gate, gate_dim)
    bound = 1e-5 if dtype == "float32" else 1.5e-2
    assert rel_err(out, want) < bound, f"{dtype} {form} {gate_kind} {totals} {counts} heads {q_heads}/{kv_heads} of {hd} {impl} runs {runs}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("form,gate", [("softmax", "head"), ("softmax", "channel"), ("capped", None), ("capped", "head"), ("sigmoid", None),
                                       ("sigmoid", "channel")])
@pytest.mark.parametrize("hd", [16, 48, 64, 96, 128])
def test_forms_of_the_scores_and_the_output_stage_in_the_tiled_kernels(dtype, form, gate, hd):
    """Prompts, chunks behind a context and decode steps; unequal sequences; blocks' unused places hold NaN."""
    run_case(dtype, form, gate, [70, 5, 200], [70, 5, 130], 4, 2, hd, seed=hd)
    run_case(dtype, form, gate, [150, 1, 65], [1, 1, 1], 6, 2, hd, seed=hd + 1)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("form,gate", [("softmax", "channel"), ("capped", "head"), ("sigmoid", "channel")])
@pytest.mark.parametrize("hd,impl", [(20, "plain"), (128, "plain"), (208, "plain"), (64, "auto"), (128, "auto")])
def test_the_plain_kernel_and_decoding_in_runs(dtype, form, gate, hd, impl):
    if impl == "plain":
        run_case(dtype, form, gate, [90, 7], [20, 7], 4, 2, hd, impl="plain", seed=hd)
        run_case(dtype, form, gate, [1100], [1], 2, 1, hd, impl="plain", seed=hd)
    else:                     # five runs of the keys, some of them empty for the short sequence
        run_case(dtype, form, gate, [700, 40], [1, 1], 4, 2, hd, runs=5, seed=hd)


@pytest.mark.parametrize("form", ["softmax", "capped", "sigmoid"])
@pytest.mark.parametrize("hd", [48, 64, 128])
def test_32_bit_rows_of_bfloat16_attention(form, hd):
    for totals, counts, runs in (([130, 9], [130, 9], None), ([100, 3], [1, 1], None), ([600, 30], [1, 1], 3)):
        run_case("bfloat16", form, "head" if form == "sigmoid" else None, totals, counts, 4, 2, hd, runs=runs, f32_out=True, seed=hd)
    run_case("bfloat16", form, None, [40], [40], 2, 1, hd, impl="plain", f32_out=True, seed=hd)


@pytest.mark.parametrize("hd", [64, 80, 96, 112, 128])
def test_chunks_of_prompts_in_runs(hd):
    """The prompt kernels of heads of 64 to 128 with their keys in runs (joined by a second kernel), some of them empty for
    the early tiles and the short sequence, all forms; a gate whose rows take 16-byte loads and one whose rows do not."""
    for number, form in enumerate(("softmax", "capped", "sigmoid")):
        counts, totals, runs = [130, 40], [900, 40], 5
        case = PagedCase(totals, counts, 2, hd, torch.bfloat16, DEV, seed=3, poison=True)
        gen = torch.Generator().manual_seed(1)
        tokens = sum(counts)
        q = (torch.randn(tokens, 4 * hd, generator=gen) * 0.6).to(torch.bfloat16)
        gate = torch.randn(tokens, 4 * hd + number, generator=gen)
        bias = torch.randn(4, generator=gen) - 2.0 if form == "sigmoid" else None
        out = torch.full((tokens, 4 * hd), float("nan"), dtype=torch.bfloat16, device=DEV)
        partial = torch.full((tokens * 4 * runs, hd + 2), float("nan"), device=DEV)
        args = K.attention_args(q.to(DEV), out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, 4, 2, 130, 0.125, 0,
                                partial, runs=runs, softcap=4.0 if form == "capped" else 0.0, sigmoid=form == "sigmoid",
                                score_bias=bias.to(DEV) if bias is not None else None, gate=gate.to(DEV), gate_dim=hd)
        K.attention(args, torch.bfloat16, False)
        assert rel_err(out, reference(case, q, 4, 0.125, form, 4.0, bias, gate, hd)) < 1.5e-2, form


@pytest.mark.parametrize("hd", [80, 96, 112, 128])
@pytest.mark.parametrize("window,chunk", [(0, 0), (70, 0), (1, 0), (200, 0), (0, 50), (0, 128), (90, 100)])
def test_prompts_of_wide_heads_with_windows_and_chunks(hd, window, chunk):
    """The prompt kernel of heads of 80 to 128: windows and chunks that begin inside blocks, at their borders and blocks
    apart; prompts and chunks of prompts of unequal sequences, one cached head for many query heads, many units."""
    for q_heads, kv_heads, totals, counts in ((4, 1, [300, 5], [300, 5]), (6, 2, [500, 129, 64, 1, 260], [140, 129, 64, 1, 2])):
        case = PagedCase(totals, counts, kv_heads, hd, torch.bfloat16, DEV, seed=hd, poison=True)
        gen = torch.Generator().manual_seed(window + chunk)
        q = (torch.randn(case.n_tokens, q_heads * hd, generator=gen) * 0.6).to(torch.bfloat16)
        out = torch.full((case.n_tokens, q_heads * hd), float("nan"), dtype=torch.bfloat16, device=DEV)
        args = K.attention_args(q.to(DEV), out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, q_heads,
                                len(totals), max(counts), 1.0 / math.sqrt(hd), window, chunk=chunk)
        K.attention(args, torch.bfloat16, False)
        want = torch.zeros(case.n_tokens, q_heads, hd, dtype=F64)
        row = 0
        for s, (total, count) in enumerate(zip(totals, counts)):
            k = case.k_rows[s].double().view(total, kv_heads, hd)
            v = case.v_rows[s].double().view(total, kv_heads, hd)
            for pos in range(total - count, total):
                lo = max(pos - window + 1 if window else 0, pos - pos % chunk if chunk else 0, 0)
                for h in range(q_heads):
                    j = h // (q_heads // kv_heads)
                    scores = (k[lo:pos + 1, j] @ q[row, h * hd:(h + 1) * hd].double()) / math.sqrt(hd)
                    want[row, h] = torch.softmax(scores, 0) @ v[lo:pos + 1, j]
                row += 1
        assert rel_err(out, want.reshape(case.n_tokens, -1)) < 1.5e-2, (q_heads, totals, counts)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("decode", [False, True])
@pytest.mark.parametrize("form", ["capped", "sigmoid"])
def test_one_key_that_stands_out(dtype, decode, form):
    """A key that is the only one a query's score is large for, at the start, around block borders and at the query
    itself: the output is (nearly) that key's value."""
    hd, total = 64, 321
    for place in (0, 63, 64, 127, 128, 255, 256, 319, 320):
        case = PagedCase([total], [1 if decode else 70], 1, hd, DTYPES[dtype], DEV, seed=place)
        q = torch.zeros(case.n_tokens, hd)
        q[-1] = case.k_rows[0][place].float() * 20.0
        q = q.to(DTYPES[dtype])
        bias = torch.full((1,), -40.0)
        out = torch.zeros(case.n_tokens, hd, dtype=DTYPES[dtype], device=DEV)
        args = K.attention_args(q.to(DEV), out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, 1, 1,
                                1 if decode else 70, 0.125, 0, softcap=40.0 if form == "capped" else 0.0, sigmoid=form == "sigmoid",
                                score_bias=bias.to(DEV) if form == "sigmoid" else None)
        K.attention(args, DTYPES[dtype], decode)
        want = reference(case, q, 1, 0.125, form, 40.0, bias, None, 0)
        value = case.v_rows[0][place].double()
        assert float((want[-1] - value).abs().max()) < 0.2 * float(value.abs().max())        # the premise
        assert rel_err(out[-1:], want[-1:]) < (1e-5 if dtype == "float32" else 1.5e-2), f"the key at {place}"


def test_what_the_forms_refuse():
    case = PagedCase([8], [8], 1, 64, torch.float32, DEV)
    q, out = torch.zeros(8, 64, device=DEV), torch.zeros(8, 64, device=DEV)
    base = (q, out, case.view(), case.tok_seq, case.tok_pos, case.seq_off, case.seq_start, 1, 1, 8, 0.1)
    for impl in ("auto", "plain"):
        with pytest.raises(K.KernelError, match="sink"):
            K.attention(K.attention_args(*base, sigmoid=True, sink=torch.zeros(1, device=DEV)), torch.float32, False, impl=impl)
        with pytest.raises(K.KernelError, match="gate"):
            K.attention(K.attention_args(*base, gate=torch.zeros(8, 10, device=DEV), gate_dim=64), torch.float32, False, impl=impl)
        with pytest.raises(K.KernelError, match="bias"):
            K.attention(K.attention_args(*base, score_bias=torch.zeros(1, device=DEV), softcap=1.0), torch.float32, False, impl=impl)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,kv_heads,dim,vdim,rot_dims,hd", [(4, 2, 24, 40, 12, 48), (3, 3, 5, 13, 2, 16), (2, 1, 64, 128, 64, 128), (1, 1, 7, 9, 0, 16)])
def test_two_maps_into_one_cached_head(dtype, heads, kv_heads, dim, vdim, rot_dims, hd):
    totals = [70, 3]
    case = PagedCase(totals, totals, kv_heads, hd, DTYPES[dtype], DEV, seed=2, poison=True)
    gen = torch.Generator().manual_seed(1)
    tokens, n_q, n_k = sum(totals), heads * 2 * dim, kv_heads * 2 * dim
    fused = torch.randn(tokens, n_q + n_k + kv_heads * vdim + 3, generator=gen)
    q_out = torch.full((tokens, heads * 2 * hd), float("nan"), dtype=DTYPES[dtype], device=DEV)
    inv = rotary_frequencies(rot_dims, 100.0).float().to(DEV) if rot_dims else None
    K.head_rotary(fused.to(DEV), heads, kv_heads, dim, vdim, rot_dims, inv, None, None, 0.0, q_out, case.tok_seq, case.tok_pos, case.view(),
                  DTYPES[dtype], maps=2)
    positions = torch.cat([torch.arange(t) for t in totals])
    rot, f = {"dims": rot_dims, "base": 100.0}, fused.double()
    bound = 1e-5 if dtype == "float32" else 1e-2
    q = plain.turn(f[:, :n_q].view(tokens, 2 * heads, dim), positions, rot).view(tokens, heads, 2, dim)
    want = torch.zeros(tokens, heads, 2, hd, dtype=F64)
    want[:, :, 0, :dim], want[:, :, 1, dim:2 * dim] = q[:, :, 0], q[:, :, 1]
    assert rel_err(q_out, want.reshape(tokens, -1)) < bound
    assert float(q_out.view(tokens, heads, 2, hd)[:, :, 0, dim:].float().abs().max()) == 0.0
    keys, values = case.read_back()
    k = plain.turn(f[:, n_q:n_q + n_k].view(tokens, 2 * kv_heads, dim), positions, rot).reshape(tokens, kv_heads, 2 * dim)
    assert rel_err(keys.view(tokens, kv_heads, hd)[..., :2 * dim], k) < bound
    assert rel_err(values.view(tokens, kv_heads, hd)[..., :vdim], f[:, n_q + n_k:n_q + n_k + kv_heads * vdim].view(tokens, kv_heads, vdim)) < bound
    for rows, own in ((keys, 2 * dim), (values, vdim)):
        assert own == hd or float(rows.view(tokens, kv_heads, hd)[..., own:].float().abs().max()) == 0.0


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("every", [1, 7, 64])
def test_values_from_keys_whole_norms_and_a_temperature(dtype, every):
    """The values are the key columns before their norm; queries grow where position + 1 reaches a multiple of ``every``."""
    heads, kv_heads, dim, hd, coef, eps = 4, 2, 20, 32, 0.35, 1e-4
    totals, starts = [140, 3], [0, 0]
    case = PagedCase(totals, totals, kv_heads, hd, DTYPES[dtype], DEV, seed=4, poison=True)
    gen = torch.Generator().manual_seed(every)
    tokens, n_q, n_k = sum(totals), heads * dim, kv_heads * dim
    fused = torch.randn(tokens, n_q + n_k + 7, generator=gen)
    q_gamma, k_gamma = torch.randn(n_q, generator=gen), torch.randn(n_k, generator=gen)
    q_out = torch.full((tokens, heads * hd), float("nan"), dtype=DTYPES[dtype], device=DEV)
    K.head_rotary(fused.to(DEV), heads, kv_heads, dim, dim, 0, None, q_gamma.to(DEV), k_gamma.to(DEV), eps, q_out, case.tok_seq, case.tok_pos,
                  case.view(), DTYPES[dtype], whole_norm=True, values_from_keys=True, temperature=(coef, every))
    positions = torch.cat([torch.arange(s, s + t) for s, t in zip(starts, totals)])
    f = fused.double()
    q = plain.unit_rms(f[:, :n_q], eps) * q_gamma.double() * plain.temperature(positions, coef, every)[:, None]
    k = plain.unit_rms(f[:, n_q:n_q + n_k], eps) * k_gamma.double()
    bound = 1e-5 if dtype == "float32" else 1e-2
    got = q_out.view(tokens, heads, hd)[..., :dim].double().cpu()
    want = q.view(tokens, heads, dim)
    assert float(((got - want).abs() / want.abs().amax(dim=(1, 2), keepdim=True)).max()) < bound       # row by row: each has its own factor
    keys, values = case.read_back()
    assert rel_err(keys.view(tokens, kv_heads, hd)[..., :dim], k.view(tokens, kv_heads, dim)) < bound
    assert rel_err(values.view(tokens, kv_heads, hd)[..., :dim], f[:, n_q:n_q + n_k].view(tokens, kv_heads, dim)) < bound
    assert float(keys.view(tokens, kv_heads, hd)[..., dim:].float().abs().max()) == 0.0


@pytest.mark.parametrize("out_dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("heads,vdim,pitch", [(4, 40, 48), (3, 5, 16), (1, 200, 208), (2, 128, 128)])
def test_the_difference_of_two_maps(out_dtype, heads, vdim, pitch):
    """Row-major with columns behind the heads, and chunk-major; maps that nearly cancel keep their digits."""
    gen = torch.Generator().manual_seed(vdim)
    tokens, lam, post, eps = 21, 0.93, 0.6, 1e-5
    rows = torch.randn(tokens, heads, 2, pitch, generator=gen)
    rows[0, 0, 1] = rows[0, 0, 0] / lam * (1.0 + 1e-3 * torch.randn(pitch, generator=gen))
    a = rows.double()[..., :vdim]
    want = (plain.unit_rms(a[:, :, 0] - torch.tensor(lam, dtype=torch.float32).double() * a[:, :, 1], eps) * post).reshape(tokens, -1)
    bound = 2e-4 if out_dtype == "float32" else 1e-2
    columns = (heads * vdim + 7) // 8 * 8
    out = torch.full((tokens, columns + 8), float("nan"), dtype=DTYPES[out_dtype], device=DEV)
    flat = rows.reshape(tokens, -1).to(DEV)
    K.differential(flat, heads, vdim, pitch, lam, post, eps, out[:, :columns])
    assert rel_err(out[:, :heads * vdim], want) < bound
    assert columns == heads * vdim or float(out[:, heads * vdim:columns].float().abs().max()) == 0.0
    chunk = 32 if out_dtype == "bfloat16" else 16
    padded = (columns + chunk - 1) // chunk * chunk
    chunked = K.Chunked(torch.zeros(tokens, padded, dtype=DTYPES[out_dtype], device=DEV), tokens, columns)
    K.differential(flat, heads, vdim, pitch, lam, post, eps, chunked)
    assert torch.equal(chunked.to_rows()[:, :heads * vdim], out[:, :heads * vdim])


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("m", [1, 5, 12, 33, 64])
@pytest.mark.parametrize("n,sums,k", [(200, 72, 96), (64, 4, 40), (1100, 516, 256), (77, 60, 64)])
def test_a_product_with_32_bit_and_activated_columns(dtype, m, n, sums, k):
    gen = torch.Generator().manual_seed(m + n)
    a, w = torch.randn(m, k, generator=gen).to(DTYPES[dtype]), (torch.randn(n, k, generator=gen) / 8).to(DTYPES[dtype])
    want = a.double() @ w.double().T
    first = torch.full((m, sums + 3), float("nan"), device=DEV)[:, :sums]
    act = torch.full((m, (n - sums + 7) // 8 * 8), float("nan"), dtype=DTYPES[dtype], device=DEV)
    K.gemm(a.to(DEV), w.to(DEV), K.epilogue_f32_act(first, sums, act, "squared_relu"))
    assert rel_err(first, want[:, :sums]) < 1e-5
    assert rel_err(act[:, :n - sums], plain.squared_relu(want[:, sums:])) < (1e-5 if dtype == "float32" else 1e-2)
    chunk = 32 if dtype == "bfloat16" else 16
    padded = (n - sums + chunk - 1) // chunk * chunk
    chunked = K.Chunked(torch.zeros(m, padded, dtype=DTYPES[dtype], device=DEV), m, n - sums)
    again = torch.zeros(m, sums, device=DEV)
    packed = (K.pack_columns(w.to(DEV), 16), 16)
    K.gemm(a.to(DEV), w.to(DEV), K.epilogue_f32_act(again, sums, chunked, "squared_relu"), packed=packed)
    assert torch.equal(again, first) and torch.equal(chunked.to_rows()[:, :n - sums], act[:, :n - sums])


@pytest.mark.parametrize("m", [1, 4, 11])
def test_a_product_of_two_kinds_that_normalises_its_rows_itself(m):
    gen = torch.Generator().manual_seed(m)
    k, n, sums, eps = 72, 130, 68, 1e-4
    x, gamma = torch.randn(m, k, generator=gen), torch.randn(k, generator=gen)
    w = (torch.randn(n, k, generator=gen) / 8).to(torch.bfloat16)
    want = (plain.unit_rms(x.double(), eps) * gamma.double()).to(torch.bfloat16).double() @ w.double().T
    first, act = torch.zeros(m, sums, device=DEV), torch.zeros(m, 64, dtype=torch.bfloat16, device=DEV)
    rows = K.Normalized(x.to(DEV), gamma.to(DEV), None, eps, "rms_norm")
    assert K.takes_two_kinds(rows)
    K.gemm(rows, w.to(DEV), K.epilogue_f32_act(first, sums, act, "squared_relu"))
    assert rel_err(first, want[:, :sums]) < 5e-3
    assert rel_err(act[:, :n - sums], plain.squared_relu(want[:, sums:])) < 1.5e-2


@pytest.mark.parametrize("impl,m", [("plain", 70), ("tile", 70), ("tile", 300), ("skinny", 20)])
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_square_of_relu_in_every_product(dtype, impl, m):
    gen = torch.Generator().manual_seed(m)
    a, w = torch.randn(m, 128, generator=gen).to(DTYPES[dtype]), (torch.randn(96, 128, generator=gen) / 8).to(DTYPES[dtype])
    out = torch.zeros(m, 96, dtype=DTYPES[dtype], device=DEV)
    K.gemm(a.to(DEV), w.to(DEV), K.epilogue_act(out, "squared_relu"), impl=impl)
    assert rel_err(out, plain.squared_relu(a.double() @ w.double().T)) < (1e-5 if dtype == "float32" else 1e-2)
    with pytest.raises(K.KernelError):
        if impl == "skinny":
            K.gemm(a.to(DEV), w.to(DEV), K.epilogue_f32_act(torch.zeros(m, 98, device=DEV), 98, out, "squared_relu"))
        else:
            K.gemm(a.to(DEV), w.to(DEV), K.epilogue_f32_act(torch.zeros(m, 48, device=DEV), 48, out, "squared_relu"), impl=impl)


def test_columns_of_a_chunk_major_matrix():
    whole = K.Chunked(torch.arange(10 * 96, dtype=torch.float32, device=DEV).view(10, 96), 10, 96)
    assert torch.equal(whole.columns_from(32, 40).to_rows(), whole.to_rows()[:, 32:72])
    assert torch.equal(whole.columns_from(0, 16).to_rows(), whole.to_rows()[:, :16])
