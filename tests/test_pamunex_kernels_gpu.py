"""Kernels that the Pamunex layers brought, each against the plain version of the same operation in float64: queries and keys
normed with a weight in front of the rotation (both kernels that prepare them, and their order of norm and rotation as other
models have it), the layer norm that forms the experts' sum itself, the choice by the two largest scores of a group, the
square of relu in every place an activation stands, one matrix per head in the order the batched product reads."""

import math

import pytest
import torch

from tests.plain import pamunex_plain as plain

pytestmark = pytest.mark.gpu


def dev(t):
    return t.cuda()


def close(got, want, tol, what=""):
    got, want = got.detach().double().cpu(), want.double()
    scale = float(want.abs().max())
    err = float((got - want).abs().max()) / max(scale, 1e-30)
    assert math.isfinite(err) and err <= tol, (what, err)


# --------------------------------------------------------------------------- queries and keys in front of the pages
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("norm_first,weighted,interleaved", [(True, True, False), (True, False, False), (False, True, False), (False, False, False), (True, True, True)])
@pytest.mark.parametrize("H,G,d,dv,rot", [(4, 2, 24, 40, 16), (3, 1, 64, 64, 64), (5, 5, 96, 16, 24), (2, 1, 128, 128, 8), (2, 2, 160, 32, 160), (6, 2, 10, 6, 6), (1, 1, 4, 72, 0),
                                          (7, 1, 20, 33, 12), (8, 1, 256, 256, 128)])
def test_queries_keys_and_values_in_front_of_the_pages(H, G, d, dv, rot, norm_first, weighted, interleaved, dtype):
    """Head sizes, rotated widths and pairings that the kernel of four elements a lane takes and ones that it does not; a
    projection with further columns behind; a token without a place in the pages."""
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(H * d + rot)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    T, block, eps, base = 9, 16, 1e-2, 50.0
    D = -(-max(d, dv) // 16) * 16
    channels = (H + G) * d + G * dv
    proj, bias = rnd(T, channels + 4), rnd(channels)
    wq, wk = rnd(d), rnd(d)
    positions = torch.tensor([0, 1, 2, 40, 41, 7, 100, 3, 63], dtype=torch.int32)
    slots = torch.tensor([5, 17, 31, 32, -1, 0, 79, 48, 15], dtype=torch.int32)
    cos = sin = None
    if rot:
        ang = torch.arange(128, dtype=torch.float64)[:, None] * base ** (-torch.arange(0, rot, 2, dtype=torch.float64) / rot)[None]
        cos, sin = dev(torch.cos(ang).float()), dev(torch.sin(ang).float())
    k_pages, v_pages = dev(torch.full((5, G, block, D), 7.0).to(dtype)), dev(torch.full((5, G, D, block), 7.0).to(dtype))
    q = ops.attn_prepare(dev(proj), dev(bias), None, None, None, None, None, T, dev(positions), cos, sin, rot, interleaved, eps, H, G, d, dv, D, dtype,
                         dev(slots), k_pages, v_pages, norm_weights=(dev(wq), dev(wk)) if weighted else None, norm_first=norm_first)
    x = proj[:, :channels].double() + bias.double()
    want_q, want_k, want_v = x[:, :H * d].view(T, H, d), x[:, H * d:(H + G) * d].view(T, G, d), x[:, (H + G) * d:].view(T, G, dv)

    def turn(t):
        if not rot:
            return t
        if not interleaved:
            return plain.rotate_halves(t, positions.tolist(), rot, base)
        order = list(range(0, rot, 2)) + list(range(1, rot, 2)) + list(range(rot, t.shape[-1]))
        out = torch.empty_like(t)
        out[..., order] = plain.rotate_halves(t[..., order], positions.tolist(), rot, base)
        return out

    def ready(t, w):
        scale = lambda y: plain.unit_rms(y, eps) * (w.double() if weighted else 1.0)
        return turn(scale(t)) if norm_first else scale(turn(t))
    tol = 2e-6 if dtype == torch.float32 else 5e-3
    q = q.view(T, H, D)
    close(q[..., :d], ready(want_q, wq), tol, "q")
    assert not q[..., d:].any()
    want_k = ready(want_k, wk)
    touched = set()
    for t, slot in enumerate(slots.tolist()):
        if slot < 0:
            continue
        page, off = divmod(slot, block)
        touched.add((page, off))
        close(k_pages[page, :, off, :d], want_k[t], tol, ("k", t))
        close(v_pages[page, :, :dv, off], want_v[t], tol, ("v", t))
        assert not k_pages[page, :, off, d:].any() and not v_pages[page, :, dv:, off].any()
    for page in range(5):
        for off in range(block):
            if (page, off) not in touched:
                assert bool((k_pages[page, :, off] == 7).all()) and bool((v_pages[page, :, :, off] == 7).all())


# --------------------------------------------------------------------------- the norm behind experts
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,top", [(40, 3), (96, 1), (1024, 4), (2048, 6), (4096, 2), (4100, 3), (50, 2), (64, 65)])
def test_the_layer_norm_forms_the_experts_sum_itself(width, top, dtype):
    """Given the experts' rows, places and weights the kernel gives what it gives after their sum (rows of up to 4,096
    elements; longer ones, rows that no 16-byte load fits and sums of very many take the sum first), and what float64 gives."""
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(width + top)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    tokens = 7
    stream, expert_out, h = rnd(tokens, width), rnd(tokens * top, width), rnd(tokens, width).to(dtype)
    places = torch.randperm(tokens * top, generator=gen).to(torch.int32)
    places[torch.tensor([1, 5])] = -1                                        # (choices that hand the token's own row back)
    weights = torch.rand((tokens, top), generator=gen)
    w, b = rnd(width), rnd(width)
    branch = lambda: ops.ChoiceSum(dev(expert_out), dev(h), dev(places), dev(weights))
    out_dtype = torch.bfloat16 if dtype == torch.bfloat16 else None
    s1, s2 = dev(stream), dev(stream)
    rows1 = ops.layernorm(branch(), dev(w), dev(b), 1e-3, s1, None, out_dtype)
    rows2 = ops.layernorm(branch().rows(), dev(w), dev(b), 1e-3, s2, None, out_dtype)
    picked = torch.where(places.view(tokens, top, 1) >= 0, expert_out.double()[places.clamp(min=0).long()].view(tokens, top, width),
                         h.double()[:, None, :].expand(tokens, top, width))
    want = stream.double() + plain.layer_norm((weights.double()[:, :, None] * picked).sum(dim=1), w.double(), b.double(), 1e-3)
    for s in (s1, s2):
        close(s, want, 3e-6)
    if out_dtype is None:
        assert rows1 is None and rows2 is None
    else:
        assert torch.equal(rows1, s1.bfloat16()) and torch.equal(rows2, s2.bfloat16())
    assert ops.layernorm_sum_takes(width, top) == (width % 4 == 0 and width <= 4096 and top <= 64)


# --------------------------------------------------------------------------- routing and experts
@pytest.mark.parametrize("n,groups,keep,top", [(12, 4, 2, 3), (16, 4, 1, 4), (18, 3, 2, 5), (7, 7, 3, 3), (8, 1, 1, 8), (6, 2, 2, 1), (64, 8, 3, 6), (2, 1, 1, 2), (1, 1, 1, 1)])
def test_the_choice_by_the_two_largest_scores_of_a_group(n, groups, keep, top):
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(n)
    h = torch.randn((515 if n % 2 else 203, 40), generator=gen)                # (steps of up to 512 tokens and of more: one and eight tokens to a workgroup)
    w = torch.randn((n, 40), generator=gen) * 0.4
    scores = torch.sigmoid(h.double() @ w.double().T)
    want = plain.choose(scores, top, groups, keep).sort(dim=1).values
    ids, weights = ops.moe_route(dev(h), dev(w), None, groups, keep, top, "sigmoid", group_mark="two_largest")
    order = ids.cpu().long().sort(dim=1)
    assert torch.equal(order.values, want)
    close(torch.gather(weights.cpu(), 1, order.indices), torch.gather(scores, 1, want), 1e-6)
    few = ops.moe_route(dev(h[50:61]), dev(w), None, groups, keep, top, "sigmoid", group_mark="two_largest")       # the same rows in a small step
    assert torch.equal(few[0], ids[50:61]) and torch.equal(few[1], weights[50:61])
    if 1 < keep < groups and n // groups > 2:
        other = ops.moe_route(dev(h), dev(w), None, groups, keep, top, "sigmoid")[0].cpu().long().sort(dim=1).values
        assert not torch.equal(other, want), "the mark by the largest score alone chooses otherwise somewhere"


@pytest.mark.parametrize("width,ff,dtype,rows", [(*size, *form) for size in ((64, 48), (256, 136)) for form in (("float32", 16), ("bfloat16", 16), ("bfloat16", 64),
                                                 ("bfloat16", 128))] + [(50, 31, "float32", 16), (50, 31, "bfloat16", 16)])
def test_experts_with_the_square_of_relu(width, ff, dtype, rows):
    from paged_llm_amd.csrc import ops
    dt = getattr(torch, dtype)
    gen = torch.Generator().manual_seed(width + ff)
    tokens, E, top = (40 if rows == 16 else 300), 5, 2
    h = torch.randn(tokens, width, generator=gen).to(dt)
    up = (torch.randn(E, ff, width, generator=gen) * width ** -0.5).to(dt)
    down = (torch.randn(E, width, ff, generator=gen) * ff ** -0.5).to(dt)
    ids = torch.stack([torch.randperm(E, generator=gen)[:top] for _ in range(tokens)]).to(torch.int32)
    weights = torch.rand(tokens, top, generator=gen)
    sorted_pair, row_of_pair, tiles = ops.moe_align(dev(ids), E, rows)
    act = ops.moe_expert_gemm(dev(h), dev(up), tiles, sorted_pair, top, False, "relu2", tile_rows=rows, plain=True)
    out = ops.moe_expert_gemm(act, dev(down), tiles, sorted_pair, top, False, tile_rows=rows)
    got = ops.moe_combine(out, dev(h), row_of_pair, dev(weights))
    want = torch.zeros(tokens, width, dtype=torch.float64)
    for t in range(tokens):
        for k in range(top):
            e = int(ids[t, k])
            want[t] += weights[t, k].double() * (down[e].double() @ plain.relu_squared(up[e].double() @ h[t].double()))
    close(got, want, 2e-6 if dtype == "float32" else 1e-2)


# --------------------------------------------------------------------------- single elements, products
@pytest.mark.parametrize("cols,stride", [(64, 64), (37, 50), (2056, 2064)])
def test_the_square_of_relu(cols, stride):
    from paged_llm_amd.csrc import ops
    x = torch.randn(11, stride, generator=torch.Generator().manual_seed(cols)) * 3
    x[0, :6] = torch.tensor([0.0, -0.0, 1e-4, -1e-4, 1e3, -1e3])
    for src in (torch.float32, torch.bfloat16):
        for out in (torch.float32, torch.bfloat16):
            got = ops.activate_rows(dev(x.to(src))[:, :cols], "relu2", out_dtype=out)
            want = plain.relu_squared(x.to(src)[:, :cols].double())
            assert float(((got.double().cpu() - want).abs() / (want + 1e-12)).max()) < (1e-6 if out == torch.float32 else 4e-3)
            assert bool((got.cpu()[x.to(src)[:, :cols] <= 0] == 0).all())


@pytest.mark.parametrize("rows", [1, 5, 8, 16, 24, 40, 64, 128, 200])
def test_the_square_of_relu_in_the_products_kernel(rows):
    """The product's own kernels for few and some rows, and the kernel behind the product, against the product in float64."""
    from paged_llm_amd.parts.linear import Weight, activated_linear
    gen = torch.Generator().manual_seed(rows)
    for N, K in ((512, 256), (200, 1024), (1024, 2048), (31, 50)):
        x, w = torch.randn(rows, K, generator=gen).bfloat16(), (torch.randn(N, K, generator=gen) * K ** -0.5).bfloat16()
        got = activated_linear(dev(x), Weight(dev(w)), "relu2")
        assert got.dtype == torch.bfloat16
        close(got, plain.relu_squared(x.double() @ w.double().T), 1e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,heads,N,K", [(1, 4, 32, 16), (7, 3, 36, 20), (130, 16, 192, 128)])
def test_one_matrix_per_head(T, heads, N, K, dtype):
    """Rows that are views into wider ones, given and taken; the matrices as a checkpoint stores them and as a transposed view."""
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(T)
    a = torch.randn(T, heads, K + 8, generator=gen).to(dtype)
    w = (torch.randn(heads, N, K, generator=gen) * K ** -0.5).to(dtype)
    want = torch.stack([a[:, h, :K].double() @ w[h].double().T for h in range(heads)], dim=1)
    for m in (w, w.transpose(1, 2).contiguous().transpose(1, 2)):
        close(ops.gemm_heads(dev(a)[:, :, :K], ops.HeadMatrices(dev(m))), want, 2e-6 if dtype == torch.float32 else 6e-3)
        out = dev(torch.full((T, heads, N + 4), 3.0).to(dtype))
        ops.gemm_heads(dev(a)[:, :, :K], ops.HeadMatrices(dev(m)), out=out[:, :, :N])
        close(out[:, :, :N], want, 2e-6 if dtype == torch.float32 else 6e-3)
        assert bool((out[:, :, N:] == 3).all())
