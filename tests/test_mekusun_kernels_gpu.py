"""Kernels that the Mekusun layers brought, each against the plain version of the same operation in float64: the selective
scan and the delta memory token by token and in chunks (several sequences, carried states, slots in any order, sizes that fit
no tile, outputs and the states left behind), the sum over the depth in the kernel that adds and norms, the routing by a
softmax over the chosen, experts without a gate, activations of single elements, capped logits."""

import math

import pytest
import torch

from tests.plain import mekusun_plain as plain

pytestmark = pytest.mark.gpu


def dev(t):
    return t.cuda()


def sequences(lengths, starts, slots):
    cu = torch.tensor([0] + list(torch.tensor(lengths).cumsum(0)), dtype=torch.int32).cuda()
    return (torch.tensor(slots, dtype=torch.int32).cuda(), torch.tensor(starts, dtype=torch.int32).cuda(), cu, len(lengths))


def close(got, want, tol, what=""):
    got, want = got.detach().double().cpu(), want.double()
    scale = float(want.abs().max())
    err = float((got - want).abs().max()) / max(scale, 1e-30)
    assert math.isfinite(err) and err <= tol, (what, err)


# --------------------------------------------------------------------------- the selective scan
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("channels,N,lengths,max_q", [
    (64, 16, [1, 1, 1], 1), (70, 5, [7, 1, 0, 33], 33), (192, 16, [300, 2], 300), (33, 40, [129, 150], 150), (130, 8, [40, 200, 1], 200),
    (64, 200, [3, 140], 140), (257, 32, [128], 128)])
def test_selective_scan(channels, N, lengths, max_q, dtype):
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(channels + N)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    T, S, held = sum(lengths), len(lengths), ops.scan_state_size(N)
    x, z = rnd(T, channels).to(dtype), rnd(T, channels).to(dtype)
    raw, bias = rnd(T, channels), rnd(channels) - 2.0
    B, C, D = rnd(T, N).to(dtype), rnd(T, N).to(dtype), rnd(channels)
    A = -torch.exp(rnd(channels, N) * 0.7)
    pad = lambda t: torch.cat([t, t.new_zeros(t.shape[0], held - N)], dim=1)
    a2 = torch.zeros(held, channels)
    a2[:N] = (A.double() * math.log2(math.e)).T.float()
    slots, starts = list(range(S))[::-1], [0 if i % 2 == 0 else 5 for i in range(S)]
    state = torch.zeros(S + 1, held * channels + 11)
    state[:, :] = 7.0                                          # whatever a slot held before a sequence starts
    first = rnd(S, N, channels)
    for i in range(S):
        if starts[i]:
            state[slots[i], :held * channels] = torch.cat([first[i], torch.zeros(held - N, channels)]).flatten()
    st = dev(state)
    out = ops.selective_scan(dev(x), dev(raw), dev(bias), dev(torch.cat([pad(B), pad(C)], dim=1)), dev(a2), dev(D), dev(z), st,
                             *sequences(lengths, starts, slots), max_q_len=max_q)
    at = 0
    for i, n in enumerate(lengths):
        if n == 0:
            continue
        sl = slice(at, at + n)
        at += n
        dt = plain.softplus(raw[sl].double() + bias.double())
        Sx = first[i].double().T.clone() if starts[i] else torch.zeros(channels, N, dtype=torch.float64)
        ys = []
        for t in range(n):
            Sx = torch.exp(dt[t][:, None] * A.double()) * Sx + (dt[t] * x[sl][t].double())[:, None] * B[sl][t].double()
            ys.append(Sx @ C[sl][t].double() + D.double() * x[sl][t].double())
        want = torch.stack(ys) * plain.silu(z[sl].double())
        close(out[sl], want, 3e-6 if dtype == torch.float32 else 6e-3, f"outputs of sequence {i}")
        close(st[slots[i], :held * channels].view(held, channels)[:N], Sx.T, 3e-6, f"state of sequence {i}")
        assert float(st[slots[i], N * channels:held * channels].abs().max() if held > N else 0) == 0.0
        assert torch.equal(st[slots[i], held * channels:].cpu(), state[slots[i], held * channels:])
    assert torch.equal(st[S].cpu(), state[S]), "a slot that no sequence of the step has is left alone"


def test_the_scans_step_sizes_keep_small_values():
    """Step sizes of 1e-6 and less (softplus far below zero) keep their relative precision."""
    from paged_llm_amd.csrc import ops
    raw = torch.linspace(-20.0, 25.0, 64)[None, :].contiguous()
    one, zero = torch.ones(1, 64), torch.zeros(64)
    st = torch.zeros(1, 8 * 64).cuda()
    bc = torch.ones(1, 16)
    ops.selective_scan(dev(one), dev(raw), dev(zero), dev(bc), dev(torch.zeros(8, 64)), dev(zero), dev(one), st, *sequences([1], [0], [0]), max_q_len=1)
    want = plain.softplus(raw[0].double())
    assert float(((st[0, :64].double().cpu() - want) / want).abs().max()) < 1e-6


# --------------------------------------------------------------------------- the delta memory
def delta_case(H, d, T, dtype, seed, spread=1.0):
    gen = torch.Generator().manual_seed(seed)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    C = H * d
    cols = {n: i * C for i, n in enumerate(("r", "k", "v", "a", "g"))}
    rows = torch.cat([rnd(T, C), rnd(T, C) * spread, rnd(T, C), rnd(T, C) * 2, rnd(T, C), rnd(T, 3)], dim=1).to(dtype)
    return rows, cols, rnd(T, C) * 2.0, rnd(C), rnd(C), 1.0 + 0.3 * rnd(C)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,d,lengths,max_q", [
    (2, 16, [1, 1, 1], 1), (3, 20, [9, 1, 0, 30], 30), (2, 64, [100, 3], 100), (1, 70, [33, 64, 1], 64), (4, 8, [257], 257), (2, 128, [5, 96], 96),
    (1, 256, [3, 50], 50), (2, 33, [48, 49], 49), (1, 1, [60], 60), (3, 96, [31, 32, 65], 65)])
def test_delta_memory(H, d, lengths, max_q, dtype):
    from paged_llm_amd.csrc import ops
    T, S, C = sum(lengths), len(lengths), H * d
    rows, cols, raw_w, w0, bias_a, weight = delta_case(H, d, T, dtype, seed=H * 100 + d)
    gen = torch.Generator().manual_seed(9)
    slots, starts = list(range(S))[::-1], [0 if i % 2 == 0 else 5 for i in range(S)]
    first = torch.randn(S, H, d, d, generator=gen)
    state = torch.full((S + 1, C * d + 5), 7.0)
    for i in range(S):
        if starts[i]:
            state[slots[i], :C * d] = first[i].flatten()
    st = dev(state)
    eps = 1e-5
    out = ops.delta_rule(dev(rows), cols, dev(raw_w), dev(w0), dev(bias_a), dev(weight), eps, H, d, st, *sequences(lengths, starts, slots), max_q_len=max_q)
    at = 0
    for i, n in enumerate(lengths):
        if n == 0:
            continue
        sl = slice(at, at + n)
        at += n
        part = lambda name: rows[sl, cols[name]:cols[name] + C].double().view(n, H, d)
        w = torch.exp(-math.exp(-0.5) * torch.sigmoid(raw_w[sl].double() + w0.double())).view(n, H, d)
        a = torch.sigmoid(part("a") + bias_a.double().view(H, d))
        r, k, v = part("r"), part("k"), part("v")
        u = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
        Sx = first[i].double().clone() if starts[i] else torch.zeros(H, d, d, dtype=torch.float64)
        os = []
        for t in range(n):
            read = torch.einsum("hn,hnp->hp", u[t], Sx)
            Sx = w[t][..., None] * Sx - (a[t] * u[t])[..., None] * read[:, None, :] + k[t][..., None] * v[t][:, None, :]
            os.append(torch.einsum("hnp,hn->hp", Sx, r[t]))
        o = plain.unit_rms(torch.stack(os), eps).reshape(n, C) * weight.double() * torch.sigmoid(part("g").reshape(n, C))
        close(out[sl], o, 2e-5 if dtype == torch.float32 else 1e-2, f"outputs of sequence {i}")
        close(st[slots[i], :C * d].view(H, d, d), Sx, 5e-6, f"memory of sequence {i}")
        assert torch.equal(st[slots[i], C * d:].cpu(), state[slots[i], C * d:])
    assert torch.equal(st[S].cpu(), state[S])


@pytest.mark.parametrize("case", ["slow decays", "fast decays", "one direction"])
def test_delta_memory_chunks_at_the_ends_of_their_range(case):
    """Chunks against tokens where the products of decays are largest and smallest, and where every key points the same way
    (the system of a chunk is then as far from the identity as it gets)."""
    from paged_llm_amd.csrc import ops
    H, d, T = 2, 64, 200
    C = H * d
    rows, cols, raw_w, w0, bias_a, weight = delta_case(H, d, T, torch.float32, seed=3)
    if case == "slow decays":
        raw_w = raw_w * 0.1 - 12.0
    elif case == "fast decays":
        raw_w = raw_w * 0.1 + 12.0
    else:
        rows[:, cols["k"]:cols["k"] + C] = rows[:1, cols["k"]:cols["k"] + C]
        bias_a = bias_a * 0 + 3.0
        raw_w = raw_w - 6.0
    got, states = [], []
    for max_q in (T, 1):                                        # (a bound of 1 keeps the tokens one by one)
        st = torch.zeros(1, C * d).cuda()
        got.append(ops.delta_rule(dev(rows), cols, dev(raw_w), dev(w0), dev(bias_a), dev(weight), 1e-5, H, d, st, *sequences([T], [0], [0]), max_q_len=max_q))
        states.append(st)
    close(got[0], got[1].cpu(), 5e-5, case)
    close(states[0], states[1].cpu(), 2e-5, case)


# --------------------------------------------------------------------------- the sum over the depth
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("rows,H,count", [(1, 64, 1), (7, 50, 3), (33, 1024, 6), (3, 4096, 2), (2, 4100, 2), (5, 1030, 11)])
def test_depth_sum_in_the_norm_kernel(rows, H, count, dtype):
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(H + count)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    stream, branch, history, weights = rnd(rows, H), rnd(rows, H), rnd(count + 2, rows, H), rnd(count + 1)
    w_branch, w_next, bias = rnd(H), rnd(H), rnd(H)
    eps = 1e-3
    for b in (None, bias):
        s, h = dev(stream), dev(history)
        got = ops.rms_sandwich(s, dev(branch), dev(w_branch), 0.7, eps, w_next=dev(w_next), out_dtype=dtype, bias=None if b is None else dev(b),
                               depth=ops.DepthSum(h, dev(weights)))
        y = branch.double() + (0 if b is None else b.double())
        r = stream.double() + 0.7 * plain.unit_rms(y, eps) * w_branch.double()
        x = sum(weights[j].double() * history[j].double() for j in range(count)) + weights[count].double() * r
        close(h[count], r, 1e-6)
        close(s, x, 1e-6)
        close(got, plain.unit_rms(x, eps) * w_next.double(), 2e-6 if dtype == torch.float32 else 6e-3)
        assert torch.equal(h[:count].cpu(), history[:count]) and torch.equal(h[count + 1].cpu(), history[count + 1])
    # without rows behind it, and the operation on its own
    s, h = dev(stream), dev(history)
    assert ops.rms_sandwich(s, dev(branch), dev(w_branch), 0.7, eps, depth=ops.DepthSum(h, dev(weights))) is None
    r = stream.double() + 0.7 * plain.unit_rms(branch.double(), eps) * w_branch.double()
    close(s, sum(weights[j].double() * history[j].double() for j in range(count)) + weights[count].double() * r, 1e-6)
    s, h = dev(stream), dev(history)
    ops.depth_sum(s, ops.DepthSum(h, dev(weights)))
    close(s, sum(weights[j].double() * history[j].double() for j in range(count)) + weights[count].double() * stream.double(), 1e-6)
    assert torch.equal(h[count].cpu(), stream)


@pytest.mark.parametrize("H", [64, 50])
def test_depth_sum_behind_experts(H):
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(H)
    rnd = lambda *s: torch.randn(*s, generator=gen)
    rows, top, count = 9, 3, 2
    expert_out, h = rnd(rows * top, H), rnd(rows, H)
    perm = torch.randperm(rows * top, generator=gen).to(torch.int32)
    weights = torch.rand(rows, top, generator=gen)
    stream, history, dw, wb, wn = rnd(rows, H), rnd(count + 1, rows, H), rnd(count + 1), rnd(H), rnd(H)
    s, hist = dev(stream), dev(history)
    got = ops.rms_sandwich(s, ops.ChoiceSum(dev(expert_out), dev(h), dev(perm), dev(weights)), dev(wb), 1.0, 1e-5, w_next=dev(wn),
                           out_dtype=torch.float32, depth=ops.DepthSum(hist, dev(dw)))
    y = (expert_out.double()[perm.long()].view(rows, top, H) * weights.double()[..., None]).sum(1)
    r = stream.double() + plain.unit_rms(y, 1e-5) * wb.double()
    x = plain.depth_average([history[j].double() for j in range(count)] + [r], dw.double())
    close(hist[count], r, 1e-6)
    close(s, x, 1e-6)
    close(got, plain.unit_rms(x, 1e-5) * wn.double(), 2e-6)


# --------------------------------------------------------------------------- routing and experts
@pytest.mark.parametrize("tokens,n,top,width", [(1, 12, 2, 64), (5, 7, 7, 40), (140, 64, 4, 96), (600, 3, 1, 130)])
def test_routing_by_a_softmax_over_the_chosen(tokens, n, top, width):
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(n)
    h, router, bias = torch.randn(tokens, width, generator=gen), torch.randn(n, width, generator=gen), torch.randn(n, generator=gen) * 4
    ids, weights = ops.moe_route(dev(h), dev(router), dev(bias), 1, 1, top, "softmax_chosen")
    z = h.double() @ router.double().T + bias.double()
    best, want = torch.topk(z, top, dim=-1)
    assert torch.equal(ids.cpu().long(), want)
    close(weights, torch.softmax(best, dim=-1), 1e-5)


@pytest.mark.parametrize("dtype,rows", [("float32", 16), ("bfloat16", 16), ("bfloat16", 64), ("bfloat16", 128)])
@pytest.mark.parametrize("activation", ["gelu", "silu", "tanh"])
@pytest.mark.parametrize("width,ff", [(64, 48), (256, 136), (320, 200)])
def test_experts_without_a_gate(width, ff, activation, dtype, rows):
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
    act = ops.moe_expert_gemm(dev(h), dev(up), tiles, sorted_pair, top, False, activation, tile_rows=rows, plain=True)
    out = ops.moe_expert_gemm(act, dev(down), tiles, sorted_pair, top, False, tile_rows=rows)
    got = ops.moe_combine(out, dev(h), row_of_pair, dev(weights))
    f = {"gelu": plain.gelu_erf, "silu": plain.silu, "tanh": torch.tanh}[activation]
    want = torch.zeros(tokens, width, dtype=torch.float64)
    for t in range(tokens):
        for k in range(top):
            e = int(ids[t, k])
            want[t] += weights[t, k].double() * (down[e].double() @ f(up[e].double() @ h[t].double()))
    close(got, want, 2e-6 if dtype == "float32" else 1e-2)


# --------------------------------------------------------------------------- single elements
@pytest.mark.parametrize("name", ["gelu", "gelu_tanh", "silu", "xielu", "tanh", None])
@pytest.mark.parametrize("cols,stride", [(64, 64), (37, 50), (2056, 2064)])
def test_activations_of_single_elements(name, cols, stride):
    from paged_llm_amd.csrc import ops
    gen = torch.Generator().manual_seed(cols)
    x = torch.randn(11, stride, generator=gen) * 3
    x[0, :8] = torch.tensor([0.0, 1e-4, -1e-4, 1e-8, -1e-8, 30.0, -30.0, -90.0])
    p, q = 0.3, -1.2
    params = (float(plain.softplus(torch.tensor(p, dtype=torch.float64))), 0.5 + float(plain.softplus(torch.tensor(q, dtype=torch.float64))))
    f = {"gelu": plain.gelu_erf, "silu": plain.silu, "tanh": torch.tanh, None: lambda z: z,
         "gelu_tanh": lambda z: 0.5 * z * (1 + torch.tanh(math.sqrt(2 / math.pi) * (z + 0.044715 * z ** 3))),
         "xielu": lambda z: plain.xielu(z, torch.tensor(p, dtype=torch.float64), torch.tensor(q, dtype=torch.float64))}[name]
    for src in (torch.float32, torch.bfloat16):
        for out in (torch.float32, torch.bfloat16):
            rows = dev(x.to(src))[:, :cols]
            got = ops.activate_rows(rows, name, params, out_dtype=out)
            want = f(x.to(src)[:, :cols].double())
            # (a GELU far below zero is the difference of nearly equal numbers: absolute errors of z's own rounding there)
            err = ((got.double().cpu() - want).abs() / (want.abs() + 0.01 * x.to(src)[:, :cols].double().abs() + 1e-6)).max()
            assert float(err) < (2e-5 if out == torch.float32 else 5e-3), (name, src, out, float(err))


@pytest.mark.parametrize("rows", [1, 5, 8, 16, 24, 40, 64, 128, 200])
@pytest.mark.parametrize("name", ["xielu", "gelu"])
def test_activation_in_the_products_kernel(rows, name):
    """The product's own kernels for few and some rows, and the kernel behind the product, against the product in float64."""
    from paged_llm_amd.parts.linear import Weight, activated_linear
    gen = torch.Generator().manual_seed(rows)
    for N, K in ((512, 256), (200, 1024)):
        x, w = torch.randn(rows, K, generator=gen).bfloat16(), (torch.randn(N, K, generator=gen) * K ** -0.5).bfloat16()
        got = activated_linear(dev(x), Weight(dev(w)), name, (0.8, 0.9))
        z = x.double() @ w.double().T
        want = plain.gelu_erf(z) if name == "gelu" else torch.where(z > 0, 0.8 * z * z, 0.9 * (torch.expm1(z.clamp(max=0)) - z.clamp(max=0))) + 0.5 * z
        assert got.dtype == torch.bfloat16
        close(got, want, 1e-2)


def test_capped_logits():
    from paged_llm_amd.csrc import ops
    x = torch.linspace(-200, 200, 1003)[None, :].contiguous()
    got = ops.cap_rows(dev(x), 15.0)
    close(got, plain.cap_logits(x.double(), 15.0), 1e-6)
