"""Mekusun without a GPU: its configuration reader and the specification built from it, the tensor names a checkpoint must
hold and the sizes its tensors decide, the stream operations behind the layers, and the plain implementation's mechanisms
against the same sums written out another way."""

import copy
import math

import pytest
import torch

from tests.mekusun_configs import ALONE, MEKU_A, MEKU_B, MEKU_C, delta, latent, layer, mamba1, model
from tests.plain import mekusun_plain as plain


def build(cfg):
    from paged_llm_amd.config.registry import lookup_architecture
    from paged_llm_amd.models.decoder import DecoderModel
    arch = lookup_architecture(cfg)
    spec = arch.build_spec(arch.read_config(cfg))
    return spec, DecoderModel(spec, torch.float32, "cpu", max_positions=64)


def _random_weights(cfg, seed=0):
    from paged_llm_amd.weights.random_init import _declared_weights, draw_weights
    return dict(draw_weights(_declared_weights(cfg), seed, torch.float32, std=cfg["width"] ** -0.5, norm_jitter=True))


# --------------------------------------------------------------------------- configuration and specification
def test_architecture_is_registered():
    from paged_llm_amd.config.registry import lookup_architecture
    assert lookup_architecture(MEKU_A).name == "Mekusun"


def test_specification():
    spec, model_ = build(MEKU_A)
    assert [s.layer for s in spec.schedule] == list(range(6)) and [s.exit for s in spec.schedule] == list(range(6))
    assert [op.part.params["results"] for op in spec.stream_ops] == [2, 3, 4, 5, 6, 7]
    states = model_.state_specs()
    assert sorted(states) == [0, 2, 3, 4]
    assert states[0].shape == (16 * 72 + 72 * 3,)                       # 12 state elements are held as 16, three earlier inputs
    assert states[2].shape == (3 * 20 * 20,) and states[3].shape == (16 * 200 + 200,) and states[4].shape == (2 * 32 * 32,)
    groups = list(model_.cache_groups().values())
    assert sorted(g.owners for g in groups) == [[1], [5]] and all(g.spec.kind == "full" for g in groups)
    names = set(model_.weight_specs())
    assert {"embed", "head", "final.norm", "l0.norm1", "l0.norm1b", "l0.norm2", "l0.norm2b", "l0.ls1", "l0.ls2", "l0.dwa", "l0.mix.in", "l0.mix.conv",
            "l0.mix.conv.b", "l0.mix.x", "l0.mix.dt", "l0.mix.dt.b", "l0.mix.A_log", "l0.mix.D", "l0.mix.o", "l0.mlp.e0.up", "l0.mlp.e4.down",
            "l0.mlp.router", "l0.mlp.router.b", "l1.mix.q", "l1.mix.dkv", "l1.mix.dkv.norm", "l1.mix.uk", "l1.mix.uv", "l1.mix.o", "l1.mlp.up",
            "l1.mlp.down", "l1.mlp.act", "l2.mix.r", "l2.mix.k", "l2.mix.v", "l2.mix.a", "l2.mix.a.b", "l2.mix.g", "l2.mix.w0", "l2.mix.w1",
            "l2.mix.w2", "l2.mix.norm", "l2.mix.o", "l2.ls1", "l2.dwa"} <= names
    assert not {"l2.norm2", "l2.ls2", "l2.mlp.up", "l0.mlp.e0.gate", "l1.mlp.gate", "l0.mlp.correction", "l1.mix.dq", "l6.dwa"} & names
    shapes = {n: s.shape for n, s in model_.weight_specs().items()}
    assert shapes["l5.dwa"] == (7,) and shapes["l0.mix.x"] == (5 + 24, 72) and shapes["l1.mix.q"] == (3 * 32, 96) and shapes["l1.mlp.act"] == (2,)
    assert shapes["l4.mlp.router.b"] == (9,) and shapes["l4.mlp.e8.up"] == (24, 96)


def test_bad_configurations_are_refused():
    from paged_llm_amd.config.registry import lookup_architecture
    arch = lookup_architecture(MEKU_A)
    for change in (lambda c: c["layers"][0].update(type="mamba2"), lambda c: c["layers"][1]["mlp"].update(kind="gated"),
                   lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6), lambda c: c.update(layers=[]), lambda c: c.update(logit_softcap=-1.0)):
        bad = copy.deepcopy(MEKU_A)
        change(bad)
        with pytest.raises(ValueError):
            arch.read_config(bad)
    for i, change in ((0, {"conv": 17}), (0, {"state": 513}), (2, {"dim": 257}), (1, {"kv_rank": 1025})):
        bad = copy.deepcopy(MEKU_A)
        bad["layers"][i]["mixer"].update(change)
        with pytest.raises(ValueError):
            build(bad)


def test_the_checkpoint_decides_the_decay_products_inner_size():
    from paged_llm_amd.weights.loader import WeightsError, load_state_dict
    cfg = model(64, 40, [layer("general_delta", delta(heads=2, dim=8, decay_rank=5))])
    for rank in (1, 5, 23):
        cfg["layers"][0]["mixer"]["decay_rank"] = rank
        weights = _random_weights(cfg)
        assert weights["l0.mix.w1"].shape == (rank, 64) and weights["l0.mix.w2"].shape == (16, rank)
        other = copy.deepcopy(cfg)
        del other["layers"][0]["mixer"]["decay_rank"]
        spec, m = build(other)
        load_state_dict(m, weights)
        assert m.blocks[0].mixer.w_w2.shape == (16, rank) and m.blocks[0].mixer.w_in.shape == (5 * 16 + rank, 64)
        with pytest.raises(ValueError):                                  # the two matrices do not fit one another
            load_state_dict(build(other)[1], dict(weights, **{"l0.mix.w2": torch.zeros(16, rank + 1)}))
        with pytest.raises(WeightsError):                                # every other size is the configuration's
            load_state_dict(build(other)[1], dict(weights, **{"l0.mix.w1": torch.zeros(rank, 63)}))


def test_layers_without_a_feed_forward_ignore_its_vectors():
    from paged_llm_amd.weights.loader import WeightsError, load_state_dict
    cfg = ALONE["delta"]
    weights = _random_weights(cfg)
    load_state_dict(build(cfg)[1], dict(weights, **{"l0.ls2": torch.ones(64), "l0.norm2": torch.ones(64)}))
    with pytest.raises(WeightsError):
        load_state_dict(build(cfg)[1], dict(weights, **{"l0.ls3": torch.ones(64)}))


def test_factors_of_the_output_norms():
    """The factor of a norm behind a branch is (1 + w) times the layer scale, whichever arrives first."""
    from paged_llm_amd.parts.norm import RMSNorm
    from paged_llm_amd.parts.registry import BuildEnv
    env = BuildEnv(6, torch.float32, torch.device("cpu"), 8, shared={})
    w, s = torch.randn(6), torch.randn(6)
    for order in ((("", w), ("/ls1", s)), (("/ls1", s), ("", w))):
        norm = RMSNorm({"eps": 1e-5, "weight_name": "", "unit_offset": True, "scale_name": "/ls1"}, env)
        assert set(norm.weight_specs()) == {"", "/ls1"}
        for name, t in order:
            norm.assign(name, t)
        assert torch.allclose(norm.weight, (1 + w) * s)
    with pytest.raises(KeyError):
        norm.assign("ls1", s)


def test_a_sum_over_the_depth_belongs_behind_its_layer():
    from paged_llm_amd.models.decoder import DecoderModel
    from paged_llm_amd.parts.spec import ScheduleStep
    for change in (lambda s: setattr(s, "schedule", [ScheduleStep(1, exit=1), ScheduleStep(0, exit=0)] + s.schedule[2:]),
                   lambda s: setattr(s, "schedule", [ScheduleStep(0, exit=0), ScheduleStep(1, entry=1)] + s.schedule[2:])):
        spec, _ = build(MEKU_A)
        change(spec)
        with pytest.raises(ValueError):
            DecoderModel(spec, torch.float32, "cpu", max_positions=8)
    from paged_llm_amd.parts.spec import ModelSpec, PartSpec
    p = PartSpec("x")
    with pytest.raises(ValueError):                                      # a step that names an operation the model does not have
        ModelSpec(4, 4, p, [None], p, p, schedule=[ScheduleStep(0, exit=0)], embedding_name="e", final_norm_name="f", head_name="h")


def test_every_configuration_builds():
    for cfg in (*ALONE.values(), MEKU_B, MEKU_C):
        _, m = build(cfg)
        assert set(_random_weights(cfg)) == set(m.weight_specs())


def test_bench_configuration_builds():
    import bench
    spec, m = build(bench.mekusun_config(1024, 32000))
    assert len(spec.schedule) == 12 and m.graph_capturable() and m.graph_capturable(prompts=True)


# --------------------------------------------------------------------------- the plain mechanisms
def test_activations():
    z = torch.tensor([-3.0, -0.5, 0.0, 0.25, 4.0], dtype=torch.float64)
    p, q = torch.tensor(0.7, dtype=torch.float64), torch.tensor(-1.1, dtype=torch.float64)
    sp, sq = math.log(1 + math.exp(0.7)), math.log(1 + math.exp(-1.1))
    for x, y in zip(z.tolist(), plain.xielu(z, p, q).tolist()):
        want = sp * x * x + x / 2 if x > 0 else (0.5 + sq) * (math.exp(x) - 1 - x) + x / 2
        assert abs(y - want) < 1e-12
    for x, y in zip(z.tolist(), plain.gelu_erf(z).tolist()):
        assert abs(y - x * 0.5 * math.erfc(-x / math.sqrt(2))) < 1e-12
    assert float(plain.softplus(torch.tensor(-40.0, dtype=torch.float64))) == pytest.approx(math.exp(-40), rel=1e-12)
    assert plain.cap_logits(torch.tensor([100.0, -3.0]), 5.0).tolist() == pytest.approx([5.0 * math.tanh(20.0), 5.0 * math.tanh(-0.6)])


def test_rotation_pairs_the_halves():
    x = torch.randn(5, 2, 8, dtype=torch.float64)
    y = plain.rotate_halves(x, range(5), 8, 10.0)
    for p in range(5):
        for i in range(4):
            a = p * 10.0 ** (-2 * i / 8)
            u, v = x[p, :, i], x[p, :, i + 4]
            assert torch.allclose(y[p, :, i], u * math.cos(a) - v * math.sin(a)) and torch.allclose(y[p, :, i + 4], v * math.cos(a) + u * math.sin(a))


def test_selective_scan_against_the_sum_over_earlier_tokens():
    torch.manual_seed(0)
    T, C, N = 9, 4, 3
    d = lambda *s: torch.randn(*s, dtype=torch.float64)
    x, dt, A, B, Cm, D = d(T, C), torch.rand(T, C, dtype=torch.float64), -torch.rand(C, N, dtype=torch.float64), d(T, N), d(T, N), d(C)
    got = plain.selective_scan(x, dt, A, B, Cm, D)
    want = D * x
    for t in range(T):
        for s in range(t + 1):
            carry = torch.exp(A * dt[s + 1:t + 1].sum(0)[:, None])
            want[t] = want[t] + dt[s] * x[s] * (carry * B[s] * Cm[t]).sum(1)
    assert float((got - want).abs().max()) < 1e-12


def test_mamba1_reads_its_parts_in_order():
    """With W_in and W_o the identity on their parts the mixer is the scan of the activated convolution, gated."""
    torch.manual_seed(1)
    T, C, N, R = 7, 5, 2, 3
    d = lambda *s: torch.randn(*s, dtype=torch.float64)
    w = {"in": torch.eye(2 * C, dtype=torch.float64), "conv": d(C, 3), "conv.b": d(C), "x": d(R + 2 * N, C), "dt": d(C, R), "dt.b": d(C),
         "A_log": d(C, N), "D": d(C), "o": torch.eye(C, dtype=torch.float64)}
    h = d(T, 2 * C)
    got = plain.mamba1(h, w, mamba1(inner=C, state=N, dt_rank=R, conv=3))
    x = torch.zeros(T, C, dtype=torch.float64)
    for t in range(T):
        for j in range(3):
            if t - 2 + j >= 0:
                x[t] += h[t - 2 + j, :C] * w["conv"][:, j]
        x[t] += w["conv.b"]
    x = x / (1 + torch.exp(-x))
    low = x @ w["x"].T
    dt = torch.log1p(torch.exp(low[:, :R] @ w["dt"].T + w["dt.b"]))
    y = plain.selective_scan(x, dt, -torch.exp(w["A_log"]), low[:, R:R + N], low[:, R + N:], w["D"])
    z = h[:, C:]
    assert float((got - y * z / (1 + torch.exp(-z))).abs().max()) < 1e-12


def test_delta_memory_as_products_of_transitions():
    """A token moves the memory by one matrix, diag(w) - (a . u) u^T, and adds k v^T: the output as a sum over tokens of products of those matrices."""
    torch.manual_seed(2)
    T, H, n = 8, 2, 4
    d = lambda *s: torch.randn(*s, dtype=torch.float64)
    r, k, v, w, a = d(T, H, n), d(T, H, n), d(T, H, n), torch.rand(T, H, n, dtype=torch.float64), torch.rand(T, H, n, dtype=torch.float64)
    got = plain.delta_memory(r, k, v, w, a)
    for h in range(H):
        for t in range(T):
            o = torch.zeros(n, dtype=torch.float64)
            for s in range(t + 1):
                M = torch.eye(n, dtype=torch.float64)
                for j in range(s + 1, t + 1):
                    u = k[j, h] / math.sqrt(float(k[j, h] @ k[j, h]) + 1e-6)
                    M = (torch.diag(w[j, h]) - torch.outer(a[j, h] * u, u)) @ M
                o += v[s, h] * float(r[t, h] @ (M @ k[s, h]))
            assert float((got[t, h] - o).abs().max()) < 1e-10


def test_general_delta_norms_and_gates_every_head():
    torch.manual_seed(3)
    T, H, n, W = 5, 2, 3, 6
    d = lambda *s: torch.randn(*s, dtype=torch.float64)
    w = {x: d(H * n, W) for x in ("r", "k", "v", "a", "g")}
    w.update({"a.b": d(H * n), "w0": d(H * n), "w1": d(4, W), "w2": d(H * n, 4), "norm": d(H * n), "o": torch.eye(H * n, dtype=torch.float64)})
    h = d(T, W)
    got = plain.general_delta(h, w, delta(H, n), 1e-3)
    p = lambda x: (h @ w[x].T).view(T, H, n)
    dec = torch.exp(-math.exp(-0.5) / (1 + torch.exp(-(torch.tanh(h @ w["w1"].T) @ w["w2"].T + w["w0"])))).view(T, H, n)
    assert float(dec.min()) > math.exp(-math.exp(-0.5)) and float(dec.max()) < 1.0
    a = torch.sigmoid(h @ w["a"].T + w["a.b"]).view(T, H, n)
    o = plain.delta_memory(p("r"), p("k"), p("v"), dec, a)
    for t in range(T):
        for head in range(H):
            y = o[t, head] / math.sqrt(float((o[t, head] ** 2).mean()) + 1e-3)
            sl = slice(head * n, head * n + n)
            assert torch.allclose(got[t, sl], y * w["norm"][sl] / (1 + torch.exp(-(h[t] @ w["g"].T)[sl])))


def test_latent_attention_query_by_query():
    torch.manual_seed(4)
    m = latent(heads=2, dim=3, rot_dim=4, vdim=5, kv_rank=6, base=20.0, scale=0.4)
    T, W = 7, 8
    d = lambda *s: torch.randn(*s, dtype=torch.float64)
    w = {"q": d(14, W), "dkv": d(10, W), "dkv.norm": d(6), "uk": d(6, 6), "uv": d(10, 6), "o": torch.eye(10, dtype=torch.float64)}
    h = d(T, W)
    got = plain.latent_attention(h, w, m, 1e-4, range(T))
    turn = lambda x, p: plain.rotate_halves(x[None, None], [p], 4, 20.0)[0, 0]
    for i in range(T):
        q = (h[i] @ w["q"].T).view(2, 7)
        for head in range(2):
            scores, values = [], []
            for j in range(i + 1):
                dn = h[j] @ w["dkv"].T
                c = dn[:6] / math.sqrt(float((dn[:6] ** 2).mean()) + 1e-4) * w["dkv.norm"]
                k = (w["uk"] @ c)[head * 3:head * 3 + 3]
                scores.append((q[head, :3] @ k + turn(q[head, 3:], i) @ turn(dn[6:], j)) * 0.4)
                values.append((w["uv"] @ c)[head * 5:head * 5 + 5])
            p = torch.softmax(torch.stack(scores), 0)
            assert torch.allclose(got[i, head * 5:head * 5 + 5], sum(a * b for a, b in zip(p, values)))


def test_routed_experts_token_by_token():
    torch.manual_seed(5)
    W, F, E, top = 6, 4, 5, 3
    d = lambda *s: torch.randn(*s, dtype=torch.float64)
    w = {"router": d(E, W), "router.b": d(E) * 2}
    for e in range(E):
        w[f"e{e}.up"], w[f"e{e}.down"] = d(F, W), d(W, F)
    h = d(9, W)
    got = plain.routed(h, w, E, top)
    for t in range(9):
        z = {e: float(w["router"][e] @ h[t] + w["router.b"][e]) for e in range(E)}
        best = sorted(z, key=z.get, reverse=True)[:top]
        total = sum(math.exp(z[e]) for e in best)
        want = sum(math.exp(z[e]) / total * (w[f"e{e}.down"] @ plain.gelu_erf(w[f"e{e}.up"] @ h[t])) for e in best)
        assert torch.allclose(got[t], want)


def test_the_whole_model_is_the_sum_of_its_parts():
    """The stream behind every layer rebuilt from the mechanisms one by one: scales on what a sublayer adds, norms around zero
    on both sides of it, the sum over the depth over results taken in front of that sum."""
    cfg = MEKU_A
    w = {k: t.double() for k, t in _random_weights(cfg).items()}
    gen = torch.Generator().manual_seed(6)
    for i in range(6):
        w[f"l{i}.dwa"] = torch.randn(i + 2, generator=gen, dtype=torch.float64)
    toks = [7, 1, 250, 33, 33, 9, 120, 5, 64]
    outs = []
    logits = plain.forward(cfg, w, toks, torch.float64, outs)
    eps = cfg["norm"]["eps"]
    norm = lambda x, v: x / torch.sqrt((x ** 2).mean(-1, keepdim=True) + eps) * (1 + v)
    X = [w["embed"][toks] * cfg["embedding"]["scale"]]
    x = X[0]
    for i, l in enumerate(cfg["layers"]):
        wm, wf = plain.under(w, f"l{i}.mix."), plain.under(w, f"l{i}.mlp.")
        x = x + norm(plain.mixer(l, norm(x, w[f"l{i}.norm1"]), wm, eps, range(9)), w[f"l{i}.norm1b"]) * w[f"l{i}.ls1"]
        if l["mlp"]:
            x = x + norm(plain.feed_forward(l["mlp"], norm(x, w[f"l{i}.norm2"]), wf), w[f"l{i}.norm2b"]) * w[f"l{i}.ls2"]
        X.append(x)
        x = (w[f"l{i}.dwa"][:, None, None] * torch.stack(X)).sum(0)
        assert float((outs[i] - x).abs().max()) < 1e-9
    cap = cfg["logit_softcap"]
    assert float((logits - cap * torch.tanh(norm(x, w["final.norm"]) @ w["head"].T / cap)).abs().max()) < 1e-9
    assert float((plain.forward(cfg, w, toks[:4], torch.float64) - logits[:4]).abs().max()) < 1e-9       # a later token changes nothing before it
