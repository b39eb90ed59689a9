"""Pamunex without a GPU: its configuration reader and the specification built from it, the tensor names a checkpoint must
hold, and the plain implementation's mechanisms against the same sums written out another way."""

import copy
import math

import pytest
import torch

from tests.pamunex_configs import ALONE, PAMU_A, PAMU_B, PAMU_C, blocks, latent, layer, model
from tests.plain import pamunex_plain as plain


def build(cfg):
    from paged_llm_amd.config.registry import lookup_architecture
    from paged_llm_amd.models.decoder import DecoderModel
    arch = lookup_architecture(cfg)
    spec = arch.build_spec(arch.read_config(cfg))
    return spec, DecoderModel(spec, torch.float32, "cpu", max_positions=64)


def _random_weights(cfg, seed=0):
    from paged_llm_amd.weights.random_init import _declared_weights, draw_weights
    return dict(draw_weights(_declared_weights(cfg), seed, torch.float32, std=cfg["width"] ** -0.5, norm_jitter=True))


def d(*s):
    return torch.randn(*s, dtype=torch.float64)


# --------------------------------------------------------------------------- configuration and specification
def test_architecture_is_registered():
    from paged_llm_amd.config.registry import lookup_architecture
    assert lookup_architecture(PAMU_A).name == "Pamunex"


def test_specification():
    spec, m = build(PAMU_A)
    assert not m.state_specs() and len(m.blocks) == 6
    groups = list(m.cache_groups().values())
    assert sorted((g.spec.kind, g.spec.window, g.owners) for g in groups) == [("chunk", 21, [0]), ("chunk", 33, [4]), ("chunk", 50, [2]),
                                                                             ("window", 7, [5]), ("window", 19, [1]), ("window", 45, [3])]
    shapes = {n: tuple(s.shape) for n, s in m.weight_specs().items()}
    assert "head" not in shapes and shapes["embed"] == (300, 96) and shapes["final.norm"] == shapes["final.norm.b"] == (96,)
    for i in range(6):
        assert shapes[f"l{i}.norm1"] == shapes[f"l{i}.norm1.b"] == (96,)
        assert (f"l{i}.norm2" in shapes) == (f"l{i}.norm2.b" in shapes) == (PAMU_A["layers"][i]["mlp"] is not None)
    own = lambda i, part: {n.split(f"l{i}.{part}.")[1]: s for n, s in shapes.items() if n.startswith(f"l{i}.{part}.")}
    assert own(0, "mix") == {"q": (96, 96), "k": (48, 96), "v": (80, 96), "q.b": (96,), "k.b": (48,), "v.b": (80,), "q.norm": (24,), "k.norm": (24,),
                             "sink": (4,), "o": (96, 160)}
    assert own(1, "mix") == {"q": (96, 96), "dkv": (48, 96), "dkv.norm": (36,), "uk": (60, 36), "uv": (84, 36), "sink": (3,), "o": (96, 84)}
    assert own(0, "mlp") == {"up": (72, 96), "down": (96, 72)} and own(2, "mlp") == {}
    experts = {f"e{e}.{n}": s for e in range(8) for n, s in (("up", (40, 96)), ("down", (96, 40)))}
    assert own(1, "mlp") == {"router": (8, 96), **experts}


def test_bad_configurations_are_refused():
    from paged_llm_amd.config.registry import lookup_architecture
    arch = lookup_architecture(PAMU_A)
    for change in (lambda c: c["layers"][0].update(type="mamba1"), lambda c: c["layers"][0]["mlp"].update(kind="gated"),
                   lambda c: c["layers"][1]["mixer"]["rot"].update(dims=6), lambda c: c.update(layers=[]), lambda c: c.update(vocab=0)):
        bad = copy.deepcopy(PAMU_A)
        change(bad)
        with pytest.raises(ValueError):
            arch.read_config(bad)
    for i, change in ((0, {"kv_heads": 3}), (0, {"dim": 300}), (1, {"kv_rank": 1025})):
        bad = copy.deepcopy(PAMU_A)
        bad["layers"][i]["mixer"].update(change)
        with pytest.raises(ValueError):
            build(bad)
    bad = copy.deepcopy(PAMU_A)
    bad["layers"][1]["mlp"]["router"].update(top=5)                          # two groups of two experts hold four
    with pytest.raises(ValueError):
        build(bad)


def test_missing_and_further_tensors_are_named():
    from paged_llm_amd.weights.loader import WeightsError, load_state_dict
    cfg = PAMU_A
    weights = _random_weights(cfg)
    load_state_dict(build(cfg)[1], dict(weights, **{"l2.norm2": torch.ones(96), "l2.norm2.b": torch.ones(96)}))      # of a layer without a feed-forward
    with pytest.raises(WeightsError, match="l0.mix.sink"):
        load_state_dict(build(cfg)[1], {k: t for k, t in weights.items() if k != "l0.mix.sink"})
    with pytest.raises(WeightsError, match="l0.mix.o.b"):
        load_state_dict(build(cfg)[1], dict(weights, **{"l0.mix.o.b": torch.ones(96)}))


def test_the_scale_of_the_logits_is_a_factor_of_the_last_norm():
    from paged_llm_amd.weights.loader import load_state_dict
    for scale in (1.0, 0.37):
        cfg = model(64, 40, [layer("latent_attention", latent())], logit_scale=scale)
        weights = _random_weights(cfg)
        m = build(cfg)[1]
        load_state_dict(m, weights)
        assert torch.allclose(m.final_norm.weight, weights["final.norm"] * scale) and torch.allclose(m.final_norm.bias, weights["final.norm.b"] * scale)
        assert torch.equal(m.blocks[0].parts["mixer_norm"].weight, weights["l0.norm1"])


def test_every_configuration_builds():
    for cfg in (*ALONE.values(), PAMU_B, PAMU_C):
        _, m = build(cfg)
        assert set(_random_weights(cfg)) == set(m.weight_specs())


def test_bench_configuration_builds():
    import bench
    spec, m = build(bench.pamunex_config(1024, 32000))
    assert len(spec.layers) == 12 and m.graph_capturable() and m.graph_capturable(prompts=True)


# --------------------------------------------------------------------------- the plain mechanisms
def test_small_pieces():
    z = torch.tensor([-3.0, -0.0, 0.5, 2.0])
    assert plain.relu_squared(z).tolist() == [0.0, 0.0, 0.25, 4.0]
    x, w, b = d(3, 7), d(7), d(7)
    assert torch.allclose(plain.layer_norm(x, w, b, 1e-3), torch.nn.functional.layer_norm(x, (7,), w, b, 1e-3))
    assert torch.allclose(plain.unit_rms(x, 0.25)[1], x[1] / math.sqrt(float((x[1] ** 2).sum()) / 7 + 0.25))
    y = plain.rotate_halves(x[:, None], range(3), 4, 10.0)[:, 0]
    for p in range(3):
        for i in range(2):
            c, s = math.cos(p * 10.0 ** (-i / 2)), math.sin(p * 10.0 ** (-i / 2))
            assert torch.allclose(y[p, i], x[p, i] * c - x[p, i + 2] * s) and torch.allclose(y[p, i + 2], x[p, i + 2] * c + x[p, i] * s)
    assert torch.equal(y[:, 4:], x[:, 4:])


def test_masks():
    T = 11
    for size in (1, 3, 4, 20):
        block, window = plain.seen_in_block(T, size), plain.seen_in_window(T, size)
        for i in range(T):
            assert [j for j in range(T) if block[i, j]] == list(range(i - i % size, i + 1))
            assert [j for j in range(T) if window[i, j]] == list(range(max(0, i - size + 1), i + 1))


def test_a_sink_is_one_more_key_without_a_value():
    scores, seen = d(4, 5), plain.seen_in_window(5, 3)[1:]
    for sink in (-50.0, 0.3, 40.0):
        got = plain.softmax_with_sink(scores, seen, torch.tensor(sink, dtype=torch.float64))
        for i in range(4):
            keys = [j for j in range(5) if seen[i, j]]
            weights = torch.softmax(torch.cat([scores[i, keys], torch.tensor([sink], dtype=torch.float64)]), 0)
            assert torch.allclose(got[i, keys], weights[:-1]) and float(got[i].sum()) == pytest.approx(1 - float(weights[-1]))


def test_attention_query_by_query():
    torch.manual_seed(4)
    m, eps, T, W = blocks(heads=4, kv_heads=2, dim=6, vdim=5, size=3, rot_dims=4, base=20.0, scale=0.4), 1e-3, 8, 7
    w = {"q": d(24, W), "k": d(12, W), "v": d(10, W), "q.b": d(24), "k.b": d(12), "v.b": d(10), "q.norm": d(6), "k.norm": d(6), "sink": d(4), "o": torch.eye(20, dtype=torch.float64)}
    h = d(T, W)
    got = plain.attention(h, w, m, eps, range(T))

    def head(name, pos, at, turned=True):
        row = (w[name] @ h[pos] + w[name + ".b"])
        if not turned:
            return row[at * 5:at * 5 + 5]
        row = row[at * 6:at * 6 + 6]
        row = row / math.sqrt(float((row ** 2).mean()) + eps) * w[name + ".norm"]
        return plain.rotate_halves(row[None, None], [pos], 4, 20.0)[0, 0]
    for i in range(T):
        for a in range(4):
            keys = range(i - i % 3, i + 1)
            s = torch.stack([head("q", i, a) @ head("k", j, a // 2) * 0.4 for j in keys] + [w["sink"][a]])
            p = torch.softmax(s, 0)
            assert torch.allclose(got[i, a * 5:a * 5 + 5], sum(p[n] * head("v", j, a // 2, False) for n, j in enumerate(keys)))


def test_latent_attention_query_by_query():
    torch.manual_seed(5)
    m, T, W = latent(heads=2, dim=3, rot_dim=4, vdim=5, kv_rank=6, size=3, base=20.0, scale=0.4), 7, 8
    w = {"q": d(14, W), "dkv": d(10, W), "dkv.norm": d(6), "uk": d(6, 6), "uv": d(10, 6), "sink": d(2), "o": torch.eye(10, dtype=torch.float64)}
    h = d(T, W)
    got = plain.latent_attention(h, w, m, 1e-4, range(T))
    turn = lambda x, p: plain.rotate_halves(x[None, None], [p], 4, 20.0)[0, 0]
    for i in range(T):
        q = (h[i] @ w["q"].T).view(2, 7)
        for head in range(2):
            scores, values = [], []
            for j in range(max(0, i - 2), i + 1):
                dn = h[j] @ w["dkv"].T
                c = dn[:6] / math.sqrt(float((dn[:6] ** 2).mean()) + 1e-4) * w["dkv.norm"]
                scores.append((q[head, :3] @ (w["uk"] @ c)[head * 3:head * 3 + 3] + turn(q[head, 3:], i) @ turn(dn[6:], j)) * 0.4)
                values.append((w["uv"] @ c)[head * 5:head * 5 + 5])
            p = torch.softmax(torch.stack(scores + [w["sink"][head]]), 0)
            assert torch.allclose(got[i, head * 5:head * 5 + 5], sum(a * b for a, b in zip(p, values)))


def test_the_choice_by_hand():
    s = torch.tensor([[0.9, 0.1, 0.6, 0.5, 0.4, 0.45, 0.3, 0.2]])             # sums of the two largest: 1.0, 1.1, 0.85, 0.5
    assert sorted(plain.choose(s, 3, 4, 2)[0].tolist()) == [0, 2, 3]
    assert sorted(plain.choose(s, 2, 4, 1)[0].tolist()) == [2, 3]             # the largest score's own group is not the best
    assert sorted(plain.choose(s, 3, 1, 1)[0].tolist()) == [0, 2, 3]
    assert sorted(plain.choose(s, 2, 2, 1)[0].tolist()) == [0, 2]             # 1.5 against 0.85
    assert sorted(plain.choose(s, 2, 8, 2)[0].tolist()) == [0, 2]             # groups of one expert: the mark is its score


def test_routed_experts_token_by_token():
    torch.manual_seed(6)
    W, F, E, groups, keep, top = 6, 4, 9, 3, 2, 4
    w = {"router": d(E, W)}
    for e in range(E):
        w[f"e{e}.up"], w[f"e{e}.down"] = d(F, W), d(W, F)
    h = d(9, W)
    got = plain.routed(h, w, {"experts": E, "top": top, "groups": {"count": groups, "keep": keep}})
    for t in range(9):
        s = {e: 1 / (1 + math.exp(-float(w["router"][e] @ h[t]))) for e in range(E)}
        mark = {g: sum(sorted((s[e] for e in range(3 * g, 3 * g + 3)), reverse=True)[:2]) for g in range(groups)}
        open_groups = sorted(mark, key=mark.get, reverse=True)[:keep]
        best = sorted((e for e in range(E) if e // 3 in open_groups), key=s.get, reverse=True)[:top]
        want = sum(s[e] * (w[f"e{e}.down"] @ torch.relu(w[f"e{e}.up"] @ h[t]) ** 2) for e in best)
        assert torch.allclose(got[t], want)


def test_the_whole_model_is_the_sum_of_its_parts():
    cfg = PAMU_A
    w = {k: t.double() for k, t in _random_weights(cfg).items()}
    toks = [7, 1, 250, 33, 33, 9, 120, 5, 64]
    outs = []
    logits = plain.forward(cfg, w, toks, torch.float64, outs)
    eps = cfg["norm"]["eps"]
    norm = lambda x, n: torch.nn.functional.layer_norm(x, (96,), w[n], w[n + ".b"], eps)
    x = w["embed"][toks]
    for i, l in enumerate(cfg["layers"]):
        x = x + norm(plain.mixer(l, x, plain.under(w, f"l{i}.mix."), eps, range(9)), f"l{i}.norm1")
        if l["mlp"]:
            x = x + norm(plain.feed_forward(l["mlp"], x, plain.under(w, f"l{i}.mlp.")), f"l{i}.norm2")
        assert float((outs[i] - x).abs().max()) < 1e-9
    assert float((logits - 1.5 * norm(x, "final.norm") @ w["embed"].T).abs().max()) < 1e-9
    assert float((plain.forward(cfg, w, toks[:4], torch.float64) - logits[:4]).abs().max()) < 1e-9       # a later token changes nothing before it
