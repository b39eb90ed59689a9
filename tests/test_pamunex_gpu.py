"""Pamunex in the engine against the plain implementation under tests/plain/: each mechanism alone, whole prompts,
token-by-token decoding, portions down to two tokens, unequal requests in one batch with pages used again, keys far back, at
page borders and just inside and just outside every window and block (with weights made so that one score stands out), logits
without a key, groups of experts whose largest score misleads, the first tokens of a sequence, long decoding, sizes of several
kinds, and greedy generation through ``LLMEngine``."""

import copy
import os
import subprocess
import sys

import numpy as np
import pytest
import torch

from tests import helpers
from tests.helpers import TraceBuilder
from tests.pamunex_configs import ALONE, PAMU_A, PAMU_B, PAMU_C, blocks, dense, latent, layer, model, moe
from tests.plain import pamunex_plain as plain

pytestmark = pytest.mark.gpu


def without_experts(cfg):
    """The same layers with dense feed-forwards in the routed ones' place."""
    out = copy.deepcopy(cfg)
    for l in out["layers"]:
        if l["mlp"] and l["mlp"]["kind"] == "moe":
            l["mlp"] = dense(l["mlp"]["expert"]["ff"] * 2)
    return out


CONFIGS = {"A": PAMU_A, "B": PAMU_B, "C": PAMU_C, "A_dense": without_experts(PAMU_A), "B_dense": without_experts(PAMU_B),
           "C_dense": without_experts(PAMU_C), **ALONE}
NARROW = ("B", "B_dense")
TOL = {"float32": 3e-5, "bfloat16": 6e-2}
ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def lively(tensors):
    """Weights that leave no mechanism near its neutral point: logits without a key of both signs, weights of the q/k norm and
    of the latents' norm that differ from element to element, biases of the projections that are not small, router rows that
    spread the scores."""
    gen = torch.Generator().manual_seed(5)
    rnd = lambda t: torch.randn(t.shape, generator=gen)
    for name in list(tensors):
        t, new = tensors[name], None
        if name.endswith(".sink"):
            new = rnd(t) * 1.5
        elif name.endswith((".q.norm", ".k.norm", ".dkv.norm")):
            new = 1.0 + 0.4 * rnd(t)
        elif name.endswith((".q.b", ".k.b", ".v.b")):
            new = rnd(t) * 0.3
        elif name.endswith(".router"):
            new = t.float() * 2.0
        if new is not None:
            tensors[name] = new.to(t.dtype)


def write_folder(path, cfg, seed, stored, edit=None):
    from safetensors.torch import load_file, save_file
    from paged_llm_amd.weights import write_random_model
    folder = write_random_model(str(path), cfg, seed=seed, dtype=stored, std=cfg["width"] ** -0.5, norm_jitter=True)
    file = os.path.join(folder, "model.safetensors")
    tensors = load_file(file)
    lively(tensors)
    if edit is not None:
        edit(tensors)
    save_file({k: v.contiguous() for k, v in tensors.items()}, file)
    return folder


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    made = {}

    def get(name, stored):
        if (name, stored) not in made:
            made[name, stored] = write_folder(tmp_path_factory.mktemp(f"pamunex_{name}_{stored}"), CONFIGS[name],
                                              seed=29 + len(name), stored=stored)
        return made[name, stored]
    return get


_plain_cache: dict = {}


def plain_logits(folder, tokens):
    key = (folder, tuple(tokens))
    if key not in _plain_cache:
        _plain_cache[key] = plain.forward(plain.read_config(folder), plain.load_weights(folder), list(tokens)).numpy()
    return _plain_cache[key]


def session_for(folder, dtype, max_tokens, **kw):
    from paged_llm_amd.engine.replay import ReplaySession
    return ReplaySession(folder, dtype, max_tokens, None, **kw)


_noise_cache: dict = {}


def rounding_scale(folder, tokens):
    """Per position: how far the plain logits move (root mean square over four draws of ``helpers.worst``) when every
    product's rows and result carry the relative error of bfloat16 rounding."""
    key = (folder, tuple(tokens))
    if key not in _noise_cache:
        exact = plain_logits(folder, tokens)
        cfg, weights = plain.read_config(folder), plain.load_weights(folder)
        sq = np.zeros(len(tokens))
        for seed in range(4):
            with plain.rounding_noise(seed):
                moved = plain.forward(cfg, weights, list(tokens)).numpy()
            sq += (np.abs(moved - exact).max(axis=1) / np.abs(exact).max(axis=1)) ** 2
        _noise_cache[key] = np.sqrt(sq / 4)
    return _noise_cache[key]


_exact_cache: dict = {}


def float32_scale(folder, tokens):
    """Per position: how far the plain implementation in float32 is from itself in float64."""
    key = (folder, tuple(tokens))
    if key not in _exact_cache:
        exact = plain.forward(plain.read_config(folder), plain.load_weights(folder), list(tokens), dtype=torch.float64).numpy()
        _exact_cache[key] = np.abs(plain_logits(folder, tokens) - exact).max(axis=1) / np.abs(exact).max(axis=1)
    return _exact_cache[key]


def bound_at(folder, tokens, pos, dtype):
    """What a row may differ by: in float32 3e-5, or 5 times the plain implementation's own float32 error at that
    position if that is more; in bfloat16 4 times the position's rounding scale, at least 3e-2."""
    if dtype == "float32":
        return max(TOL[dtype], 5.0 * float(float32_scale(folder, tokens)[pos]))
    return max(3e-2, 4.0 * float(rounding_scale(folder, tokens)[pos]))


def check(got: dict, folder, reqs: dict, dtype, narrow=False):
    """Every row within its bound in float32.  In bfloat16, models without routed experts: no row beyond twice its bound (four
    times for ``narrow`` models, whose few channels average little rounding away), at most one in fifty beyond it, and the
    median error below 2.5e-2.  With routed experts the choice of an expert is a discrete step: where two router outputs are closer
    than the rounding of the rows in front of them the engine and the plain implementation may choose differently, which
    reaches every later position; such runs are judged by the median error and the share of rows beyond their bound (the
    float32 runs of the same models hold every row to its bound, and the same layers run with dense feed-forwards as well)."""
    want = {rid: plain_logits(folder, toks) for rid, toks in reqs.items()}
    routed = any((l.get("mlp") or {}).get("kind") == "moe" for l in plain.read_config(folder)["layers"])
    ratios, errs = {}, []
    for (rid, pos), row in got.items():
        err = helpers.worst(row, want[rid][pos])
        errs.append(err)
        ratios[rid, pos] = err / bound_at(folder, reqs[rid], pos, dtype)
    worst_at = max(ratios, key=ratios.get)
    over = sum(1 for r in ratios.values() if r > 1.0)
    said = f"{worst_at}: {ratios[worst_at]:.3g} of its bound (median error {np.median(errs):.3g}), {over} of {len(ratios)} rows over"
    if dtype == "float32":
        assert ratios[worst_at] <= 1.0, said
    elif routed:
        assert np.median(errs) <= 5e-2 and over <= len(ratios) // 2, said
    else:
        most, middle = (4.0, 5e-2) if narrow else (2.0, 2.5e-2)
        assert ratios[worst_at] <= most and over <= max(1, len(ratios) // 50) and np.median(errs) <= middle, said


def whole(reqs):
    trace = TraceBuilder()
    for rid, toks in reqs.items():
        trace.step([(rid, toks, "all")], end=[rid])
    return trace


def prompt_then_single(rid, toks, cut, want="all"):
    trace = TraceBuilder().step([(rid, toks[:cut], want)], end=[rid] if cut == len(toks) else [])
    for i in range(cut, len(toks)):
        trace.step([(rid, toks[i:i + 1], "all")], end=[rid] if i == len(toks) - 1 else [])
    return trace


def stored_as(dtype):
    return "float32" if dtype == "float32" else "bfloat16"


# --------------------------------------------------------------------------- each mechanism alone, and whole models
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", sorted(CONFIGS))
def test_whole_prompts(folders, name, dtype):
    folder = folders(name, stored_as(dtype))
    vocab = CONFIGS[name]["vocab"]
    reqs = {"p1": helpers.random_tokens(1, vocab, 1), "p5": helpers.random_tokens(5, vocab, 2), "p70": helpers.random_tokens(70, vocab, 3)}
    got = helpers.replay_in_process(session_for(folder, dtype, 128), whole(reqs))
    assert len(got) == 76
    check(got, folder, reqs, dtype, narrow=name in NARROW)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "A_dense", "B_dense", "C_dense", "blocks", "latent", "latent_wide", "moe"])
def test_prompt_then_token_by_token(folders, name, dtype):
    """A prompt in one step and then single tokens, replayed from graphs: pages, windows and blocks whose edges pass among decoded
    tokens."""
    folder = folders(name, stored_as(dtype))
    toks = helpers.random_tokens(75, CONFIGS[name]["vocab"], 17)
    session = session_for(folder, dtype, 128)
    check(helpers.replay_in_process(session, prompt_then_single("r", toks, 13)), folder, {"r": toks}, dtype, narrow=name in NARROW)
    assert any(key[0] != "prompt" for key in session.runner._graphs), "single-token steps are replayed from graphs"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "A_dense", "C_dense"])
def test_token_by_token_from_the_first(folders, name, dtype):
    """No prompt step at all: the first queries see themselves and the logit without a key, windows and blocks of one position."""
    folder = folders(name, stored_as(dtype))
    toks = helpers.random_tokens(12, CONFIGS[name]["vocab"], 8)
    check(helpers.replay_in_process(session_for(folder, dtype, 64), prompt_then_single("r", toks, 1)), folder, {"r": toks}, dtype, narrow=name in NARROW)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "A_dense", "C_dense"])
@pytest.mark.parametrize("sizes", [[2], [3, 2, 7], [16, 1, 17, 2, 31], [64, 5]])
def test_portions(folders, name, dtype, sizes):
    """Prompts cut into portions of several sizes, down to two tokens, cut in the middle of pages, windows and blocks."""
    folder = folders(name, stored_as(dtype))
    toks = helpers.random_tokens(97, CONFIGS[name]["vocab"], 9)
    trace, at, k = TraceBuilder(), 0, 0
    while at < len(toks):
        n = min(sizes[k % len(sizes)], len(toks) - at)
        trace.step([("r", toks[at:at + n], "all")], end=["r"] if at + n == len(toks) else [])
        at, k = at + n, k + 1
    check(helpers.replay_in_process(session_for(folder, dtype, 128), trace), folder, {"r": toks}, dtype, narrow=name in NARROW)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "A_dense", "B", "C_dense"])
def test_long_portions(folders, name, dtype):
    """Portions of hundreds of tokens (a short sequence beside the long one), whose queries' windows and blocks lie inside the
    portion and in front of it, then single tokens."""
    folder = folders(name, stored_as(dtype))
    vocab = CONFIGS[name]["vocab"]
    reqs = {"long": helpers.random_tokens(437, vocab, 11), "short": helpers.random_tokens(9, vocab, 12)}
    trace = TraceBuilder().step([("long", reqs["long"][:301], [0, 30, 31, 32, 33, 63, 64, 300]), ("short", reqs["short"][:7], "all")])
    trace.step([("long", reqs["long"][301:431], [0, 1, 31, 32, 63, 64, 65, 129]), ("short", reqs["short"][7:8], "all")])
    trace.step([("short", reqs["short"][8:], "all")], end=["short"])
    for i in range(431, 437):
        trace.step([("long", reqs["long"][i:i + 1], "all")], end=["long"] if i == 436 else [])
    check(helpers.replay_in_process(session_for(folder, dtype, 576), trace), folder, reqs, dtype, narrow=name in NARROW)


@pytest.mark.parametrize("name,dtype", [("A", "float32"), ("A_dense", "float32"), ("C_dense", "float32"), ("A_dense", "bfloat16"), ("C_dense", "bfloat16")])
def test_logits_do_not_depend_on_the_cut(folders, name, dtype):
    """The same request whole, in portions and token by token: equal within rounding of the compute type."""
    folder = folders(name, stored_as(dtype))
    toks = helpers.random_tokens(60, CONFIGS[name]["vocab"], 10)
    a = helpers.replay_in_process(session_for(folder, dtype, 64), whole({"r": toks}))
    trace = TraceBuilder().step([("r", toks[:31], "all")]).step([("r", toks[31:33], "all")])
    for i in range(33, 60):
        trace.step([("r", toks[i:i + 1], "all")], end=["r"] if i == 59 else [])
    b = helpers.replay_in_process(session_for(folder, dtype, 64), trace)
    if dtype == "float32":
        assert max(helpers.worst(b[k], a[k]) / bound_at(folder, toks, k[1], dtype) for k in a) <= 1.0
    else:
        assert max(helpers.worst(b[k], a[k]) / bound_at(folder, toks, k[1], dtype) for k in a) <= 2.0


# --------------------------------------------------------------------------- batches, pages used again
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["A", "B", "C", "A_dense"])
def test_mixed_batches_with_pages_used_again(folders, name, dtype):
    from tests.test_replay_gpu import mixed_trace
    folder = folders(name, stored_as(dtype))
    vocab = CONFIGS[name]["vocab"]
    lengths = [33, 1, 90, 17, 64, 5, 48, 2, 71]
    reqs = {f"q{i}": helpers.random_tokens(n, vocab, 40 + i) for i, n in enumerate(lengths)}
    trace, peak = mixed_trace(reqs, max_live=3, seed=3)
    session = session_for(folder, dtype, peak, max_requests=3)
    got = helpers.replay_in_process(session, trace)
    assert len(got) == sum(lengths)
    check(got, folder, reqs, dtype, narrow=name in NARROW)
    session.manager.check_invariants()
    assert all(session.manager.num_free_pages(g) == session.manager.num_pages(g) for g in session.manager.groups)
    kinds = {"prompt" if key[0] == "prompt" else "decode" for key in session.runner._graphs}
    assert kinds == {"prompt", "decode"}, "steps of both kinds were replayed from graphs"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_pages_that_another_request_left_full(folders, dtype):
    """A page pool of one request: the second request gets the pages the first one left full, in windows and blocks whose
    pages are given back while the request runs."""
    folder = folders("A_dense", stored_as(dtype))
    vocab = PAMU_A["vocab"]
    reqs = {"first": helpers.random_tokens(62, vocab, 60), "second": helpers.random_tokens(57, vocab, 61)}
    trace = TraceBuilder()
    for rid, toks in reqs.items():
        trace.step([(rid, toks[:20], "all")])
        trace.step([(rid, toks[20:22], "all")])
        for i in range(22, len(toks)):
            trace.step([(rid, toks[i:i + 1], "all")], end=[rid] if i == len(toks) - 1 else [])
    check(helpers.replay_in_process(session_for(folder, dtype, 64, max_requests=1), trace), folder, reqs, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_long_decoding(folders, dtype):
    """Two hundred single tokens behind a short prompt: the context passes a dozen page borders and every window's and block's edge
    several times."""
    folder = folders("A_dense", stored_as(dtype))
    toks = helpers.random_tokens(215, PAMU_A["vocab"], 70)
    check(helpers.replay_in_process(session_for(folder, dtype, 256), prompt_then_single("r", toks, 15)), folder, {"r": toks}, dtype)


# --------------------------------------------------------------------------- where random weights would hide a fault
def aimed_blocks(size, dtype, key_pos, at, n, seed):
    """(configuration, tokens, edit): one attention layer whose head 0, at the positions ``at``, has the query that the key at
    ``key_pos`` has in its elements that are not rotated, and zero in the rotated ones: the largest product that normed rows
    of their lengths can have.  The sublayer reads the embedding itself, so the queries' tokens get the embedding that the
    projection maps to that row."""
    m = blocks(heads=2, kv_heads=1, dim=32, vdim=16, size=size, rot_dims=4, base=100.0, scale=0.6)
    cfg = model(64, 120, [layer("attention", m)], eps=1e-6)
    toks = [5 + t % 100 for t in helpers.random_tokens(n, 100, seed)]
    toks[key_pos] = 4                                       # the key's token stands nowhere else
    for pos in at:
        toks[pos] = 3                                       # ... and the aimed query's token only here

    def edit(t):
        f = lambda name: t[name].to(torch.float64)
        t["l0.mix.q.b"] = (t["l0.mix.q.b"].float() * 0.1).to(t["embed"].dtype)
        key = f("l0.mix.k") @ f("embed")[4] + f("l0.mix.k.b")
        key = plain.unit_rms(key, 1e-6) * f("l0.mix.k.norm")
        key[:4] = 0.0
        row = key / f("l0.mix.q.norm")                      # (the query's own weight turns it into the key again)
        row = row / row.norm() * 0.5                        # (a short embedding: the sublayer's part of the stream outweighs it)
        e = torch.linalg.lstsq(f("l0.mix.q")[:32], (row - f("l0.mix.q.b")[:32])[:, None]).solution[:, 0]
        t["embed"][3] = e.to(t["embed"].dtype)
    return cfg, toks, edit


def aimed_latent(size, dtype, key_pos, at, n, seed, kv_rank=24):
    """The same with a latent attention layer: the key's token and the queries' token have embeddings along one unit vector
    each; the latent of the key's token lights one element up, which other tokens hardly have and which head 0's
    up-projection of keys meets with the column that head 0's query of the aimed token carries."""
    cfg = model(128, 120, [layer("latent_attention", latent(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=kv_rank, size=size, base=100.0))], eps=1e-6)
    toks = [5 + t % 100 for t in helpers.random_tokens(n, 100, seed)]
    toks[key_pos] = 4
    for pos in at:
        toks[pos] = 3

    def edit(t):
        gen = torch.Generator().manual_seed(77)
        stored = t["embed"].dtype
        for token, col in ((4, 1), (3, 2)):
            e = torch.zeros(128)
            e[col] = 1.0
            t["embed"][token] = e.to(stored)
        down, uk, q = t["l0.mix.dkv"].float(), t["l0.mix.uk"].float(), t["l0.mix.q"].float()
        down[:kv_rank, 1] = 0
        down[0, 1] = 3.0
        down[0, 2:] *= 0.05
        target = torch.randn(16, generator=gen)
        target *= 6.0 / target.norm()
        uk[:16, 0] = target
        q[:16, 2] = target
        q[:16, :2] = 0
        t["l0.mix.dkv"], t["l0.mix.uk"], t["l0.mix.q"] = down.to(stored), uk.to(stored), q.to(stored)
        t["l0.mix.dkv.norm"][0] = 1.0
    return cfg, toks, edit


def edge_case(tmp_path, kind, size, key_pos, dtype, seed=31, **kw):
    """(folder, tokens, last position that sees the key, first that does not), queries aimed at the key on both sides."""
    edge_in = key_pos + size - 1 if kind == "latent" else (key_pos // size + 1) * size - 1
    at, n = [edge_in - 1, edge_in, edge_in + 1, edge_in + 2], edge_in + 6
    cfg, toks, edit = (aimed_latent if kind == "latent" else aimed_blocks)(size, dtype, key_pos, at, n, seed, **kw)
    return write_folder(tmp_path, cfg, seed=seed, stored=stored_as(dtype), edit=edit), toks, edge_in, edge_in + 1


def assert_edge_shows(folder, toks, edge_in, edge_out, dtype):
    """The plain implementation with a mask one position larger or smaller differs far beyond the bound at the edge."""
    want = plain_logits(folder, toks)
    for off_by in (-1, 1):
        other = plain.read_config(folder)
        other["layers"][0]["mixer"]["mask"]["size"] += off_by
        moved = plain.forward(other, plain.load_weights(folder), toks).numpy()
        pos = edge_in if off_by < 0 else edge_out
        assert helpers.worst(moved[pos], want[pos]) > 5 * bound_at(folder, toks, pos, dtype), "the aimed key does not show at the edge"
    return want


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,size,key_pos,kw", [
    ("latent", 9, 20, {}), ("latent", 130, 3, {}), ("latent", 64, 63, {}), ("latent", 33, 15, {"kv_rank": 270}), ("latent", 16, 16, {"kv_rank": 100}),
    ("blocks", 9, 20, {}), ("blocks", 150, 151, {}), ("blocks", 64, 64, {}), ("blocks", 50, 79, {}), ("blocks", 37, 0, {})])
def test_edges_of_windows_and_blocks_in_prompts_and_in_decoding(tmp_path, kind, size, key_pos, kw, dtype):
    """One key that the queries near the edge score far above all others: the last position that sees it and the
    first that does not are compared whole, with the edge among decoded tokens, with everything behind the key decoded
    and with the edge at the start of a portion of two tokens.  Small masks, masks of more than two pages (the key far
    back, over page borders), masks of whole pages with the key on a page's first or last place, a latent that the paged
    attention kernels do not take."""
    folder, toks, edge_in, edge_out = edge_case(tmp_path, kind, size, key_pos, dtype, **kw)
    want = assert_edge_shows(folder, toks, edge_in, edge_out, dtype)
    n = len(toks)
    traces = {"whole": prompt_then_single("r", toks, n), "edge decoded": prompt_then_single("r", toks, edge_in - 3),
              "all decoded": prompt_then_single("r", toks, key_pos + 1),
              "edge starts a portion": TraceBuilder().step([("r", toks[:edge_in], "all")]).step([("r", toks[edge_in:edge_in + 2], "all")])
              .step([("r", toks[edge_in + 2:], "all")], end=["r"])}
    for label, trace in traces.items():
        got = helpers.replay_in_process(session_for(folder, dtype, -(-n // 64) * 64), trace)
        for pos in (edge_in - 1, edge_in, edge_out, edge_out + 1):
            err = helpers.worst(got["r", pos], want[pos])
            assert err <= 2.0 * bound_at(folder, toks, pos, dtype), f"{label}, position {pos}: {err:.3g}"


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind,size,key_pos", [("latent", 400, 7), ("latent", 400, 0), ("blocks", 420, 17), ("blocks", 410, 411)])
def test_a_key_far_back_among_hundreds(tmp_path, kind, size, key_pos, dtype):
    """The aimed key hundreds of tokens back among as many others, over many page borders, through portions of several sizes and
    decoded tokens."""
    folder, toks, edge_in, edge_out = edge_case(tmp_path, kind, size, key_pos, dtype, seed=37)
    assert_edge_shows(folder, toks, edge_in, edge_out, dtype)
    trace, at, k, sizes = TraceBuilder(), 0, 0, (17, 2, 64, 100, 3, 96, 60)
    while at < edge_in - 3:
        n = min(sizes[k % len(sizes)], edge_in - 3 - at)
        trace.step([("r", toks[at:at + n], "last")])
        at, k = at + n, k + 1
    for i in range(at, len(toks)):
        trace.step([("r", toks[i:i + 1], "all")], end=["r"] if i == len(toks) - 1 else [])
    got = helpers.replay_in_process(session_for(folder, dtype, -(-len(toks) // 64) * 64), trace)
    check(got, folder, {"r": toks}, dtype)
    assert ("r", edge_in) in got and ("r", edge_out) in got


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["blocks", "latent", "latent_wide"])
def test_logits_without_a_key_in_the_softmax(tmp_path, name, dtype):
    """Per-head logits of both signs in the denominator: where few keys stand beside them (the first tokens of a block or of the
    sequence) the large ones take most of the weight.  Without them the plain logits differ far beyond the bound, also one by
    one (a head that got its neighbour's number shows)."""
    cfg = ALONE[name]
    heads = cfg["layers"][0]["mixer"]["heads"]

    def edit(tensors):
        tensors["l0.mix.sink"] = torch.tensor([3.0, -2.0, 2.5, 0.0][:heads]).to(tensors["l0.mix.sink"].dtype)
    folder = write_folder(tmp_path, cfg, seed=41, stored=stored_as(dtype), edit=edit)
    toks = helpers.random_tokens(40, cfg["vocab"], 15)
    want = plain_logits(folder, toks)
    weights = plain.load_weights(folder)
    for other in (torch.full((heads,), -1e4), weights["l0.mix.sink"].float().roll(1)):
        moved = plain.forward(plain.read_config(folder), dict(weights, **{"l0.mix.sink": other}), toks).numpy()
        # (the first token: a softmax over one key and the logit, of any size, scales a head's value alone)
        assert max(helpers.worst(moved[p], want[p]) for p in (0, 1, 9, 18, 27)) > 3 * TOL["bfloat16"]
    for cut in (40, 8, 1):
        check(helpers.replay_in_process(session_for(folder, dtype, 64), prompt_then_single("r", toks, cut)), folder, {"r": toks}, dtype)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_experts_with_a_decisive_choice(tmp_path, dtype):
    """Router rows that meet one common direction of all embeddings with sizes set well apart: the scores differ from
    token to token by far less than that, so the choice is the same under any rounding while the weights still differ.  The
    group of the largest score is not among the two that are kept (its second score is small), so a mark by the largest score
    alone chooses otherwise.  Then bfloat16 rows of a model with experts can be held to the bounds of rows without."""
    cfg = ALONE["moe"]
    levels = torch.tensor([2.0, -3.0, -3.5, 1.2, 1.0, -1.0, 0.8, 0.3, -2.0, -0.5, -0.8, -1.2])       # groups of three; the marks of groups 1 and 2 win

    def edit(tensors):
        stored = tensors["embed"].dtype
        tensors["l0.norm1"] = (tensors["l0.norm1"].float() * 0.2).to(stored)
        tensors["embed"] = tensors["embed"].float() * 0.3
        tensors["embed"][:, 0] = 1.0
        tensors["embed"] = tensors["embed"].to(stored)
        tensors["l0.norm1.b"] = torch.zeros_like(tensors["l0.norm1.b"])
        tensors["l0.norm1"][0] = 0.0
        router = tensors["l0.mlp.router"].float() * 0.1
        router[:, 0] = levels
        tensors["l0.mlp.router"] = router.to(stored)
    folder = write_folder(tmp_path, cfg, seed=43, stored=stored_as(dtype), edit=edit)
    toks = helpers.random_tokens(80, cfg["vocab"], 16)
    chosen, real = [], plain.choose
    try:
        plain.choose = lambda s, *a: (chosen.append((s, real(s, *a))), chosen[-1][1])[1]
        plain.forward(plain.read_config(folder), plain.load_weights(folder), toks)
    finally:
        plain.choose = real
    scores, ids = chosen[0]
    assert {tuple(sorted(c)) for c in ids.tolist()} == {(3, 4, 6)} and float(torch.gather(scores, 1, ids).std(0).min()) > 1e-3
    got = helpers.replay_in_process(session_for(folder, dtype, 128), prompt_then_single("r", toks, 60))
    want = plain_logits(folder, toks)
    for (rid, pos), row in got.items():
        err = helpers.worst(row, want[pos])
        assert err <= 2.0 * bound_at(folder, toks, pos, dtype), (pos, err)


def random_config(seed):
    rng = np.random.default_rng(seed)
    pick = lambda *xs: xs[int(rng.integers(0, len(xs)))]
    layers = []
    for _ in range(int(rng.integers(1, 6))):
        kind = pick("attention", "latent_attention")
        if kind == "attention":
            dim, kv = int(pick(2, 8, 16, 30, 64, 96, 128, 130)), int(pick(1, 2, 3))
            m = blocks(heads=kv * int(pick(1, 2, 5, 8)), kv_heads=kv, dim=dim, vdim=int(pick(5, 16, 64, 100)), size=int(pick(1, 7, 16, 40, 64, 500)),
                       rot_dims=int(pick(2, dim // 4 * 2 or 2, dim)), base=float(pick(10.0, 1e4, 5e5)), scale=float(pick(0.08, 0.2)))
        else:
            m = latent(heads=int(pick(1, 2, 4, 7)), dim=int(pick(4, 16, 31, 64)), rot_dim=int(pick(2, 6, 16, 64)), vdim=int(pick(5, 16, 64)),
                       kv_rank=int(pick(7, 32, 64, 192, 300)), size=int(pick(1, 5, 16, 33, 64, 500)), base=float(pick(10.0, 1e4, 5e5)), scale=float(pick(0.1, 0.3)))
        f = pick(None, "dense", "moe", "moe")
        count, per = int(pick(1, 2, 3, 4)), int(pick(1, 2, 5))
        keep = int(rng.integers(1, count + 1))
        layers.append(layer(kind, m, dense(int(pick(24, 100))) if f == "dense" else
                            moe(count * per, int(rng.integers(1, min(keep * per, 6) + 1)), count, keep, int(pick(8, 30, 64))) if f == "moe" else None))
    return model(int(pick(40, 50, 64, 128)), int(pick(50, 200, 333)), layers, eps=float(pick(1e-6, 1e-5, 1e-2)), logit_scale=float(pick(0.3, 1.0, 4.0)))


@pytest.mark.parametrize("seed", range(12))
def test_configurations_drawn_at_random(tmp_path, seed):
    """Sizes, constants, options and layer orders drawn at random, in float32: a prompt, a portion of two tokens, single
    tokens, with a second request beside the first."""
    cfg = random_config(5000 + seed)
    folder = write_folder(tmp_path, cfg, seed=seed, stored="float32")
    reqs = {"a": helpers.random_tokens(83, cfg["vocab"], seed), "b": helpers.random_tokens(21, cfg["vocab"], 100 + seed)}
    trace = TraceBuilder().step([("a", reqs["a"][:49], "all")]).step([("a", reqs["a"][49:51], "all"), ("b", reqs["b"][:18], "all")])
    for i in range(51, 83):
        k = i - 51 + 18
        trace.step([("a", reqs["a"][i:i + 1], "all")] + ([("b", reqs["b"][k:k + 1], "all")] if k < 21 else []),
                   end=(["a"] if i == 82 else []) + (["b"] if k == 20 else []))
    got = helpers.replay_in_process(session_for(folder, "float32", 192), trace)
    assert len(got) == 104
    check(got, folder, reqs, "float32")


# --------------------------------------------------------------------------- the engine's own entry point
@pytest.mark.parametrize("name", ["A_dense", "C_dense", "B"])
def test_greedy_generation_through_the_engine(folders, name):
    """``LLMEngine.generate`` with portions of 16 tokens, three requests at a time for five prompts (pages are
    used again): every row the engine sampled from is within the bound of the plain logits along its own
    tokens, and in float32 the tokens are the plain implementation's greedy choice."""
    from paged_llm_amd import EngineConfig, SamplingParams
    from paged_llm_amd.engine.llm_engine import LLMEngine
    vocab = CONFIGS[name]["vocab"]
    prompts = [helpers.random_tokens(n, vocab, 70 + n) for n in (3, 41, 18, 1, 29)]
    for dtype in ("float32", "bfloat16"):
        folder = folders(name, stored_as(dtype))
        engine = LLMEngine(folder, EngineConfig(dtype=dtype, num_gpu_blocks=24, block_size=16, max_num_batched_tokens=16,
                                                max_num_seqs=3, max_model_len=128))
        rows = {}

        def keep(requests, logits):
            for r, row in zip(requests, logits.float().cpu()):
                rows[r.id, len(r.tokens) - 1] = row.numpy()
        engine.on_logits = keep
        outs = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=12, ignore_eos=True))
        for p, o in zip(prompts, outs):
            assert len(o.token_ids) == 12
            want = plain_logits(folder, p + o.token_ids)
            for i, token in enumerate(o.token_ids):
                pos = len(p) + i - 1
                err = helpers.worst(rows[o.seq_id, pos], want[pos])
                assert err <= 2.0 * bound_at(folder, p + o.token_ids, pos, dtype) and int(rows[o.seq_id, pos].argmax()) == token, (dtype, pos, err)
                if dtype == "float32":
                    top2 = np.sort(want[pos])[-2:]
                    if top2[1] - top2[0] > 1e-3 * np.abs(want[pos]).max():
                        assert token == int(want[pos].argmax()), (pos, token)


def test_preempted_requests_are_computed_again(tmp_path):
    """A page pool too small for three requests at once: the scheduler preempts the request admitted last (its pages are given
    back, its tokens kept) and computes it again later as a longer prompt.  Float32: the tokens are the plain implementation's
    greedy choice all the same."""
    from paged_llm_amd import EngineConfig, SamplingParams
    from paged_llm_amd.engine.llm_engine import LLMEngine
    cfg = copy.deepcopy(PAMU_A)
    for l in cfg["layers"]:
        l["mixer"]["mask"]["size"] = 200                    # nothing leaves sight, so no page goes back while a request runs
    folder = write_folder(tmp_path, cfg, seed=29, stored="float32")
    vocab = cfg["vocab"]
    prompts = [helpers.random_tokens(n, vocab, 400 + n) for n in (30, 22, 27)]
    engine = LLMEngine(folder, EngineConfig(dtype="float32", num_gpu_blocks=10, block_size=16, max_num_batched_tokens=32,
                                            max_num_seqs=3, max_model_len=128))
    outs = engine.generate(prompts, SamplingParams(temperature=0.0, max_tokens=40, ignore_eos=True))
    assert engine.stats.num_preemptions > 0 and sum(o.num_preemptions for o in outs) > 0
    for p, o in zip(prompts, outs):
        assert len(o.token_ids) == 40
        want = plain_logits(folder, p + o.token_ids)
        for i, token in enumerate(o.token_ids):
            row = want[len(p) + i - 1]
            top2 = np.sort(row)[-2:]
            if top2[1] - top2[0] > 1e-3 * np.abs(row).max():
                assert token == int(row.argmax()), (len(p), i)


def test_the_replay_program_and_the_command_line(folders, tmp_path):
    folder = folders("B", "float32")
    toks = helpers.random_tokens(30, PAMU_B["vocab"], 5)
    trace = TraceBuilder().step([("r", toks[:20], "last")]).step([("r", toks[20:], "all")], end=["r"])
    out = tmp_path / "out"
    done = subprocess.run([os.path.join(ROOT, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(out), "--max-tokens", "64"],
                          input=trace.jsonl(), capture_output=True, text=True, timeout=600)
    assert done.returncode == 0, done.stderr[-2000:]
    assert [l for l in done.stdout.split("\n") if l.startswith("done")] == ["done 0", "done 1"]
    got = helpers.read_replay_output(str(out), trace, PAMU_B["vocab"])
    check(got, folder, {"r": toks}, "float32")
    gen = subprocess.run([sys.executable, os.path.join(ROOT, "examples", "generate.py"), "--model", folder, "--dtype", "float32",
                          "--prompt-ids", ",".join(str(t) for t in toks[:9]), "--prompt-ids", "9", "--max-tokens", "5", "--num-gpu-blocks", "16",
                          "--max-model-len", "64", "--ignore-eos"], capture_output=True, text=True, timeout=600)
    assert gen.returncode == 0, gen.stderr[-2000:]
