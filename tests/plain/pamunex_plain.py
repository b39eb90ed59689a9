"""A plain, slow Pamunex: whole sequences, no cache, no paging, no batches, one function per mechanism.

Pamunex keeps the token embedding as its residual stream; a sublayer reads the stream itself and a layer norm (weight and
bias) stands on what it returns, x <- x + LN1(mixer(x)), x <- x + LN2(ff(x)).  A layer holds one of two mixers:

* ``attention``: grouped heads with biases on q, k and v, queries and keys divided by their root mean square per head and
  multiplied by a weight, then turned (pairs (i, i + r/2) of the first r elements); a query sees the keys of its own block
  of positions; the softmax's denominator holds one more learned term per head.
* ``latent_attention``: keys and values from one normed latent per token, one rotated key part for all heads, a sliding
  window, the same further term in the denominator.

and a dense feed-forward without a gate (the square of relu) or routed experts of the same form: sigmoid scores, groups of
neighbouring experts marked by the sum of their two largest scores, weights = the chosen scores as they are.  The logits come
from the embedding table, times a constant.  Everything is computed in one floating type chosen by the caller.  It shares no
code with the engine under ``paged-llm_amd/``.
"""

from __future__ import annotations

import json
import os

import torch


def read_config(model_dir: str) -> dict:
    with open(os.path.join(model_dir, "config.json")) as f:
        return json.load(f)


def load_weights(model_dir: str) -> dict:
    from safetensors import safe_open
    out = {}
    with safe_open(os.path.join(model_dir, "model.safetensors"), framework="pt", device="cpu") as f:
        for name in f.keys():
            out[name] = f.get_tensor(name)
    return out


# --------------------------------------------------------------------------- small pieces
def unit_rms(x, eps):
    """x divided by the root of its mean square."""
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def layer_norm(x, w, b, eps):
    centred = x - x.mean(-1, keepdim=True)
    return centred / torch.sqrt((centred * centred).mean(-1, keepdim=True) + eps) * w + b


def relu_squared(z):
    return torch.clamp(z, min=0) ** 2


_NOISE = None      # a function applied to every product's operand rows and result (see ``rounding_noise``), or None


def product(x, w, b=None):
    """x W^T (+ b); with ``_NOISE`` set, rows and result are disturbed as a 16-bit compute type would round them."""
    if _NOISE is None:
        y = x @ w.T
        return y if b is None else y + b
    y = _NOISE(x) @ w.T
    return _NOISE(y if b is None else y + b)


class rounding_noise:
    """Inside ``with rounding_noise(seed):`` every product's rows and result are multiplied by 1 + u * 2^-8 with u uniform
    in (-1, 1), drawn from ``seed``: the relative error of two roundings to bfloat16, at random.  Several seeds show how
    far the logits of one position move under the compute type's rounding alone; norms, scores, the router and the residual
    stream stay exact, as the design keeps them in 32 bits."""

    def __init__(self, seed: int, amplitude: float = 2.0 ** -8):
        self.gen = torch.Generator().manual_seed(seed)
        self.amplitude = amplitude

    def __call__(self, t):
        return t * (1.0 + (torch.rand(t.shape, generator=self.gen, dtype=t.dtype) * 2.0 - 1.0) * self.amplitude)

    def __enter__(self):
        global _NOISE
        _NOISE = self
        return self

    def __exit__(self, *exc):
        global _NOISE
        _NOISE = None


def embedding(tokens, table):
    return table[torch.tensor(list(tokens))]


def rotate_halves(x, positions, dims: int, base: float):
    """x [T, heads, r]: pairs (i, i + dims/2) of the first ``dims`` elements turned by position * base^(-2i/dims)."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    ang = torch.tensor(list(positions), dtype=torch.float64)[:, None] * f[None, :]
    cos, sin = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


# --------------------------------------------------------------------------- mixers
def seen_in_block(T: int, size: int):
    """[T, T]: row i marks the keys j <= i of i's own block of ``size`` positions, counted from position 0 (size 0: every j <= i)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i // size == j // size) if size > 0 else j <= i


def seen_in_window(T: int, size: int):
    """[T, T]: row i marks the keys i - size < j <= i (size 0: every j <= i)."""
    i, j = torch.arange(T)[:, None], torch.arange(T)[None, :]
    return (j <= i) & (i - j < size) if size > 0 else j <= i


def softmax_with_sink(scores, seen, sink):
    """exp(s_ij) over exp(sink) + sum_j exp(s_ij), over the seen keys; ``sink`` a scalar tensor."""
    scores = scores.masked_fill(~seen, float("-inf"))
    top = torch.maximum(scores.max(-1, keepdim=True).values, sink)
    e = torch.exp(scores - top)
    return e / (e.sum(-1, keepdim=True) + torch.exp(sink - top))


def mask_size(m: dict) -> int:
    return int((m.get("mask") or {}).get("size") or 0)


def attention(h, w: dict, m: dict, eps: float, positions):
    T = h.shape[0]
    H, G, d, dv = int(m["heads"]), int(m["kv_heads"]), int(m["dim"]), int(m["vdim"])
    q = product(h, w["q"], w["q.b"]).view(T, H, d)
    k = product(h, w["k"], w["k.b"]).view(T, G, d)
    v = product(h, w["v"], w["v.b"]).view(T, G, dv)
    q, k = unit_rms(q, eps) * w["q.norm"], unit_rms(k, eps) * w["k.norm"]
    if m.get("rot"):
        q, k = (rotate_halves(t, positions, int(m["rot"]["dims"]), float(m["rot"]["base"])) for t in (q, k))
    seen = seen_in_block(T, mask_size(m))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        g = head // (H // G)
        out[:, head] = softmax_with_sink((q[:, head] @ k[:, g].T) * float(m["scale"]), seen, w["sink"][head]) @ v[:, g]
    return product(out.reshape(T, H * dv), w["o"])


def latent_attention(h, w: dict, m: dict, eps: float, positions):
    T = h.shape[0]
    H, d, r, dv, rank = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    q = product(h, w["q"]).view(T, H, d + r)
    down = product(h, w["dkv"])
    c = unit_rms(down[:, :rank], eps) * w["dkv.norm"]
    kr = rotate_halves(down[:, None, rank:], positions, r, float(m["rot"]["base"]))[:, 0]
    qr = rotate_halves(q[..., d:], positions, r, float(m["rot"]["base"]))
    k, v = product(c, w["uk"]).view(T, H, d), product(c, w["uv"]).view(T, H, dv)
    seen = seen_in_window(T, mask_size(m))
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        s = (q[:, head, :d] @ k[:, head].T + qr[:, head] @ kr.T) * float(m["scale"])
        out[:, head] = softmax_with_sink(s, seen, w["sink"][head]) @ v[:, head]
    return product(out.reshape(T, H * dv), w["o"])


# --------------------------------------------------------------------------- feed-forwards
def dense(h, w: dict):
    return product(relu_squared(product(h, w["up"])), w["down"])


def choose(scores, top: int, groups: int, keep: int):
    """scores [T, experts] -> ids [T, top]: the largest scores among the experts of the ``keep`` groups whose two largest
    scores have the largest sums."""
    T, E = scores.shape
    per = E // groups
    marks = scores.view(T, groups, per).topk(min(2, per), dim=-1).values.sum(-1)
    kept = torch.zeros(T, groups, dtype=torch.bool).scatter(1, marks.topk(keep, dim=-1).indices, True)
    return scores.masked_fill(~kept.repeat_interleave(per, dim=1), float("-inf")).topk(top, dim=-1).indices


def routed(h, w: dict, router: dict):
    groups = router.get("groups") or {}
    scores = torch.sigmoid(h @ w["router"].T)
    ids = choose(scores, int(router["top"]), int(groups.get("count") or 1), int(groups.get("keep") or 1))
    out = torch.zeros_like(h)
    for e in range(int(router["experts"])):
        hit = (ids == e).any(dim=-1)
        if bool(hit.any()):
            y = product(relu_squared(product(h[hit], w[f"e{e}.up"])), w[f"e{e}.down"])
            out[hit] = out[hit] + scores[hit, e][:, None] * y
    return out


# --------------------------------------------------------------------------- the model
def under(W: dict, prefix: str) -> dict:
    return {k[len(prefix):]: t for k, t in W.items() if k.startswith(prefix)}


def mixer(layer: dict, h, w: dict, eps: float, positions):
    if layer["type"] == "attention":
        return attention(h, w, layer["mixer"], eps, positions)
    if layer["type"] == "latent_attention":
        return latent_attention(h, w, layer["mixer"], eps, positions)
    raise ValueError(layer["type"])


def feed_forward(mlp: dict, h, w: dict):
    return dense(h, w) if mlp["kind"] == "dense" else routed(h, w, mlp["router"])


def forward(cfg: dict, weights: dict, tokens, dtype=torch.float32, layer_outputs: list | None = None):
    """Logits [T, vocab] of one sequence from its first token on.  ``layer_outputs``: a list that receives the stream
    behind every layer."""
    with torch.no_grad():
        W = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in weights.items()}
        eps = float(cfg["norm"]["eps"])
        x, positions = embedding(tokens, W["embed"]), range(len(tokens))
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            x = x + layer_norm(mixer(layer, x, under(W, p + "mix."), eps, positions), W[p + "norm1"], W[p + "norm1.b"], eps)
            if layer.get("mlp"):
                x = x + layer_norm(feed_forward(layer["mlp"], x, under(W, p + "mlp.")), W[p + "norm2"], W[p + "norm2.b"], eps)
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        return product(layer_norm(x, W["final.norm"], W["final.norm.b"], eps), W["embed"]) * float(cfg.get("logit_scale", 1.0))
