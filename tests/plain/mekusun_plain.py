"""A plain, slow Mekusun: whole sequences, no cache, no paging, no batches, one function per mechanism.

Mekusun keeps a scaled token embedding as its residual stream and norms on both sides of every sublayer,
x <- x + s1 * N1b(mixer(N1(x))), x <- x + s2 * N2b(ff(N2(x))), with RMS norms whose factor is 1 + w and an element-wise
scale s on what a sublayer adds.  Behind every layer the stream becomes a weighted sum over the embedding's output and
the results of all layers up to this one, each result taken before that sum.  A layer holds one of three mixers:

* ``mamba1``: a vector of states per channel, s_c <- e^(dt_c A_c) * s_c + (dt_c x_c) B, behind a short convolution.
* ``latent_attention``: keys and values from one normed latent per token, one rotated key part for all heads.
* ``general_delta``: per head a matrix memory whose rows decay one by one and from which a part of what the unit key
  reads (z = S^T u) is removed along another direction, S <- w . S - (a . u) z^T + k v^T, row by row.

and a dense feed-forward with a learned activation, or routed ungated experts.  The logits are capped by a tanh.
Everything is computed in one floating type chosen by the caller.  It shares no code with the engine under
``paged-llm_amd/``.
"""

from __future__ import annotations

import json
import math
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


def layer_norm_around_zero(x, w, eps):
    return unit_rms(x, eps) * (1.0 + w)


def silu(z):
    return z * torch.sigmoid(z)


def softplus(z):
    return torch.clamp(z, min=0) + torch.log1p(torch.exp(-z.abs()))


def gelu_erf(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def xielu(z, p, q):
    """softplus(p) z^2 + z/2 above zero; (1/2 + softplus(q)) (e^z - 1 - z) + z/2 below."""
    up = softplus(p) * z * z + 0.5 * z
    low = torch.clamp(z, max=0)
    down = (0.5 + softplus(q)) * (torch.expm1(low) - low) + 0.5 * low
    return torch.where(z > 0, up, down)


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
    far the logits of one position move under the compute type's rounding alone; norms, scores, the router, the recurrences'
    gates and states and the residual stream stay exact, as the design keeps them in 32 bits."""

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


def embedding(tokens, table, scale: float):
    return table[torch.tensor(list(tokens))] * scale


def rotate_halves(x, positions, dims: int, base: float):
    """x [T, heads, r]: pairs (i, i + dims/2) of the first ``dims`` elements turned by position * base^(-2i/dims)."""
    half = dims // 2
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(half)], dtype=torch.float64)
    ang = torch.tensor(list(positions), dtype=torch.float64)[:, None] * f[None, :]
    cos, sin = torch.cos(ang).to(x.dtype)[:, None, :], torch.sin(ang).to(x.dtype)[:, None, :]
    u, v = x[..., :half], x[..., half:dims]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, x[..., dims:]], dim=-1)


# --------------------------------------------------------------------------- mixers
def causal_convolution(x, w, b):
    """x [T, C], w [C, taps] (the last column meets the current token), zeros in front of the sequence."""
    taps = w.shape[1]
    padded = torch.cat([torch.zeros(taps - 1, x.shape[1], dtype=x.dtype), x])
    out = b.expand(x.shape[0], -1).clone()
    for j in range(taps):
        out = out + padded[j:j + x.shape[0]] * w[:, j]
    return out


def selective_scan(x, dt, A, B, C, D):
    """x, dt [T, channels], A [channels, state], B, C [T, state]: token by token, a state per channel."""
    S = torch.zeros_like(A)
    out = []
    for t in range(x.shape[0]):
        S = torch.exp(dt[t][:, None] * A) * S + (dt[t] * x[t])[:, None] * B[t][None, :]
        out.append(S @ C[t] + D * x[t])
    return torch.stack(out)


def mamba1(h, w: dict, m: dict):
    inner, n, rank = int(m["inner"]), int(m["state"]), int(m["dt_rank"])
    rows = product(h, w["in"])
    x, z = rows[:, :inner], rows[:, inner:]
    x = silu(causal_convolution(x, w["conv"], w["conv.b"]))
    low = product(x, w["x"])
    dt = softplus(product(low[:, :rank], w["dt"]) + w["dt.b"])
    y = selective_scan(x, dt, -torch.exp(w["A_log"]), low[:, rank:rank + n], low[:, rank + n:], w["D"])
    return product(y * silu(z), w["o"])


def latent_attention(h, w: dict, m: dict, eps: float, positions):
    T = h.shape[0]
    H, d, r, dv, rank = int(m["heads"]), int(m["dim"]), int(m["rot_dim"]), int(m["vdim"]), int(m["kv_rank"])
    q = product(h, w["q"]).view(T, H, d + r)
    down = product(h, w["dkv"])
    c = unit_rms(down[:, :rank], eps) * w["dkv.norm"]
    kr = rotate_halves(down[:, None, rank:], positions, r, float(m["rot"]["base"]))[:, 0]
    qr = rotate_halves(q[..., d:], positions, r, float(m["rot"]["base"]))
    k, v = product(c, w["uk"]).view(T, H, d), product(c, w["uv"]).view(T, H, dv)
    hidden = torch.ones(T, T, dtype=torch.bool).triu(1)
    out = torch.zeros(T, H, dv, dtype=h.dtype)
    for head in range(H):
        s = (q[:, head, :d] @ k[:, head].T + qr[:, head] @ kr.T) * float(m["scale"])
        out[:, head] = torch.softmax(s.masked_fill(hidden, float("-inf")), dim=-1) @ v[:, head]
    return product(out.reshape(T, H * dv), w["o"])


def delta_memory(r, k, v, w, a):
    """r, k, v, w, a [T, heads, d]: z = S^T u with u the unit key, S <- w . S - (a . u) z^T + k v^T (w . S row by row);
    o = S^T r."""
    u = k / torch.sqrt((k * k).sum(-1, keepdim=True) + 1e-6)
    T, H, d = k.shape
    S = torch.zeros(H, d, v.shape[-1], dtype=k.dtype)
    out = []
    for t in range(T):
        read = torch.einsum("hn,hnp->hp", u[t], S)
        S = w[t][..., None] * S - (a[t] * u[t])[..., None] * read[:, None, :] + k[t][..., None] * v[t][:, None, :]
        out.append(torch.einsum("hnp,hn->hp", S, r[t]))
    return torch.stack(out)


def general_delta(h, w: dict, m: dict, eps: float):
    T, H, d = h.shape[0], int(m["heads"]), int(m["dim"])
    r, k, v = (product(h, w[n]).view(T, H, d) for n in ("r", "k", "v"))
    gate = product(torch.tanh(product(h, w["w1"])), w["w2"]) + w["w0"]
    decay = torch.exp(-math.exp(-0.5) * torch.sigmoid(gate)).view(T, H, d)
    a = torch.sigmoid(product(h, w["a"]) + w["a.b"]).view(T, H, d)
    o = unit_rms(delta_memory(r, k, v, decay, a), eps).reshape(T, H * d)
    return product(o * w["norm"] * torch.sigmoid(product(h, w["g"])), w["o"])


# --------------------------------------------------------------------------- feed-forwards
def dense(h, w: dict):
    return product(xielu(product(h, w["up"]), w["act"][0], w["act"][1]), w["down"])


def routed(h, w: dict, experts: int, top: int):
    z = h @ w["router"].T + w["router.b"]
    best, ids = torch.topk(z, top, dim=-1)
    share = torch.softmax(best, dim=-1)
    out = torch.zeros_like(h)
    for e in range(experts):
        for slot in range(top):
            hit = ids[:, slot] == e
            if bool(hit.any()):
                y = product(gelu_erf(product(h[hit], w[f"e{e}.up"])), w[f"e{e}.down"])
                out[hit] = out[hit] + share[hit, slot][:, None] * y
    return out


# --------------------------------------------------------------------------- the model
def under(W: dict, prefix: str) -> dict:
    return {k[len(prefix):]: t for k, t in W.items() if k.startswith(prefix)}


def depth_average(results: list, weights):
    out = weights[0] * results[0]
    for j in range(1, len(results)):
        out = out + weights[j] * results[j]
    return out


def cap_logits(z, cap: float):
    return cap * torch.tanh(z / cap) if cap else z


def mixer(layer: dict, h, w: dict, eps: float, positions):
    if layer["type"] == "mamba1":
        return mamba1(h, w, layer["mixer"])
    if layer["type"] == "latent_attention":
        return latent_attention(h, w, layer["mixer"], eps, positions)
    if layer["type"] == "general_delta":
        return general_delta(h, w, layer["mixer"], eps)
    raise ValueError(layer["type"])


def feed_forward(mlp: dict, h, w: dict):
    if mlp["kind"] == "dense":
        return dense(h, w)
    return routed(h, w, int(mlp["router"]["experts"]), int(mlp["router"]["top"]))


def forward(cfg: dict, weights: dict, tokens, dtype=torch.float32, layer_outputs: list | None = None):
    """Logits [T, vocab] of one sequence from its first token on.  ``layer_outputs``: a list that receives the stream
    behind every layer, its sum over the depth done."""
    with torch.no_grad():
        W = {k: (t.to(dtype) if t.is_floating_point() else t) for k, t in weights.items()}
        eps = float(cfg["norm"]["eps"])
        x = embedding(tokens, W["embed"], float((cfg.get("embedding") or {}).get("scale") or 1.0))
        results, positions = [x], range(len(tokens))
        for i, layer in enumerate(cfg["layers"]):
            p = f"l{i}."
            y = mixer(layer, layer_norm_around_zero(x, W[p + "norm1"], eps), under(W, p + "mix."), eps, positions)
            x = x + W[p + "ls1"] * layer_norm_around_zero(y, W[p + "norm1b"], eps)
            if layer.get("mlp"):
                y = feed_forward(layer["mlp"], layer_norm_around_zero(x, W[p + "norm2"], eps), under(W, p + "mlp."))
                x = x + W[p + "ls2"] * layer_norm_around_zero(y, W[p + "norm2b"], eps)
            results.append(x)
            x = depth_average(results, W[p + "dwa"])
            if layer_outputs is not None:
                layer_outputs.append(x.clone())
        logits = product(layer_norm_around_zero(x, W["final.norm"], eps), W["head"])
        return cap_logits(logits, float(cfg.get("logit_softcap") or 0.0))
