"""Pamunex: a decoder whose sublayers read the residual stream itself and whose layer norms (weight and bias) stand on what
the sublayers return, x <- x + LN1(mixer(x)), x <- x + LN2(ff(x)); the stream is kept in float and the logits come from the
embedding table, times a constant.  A layer holds one of two mixers and a dense feed-forward, routed experts or no feed-forward.

* ``attention``: grouped heads whose keys and values may differ in width, biases on q, k and v (none on the output), queries and
  keys divided by their root mean square per head and times a weight that the heads share, then turned (pairs (i, i + r/2) of
  the first r elements); keys visible inside the query's own block of ``mask.size`` positions; a learned logit per head in the
  softmax's denominator.
* ``latent_attention``: keys and values expanded from one cached normed latent per token, one rotated key part that all heads
  share (pairs (i, i + r/2)), a sliding window of ``mask.size`` positions, the same logit per head.

Feed-forwards have no gate and no biases, down(relu(up h)^2).  Routed experts: sigmoid scores, a group of neighbours marked by the
sum of its two largest scores, the chosen experts weighed by their scores as they are.

``config.json``: ``architecture`` "Pamunex", ``vocab``, ``width``, ``norm.eps``, ``logit_scale`` and ``layers``, a list of {``type``,
``mixer`` (the mixer's sizes and constants), ``mlp`` ({``kind``: "dense", ``ff``}, {``kind``: "moe", ``expert``: {``ff``}, ``router``:
{``experts``, ``top``, ``groups``: {``count``, ``keep``}}} or null)}.  Layer i's tensors are ``l<i>.norm1[.b]``, ``l<i>.mix.*``,
``l<i>.norm2[.b]``, ``l<i>.mlp.*``; outside the layers ``embed`` and ``final.norm[.b]``.  Importing this module registers the
architecture."""

from __future__ import annotations

from dataclasses import dataclass, field

from ..config.registry import Architecture, register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec

MIXER_TYPES = ("attention", "latent_attention")
MLP_KINDS = ("dense", "moe")


@dataclass
class PamunexLayer:
    type: str
    mixer: dict
    mlp: dict | None


@dataclass
class PamunexConfig:
    vocab: int
    width: int
    norm_eps: float
    logit_scale: float = 1.0
    layers: list = field(default_factory=list)
    max_positions: int = 4096
    torch_dtype: str = "bfloat16"

    @classmethod
    def from_json(cls, cfg: dict) -> "PamunexConfig":
        layers = [PamunexLayer(str(l["type"]), dict(l["mixer"]), (dict(l["mlp"]) if l.get("mlp") is not None else None)) for l in cfg["layers"]]
        scale = cfg.get("logit_scale")
        out = cls(vocab=int(cfg["vocab"]), width=int(cfg["width"]), norm_eps=float(cfg["norm"]["eps"]), logit_scale=1.0 if scale is None else float(scale),
                  layers=layers, max_positions=int(cfg.get("max_positions", 4096)), torch_dtype=str(cfg.get("torch_dtype") or "bfloat16"))
        out.validate()
        return out

    def validate(self) -> None:
        problems = []
        if self.vocab <= 0 or self.width <= 0 or not self.layers:
            problems.append("vocab, width and the number of layers must be positive")
        for i, l in enumerate(self.layers):
            if l.type not in MIXER_TYPES:
                problems.append(f"layer {i}: mixer type {l.type!r} is none of {MIXER_TYPES}")
            if l.mlp is not None and l.mlp.get("kind") not in MLP_KINDS:
                problems.append(f"layer {i}: feed-forward kind {l.mlp.get('kind')!r} is none of {MLP_KINDS}")
            if l.type == "latent_attention" and int((l.mixer.get("rot") or {}).get("dims") or 0) != int(l.mixer.get("rot_dim") or 0):
                problems.append(f"layer {i}: the rotated part of a latent attention layer turns as a whole (rot.dims = rot_dim)")
        if problems:
            raise ValueError("bad Pamunex config: " + "; ".join(problems))


def _rotary(rot: dict | None, head_dim: int) -> dict | None:
    dims = int((rot or {}).get("dims") or 0)
    if dims <= 0:
        return None
    return {"kind": "rotary", "params": {"head_dim": head_dim, "theta": float(rot["base"]), "rotary_dim": dims, "interleaved": False,
                                         "scaling": None, "exact_frequencies": True}}


def _mixer_spec(kind: str, m: dict, eps: float) -> PartSpec:
    size = int((m.get("mask") or {}).get("size") or 0)
    if kind == "attention":
        return PartSpec("normed_attention", {
            "heads": int(m["heads"]), "kv_heads": int(m["kv_heads"]), "key_dim": int(m["dim"]), "value_dim": int(m["vdim"]),
            "scale": float(m["scale"]), "eps": eps, "norm_weights": True, "norm_first": True, "position": _rotary(m.get("rot"), int(m["dim"])),
            "mask": "chunk" if size > 0 else "full", "mask_size": size, "bias": True, "output_bias": False, "sinks": True})
    rot = int(m.get("rot_dim") or 0)
    return PartSpec("latent_attention", {"heads": int(m["heads"]), "plain_dim": int(m["dim"]), "rot_dim": rot, "head_dim": int(m["vdim"]),
                                         "rank": int(m["kv_rank"]), "scale": float(m["scale"]), "window": size,
                                         "position": _rotary(m.get("rot"), rot), "eps": eps, "sinks": True})


def _mlp_spec(mlp: dict) -> PartSpec:
    if mlp["kind"] == "dense":
        return PartSpec("plain_mlp", {"intermediate_size": int(mlp["ff"]), "activation": "relu2", "tensor_names": {"up": "up", "down": "down"}})
    r = mlp["router"]
    groups = r.get("groups") or {}
    return PartSpec("routed_experts", {"experts": int(r["experts"]), "top": int(r["top"]), "intermediate_size": int(mlp["expert"]["ff"]),
                                       "groups": int(groups.get("count") or 1), "keep": int(groups.get("keep") or 1), "group_mark": "two_largest",
                                       "gated": False, "activation": "relu2", "correction": False, "scoring": "sigmoid"})


def build_spec(cfg: PamunexConfig) -> ModelSpec:
    eps = cfg.norm_eps
    norm = PartSpec("layernorm", {"eps": eps, "weight_name": "", "bias_name": "b"})
    layers = []
    for i, l in enumerate(cfg.layers):
        parts = {"mixer": _mixer_spec(l.type, l.mixer, eps), "mixer_norm": norm}
        names = {"mixer": "mix", "mixer_norm": "norm1", "feed_forward": l.mlp is not None}
        if l.mlp is not None:
            parts.update({"feed_forward": _mlp_spec(l.mlp), "feed_forward_norm": norm})
            names.update({"feed_forward": "mlp", "feed_forward_norm": "norm2"})
        layers.append(LayerSpec(f"l{i}", PartSpec("branch_norm", names), parts))
    # the logits are linear in the last norm's rows: their scale is a factor of that norm's weight and bias
    last = PartSpec("layernorm", {**norm.params, "factor": cfg.logit_scale})
    return ModelSpec(
        hidden_size=cfg.width, vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "float_stream": True, "tensor_name": ""}),
        layers=layers, final_norm=last, head=PartSpec("lm_head", {"vocab_size": cfg.vocab, "tied": True}),
        embedding_name="embed", final_norm_name="final.norm", head_name="head",
        ignored_suffixes=tuple(f"l{i}.norm2{b}" for i, l in enumerate(cfg.layers) if l.mlp is None for b in ("", ".b")),
        max_positions=cfg.max_positions, eos_token_id=None, stored_dtype=cfg.torch_dtype)


register_architecture(Architecture("Pamunex", PamunexConfig.from_json, build_spec))
