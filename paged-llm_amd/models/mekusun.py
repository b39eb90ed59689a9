"""Mekusun: a decoder with RMS norms in front of and behind every sublayer over a residual stream kept in float,
x <- x + s1 * N1b(mixer(N1(x))), x <- x + s2 * N2b(ff(N2(x))), where a norm's factor is stored around zero and s1, s2 are
stored vectors (the scale of what a sublayer adds).  Behind every layer the stream becomes a weighted sum over the depth: of
the embedding's output and the results of all layers up to this one.  The embedding is scaled, the logits are capped by
c tanh(z / c).

* ``mamba1``: a selective scan (a state per channel, decays per channel and state element) behind a short convolution.
* ``latent_attention``: keys and values expanded from one cached normed latent per token, one rotated key part that all heads
  share (pairs (i, i + r/2)), full causal mask.
* ``general_delta``: a matrix memory with decays per row and a removal of what the unit key reads.

Feed-forwards: dense without a gate and with a learned activation (xIELU), or routed experts without a gate (GELU), chosen by
the router's outputs with their bias and weighed by the softmax over the chosen ones.

``config.json``: ``architecture`` "Mekusun", ``vocab``, ``width``, ``norm.eps``, ``embedding.scale``, ``logit_softcap``, and
``layers``, a list of {``type``, ``mixer`` (the mixer's sizes and constants), ``mlp`` ({``kind``: "dense", ``ff``}, {``kind``: "moe",
``expert``: {``ff``}, ``router``: {``experts``, ``top``}} or null)}.  Layer i's tensors are ``l<i>.norm1``, ``l<i>.norm1b``, ``l<i>.ls1``,
``l<i>.mix.*``, ``l<i>.norm2``, ``l<i>.norm2b``, ``l<i>.ls2``, ``l<i>.mlp.*`` and ``l<i>.dwa`` (the weights of the sum over the
depth); outside the layers ``embed``, ``final.norm`` and ``head``.  Importing this module registers the architecture."""

from __future__ import annotations

from dataclasses import dataclass, field

from ..config.registry import Architecture, register_architecture
from ..parts.spec import LayerSpec, ModelSpec, PartSpec, ScheduleStep, StreamOpSpec

MIXER_TYPES = ("mamba1", "latent_attention", "general_delta")
MLP_KINDS = ("dense", "moe")


@dataclass
class MekusunLayer:
    type: str
    mixer: dict
    mlp: dict | None


@dataclass
class MekusunConfig:
    vocab: int
    width: int
    norm_eps: float
    embedding_scale: float = 1.0
    logit_softcap: float = 0.0               # 0: none
    layers: list = field(default_factory=list)
    max_positions: int = 4096
    torch_dtype: str = "bfloat16"

    @classmethod
    def from_json(cls, cfg: dict) -> "MekusunConfig":
        layers = [MekusunLayer(str(l["type"]), dict(l["mixer"]), (dict(l["mlp"]) if l.get("mlp") is not None else None)) for l in cfg["layers"]]
        out = cls(vocab=int(cfg["vocab"]), width=int(cfg["width"]), norm_eps=float(cfg["norm"]["eps"]),
                  embedding_scale=float((cfg.get("embedding") or {}).get("scale") or 1.0), logit_softcap=float(cfg.get("logit_softcap") or 0.0),
                  layers=layers, max_positions=int(cfg.get("max_positions", 4096)), torch_dtype=str(cfg.get("torch_dtype") or "bfloat16"))
        out.validate()
        return out

    def validate(self) -> None:
        problems = []
        if self.vocab <= 0 or self.width <= 0 or not self.layers:
            problems.append("vocab, width and the number of layers must be positive")
        if self.logit_softcap < 0.0:
            problems.append("logit_softcap is positive, or 0 for none")
        for i, l in enumerate(self.layers):
            if l.type not in MIXER_TYPES:
                problems.append(f"layer {i}: mixer type {l.type!r} is none of {MIXER_TYPES}")
            if l.mlp is not None and l.mlp.get("kind") not in MLP_KINDS:
                problems.append(f"layer {i}: feed-forward kind {l.mlp.get('kind')!r} is none of {MLP_KINDS}")
            if l.type == "latent_attention" and int((l.mixer.get("rot") or {}).get("dims") or 0) != int(l.mixer.get("rot_dim") or 0):
                problems.append(f"layer {i}: the rotated part of a latent attention layer turns as a whole (rot.dims = rot_dim)")
        if problems:
            raise ValueError("bad Mekusun config: " + "; ".join(problems))


def _mixer_spec(kind: str, m: dict, eps: float) -> PartSpec:
    if kind == "mamba1":
        return PartSpec("mamba1", {"inner": int(m["inner"]), "state": int(m["state"]), "dt_rank": int(m["dt_rank"]), "conv": int(m["conv"])})
    if kind == "general_delta":
        return PartSpec("general_delta", {"heads": int(m["heads"]), "dim": int(m["dim"]), "eps": eps, "decay_rank": m.get("decay_rank")})
    rot = int(m.get("rot_dim") or 0)
    position = {"kind": "rotary", "params": {"head_dim": rot, "theta": float(m["rot"]["base"]), "rotary_dim": rot, "interleaved": False,
                                             "scaling": None, "exact_frequencies": True}} if rot else None
    return PartSpec("latent_attention", {"heads": int(m["heads"]), "plain_dim": int(m["dim"]), "rot_dim": rot, "head_dim": int(m["vdim"]),
                                         "rank": int(m["kv_rank"]), "scale": float(m["scale"]), "window": 0, "position": position, "eps": eps})


def _mlp_spec(mlp: dict) -> PartSpec:
    if mlp["kind"] == "dense":
        return PartSpec("plain_mlp", {"intermediate_size": int(mlp["ff"]), "activation": "xielu",
                                      "tensor_names": {"up": "up", "down": "down", "act": "act"}})
    r = mlp["router"]
    return PartSpec("routed_experts", {"experts": int(r["experts"]), "top": int(r["top"]), "intermediate_size": int(mlp["expert"]["ff"]),
                                       "gated": False, "activation": "gelu", "correction": False, "scoring": "softmax_chosen",
                                       "router_bias": "router.b"})


def build_spec(cfg: MekusunConfig) -> ModelSpec:
    eps = cfg.norm_eps

    def norm(scale: str | None = None) -> PartSpec:
        return PartSpec("rmsnorm", {"eps": eps, "weight_name": "", "unit_offset": True, **({"scale_name": "/" + scale} if scale else {})})

    layers, schedule, stream_ops, unused = [], [], [], []
    for i, l in enumerate(cfg.layers):
        parts = {"mixer_norm": norm(), "mixer": _mixer_spec(l.type, l.mixer, eps), "mixer_out_norm": norm("ls1")}
        names = {"mixer_norm": "norm1", "mixer": "mix", "mixer_out_norm": "norm1b", "feed_forward": l.mlp is not None}
        if l.mlp is not None:
            parts.update({"feed_forward_norm": norm(), "feed_forward": _mlp_spec(l.mlp), "feed_forward_out_norm": norm("ls2")})
            names.update({"feed_forward_norm": "norm2", "feed_forward": "mlp", "feed_forward_out_norm": "norm2b"})
        else:
            unused += [f"l{i}.{n}" for n in ("norm2", "norm2b", "ls2")]           # (a checkpoint may carry them; nothing reads them)
        layers.append(LayerSpec(f"l{i}", PartSpec("sandwich_norm", names), parts))
        stream_ops.append(StreamOpSpec(f"l{i}.dwa", PartSpec("depth_average", {"results": i + 2, "tensor_name": ""})))
        schedule.append(ScheduleStep(i, exit=i))
    return ModelSpec(
        hidden_size=cfg.width, vocab_size=cfg.vocab,
        embedding=PartSpec("token_embedding", {"vocab_size": cfg.vocab, "scale": cfg.embedding_scale, "float_stream": True, "tensor_name": ""}),
        layers=layers, final_norm=norm(), head=PartSpec("lm_head", {"vocab_size": cfg.vocab, "tied": False, "tensor_name": "", "cap": cfg.logit_softcap}),
        schedule=schedule, stream_ops=stream_ops, embedding_name="embed", final_norm_name="final.norm", head_name="head",
        ignored_suffixes=tuple(unused), max_positions=cfg.max_positions, eos_token_id=None, stored_dtype=cfg.torch_dtype)


register_architecture(Architecture("Mekusun", MekusunConfig.from_json, build_spec))
