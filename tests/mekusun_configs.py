"""Small Mekusun configurations for the tests: sizes, layer orders and constants that differ from one another in every
field, and single-layer ones that show one mechanism alone."""

import copy


def mamba1(inner=72, state=12, dt_rank=5, conv=4):
    return {"inner": inner, "state": state, "dt_rank": dt_rank, "conv": conv}


def latent(heads=3, dim=20, rot_dim=12, vdim=28, kv_rank=36, base=1e4, scale=0.25):
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot_dim}, "scale": scale}


def delta(heads=3, dim=20, decay_rank=7):
    """``decay_rank`` is for the random weights: a checkpoint's tensors decide it."""
    return {"heads": heads, "dim": dim, "decay_rank": decay_rank}


def dense(ff=136):
    return {"kind": "dense", "ff": ff}


def moe(experts=5, top=2, ff=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top}}


def layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model(width, vocab, layers, eps=1e-5, scale=3.0, softcap=20.0):
    return {"architecture": "Mekusun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "logit_softcap": softcap, "layers": copy.deepcopy(layers)}


# All three mixers and all kinds of feed-forward, none among them; sizes that fit no tile.
MEKU_A = model(96, 300, [layer("mamba1", mamba1(), moe()),
                         layer("latent_attention", latent(), dense(72)),
                         layer("general_delta", delta(), None),
                         layer("mamba1", mamba1(inner=200, state=16, dt_rank=8, conv=2), dense()),
                         layer("general_delta", delta(heads=2, dim=32, decay_rank=16), moe(experts=9, top=3, ff=24)),
                         layer("latent_attention", latent(heads=5, dim=16, rot_dim=32, vdim=16, kv_rank=64, base=77.0, scale=0.3), None)])

# Another order; a width that is no multiple of 4; one state element, one head, one tap, one expert of one; states of more than
# 32 and heads of more than 64 elements; a latent wider than the paged attention kernels take; other constants.
MEKU_B = model(50, 77, [layer("general_delta", delta(heads=1, dim=70, decay_rank=3), moe(experts=1, top=1, ff=33)),
                        layer("latent_attention", latent(heads=2, dim=10, rot_dim=6, vdim=9, kv_rank=270, base=33.0, scale=0.5), moe(experts=4, top=4, ff=10)),
                        layer("mamba1", mamba1(inner=33, state=1, dt_rank=1, conv=1), None),
                        layer("mamba1", mamba1(inner=130, state=70, dt_rank=19, conv=7), dense(31))], eps=1e-3, scale=1.0, softcap=7.5)

# Layers of one kind twice in a row, a latent layer first, more of the widths the tiles like.
MEKU_C = model(128, 131, [layer("latent_attention", latent(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, base=5e5, scale=0.2), dense(256)),
                          layer("latent_attention", latent(heads=8, dim=16, rot_dim=16, vdim=24, kv_rank=112, base=1e4, scale=0.2), moe(experts=16, top=4, ff=64)),
                          layer("general_delta", delta(heads=2, dim=64, decay_rank=32), dense(128)),
                          layer("mamba1", mamba1(inner=256, state=32, dt_rank=16), moe(experts=16, top=1, ff=64))], eps=1e-6, scale=11.0, softcap=30.0)

# One mechanism each, over a width of 64.
ALONE = {
    "mamba1": model(64, 120, [layer("mamba1", mamba1(inner=96, state=16, dt_rank=4))]),
    "latent": model(64, 120, [layer("latent_attention", latent(heads=4, dim=16, rot_dim=8, vdim=16, kv_rank=32, base=50.0))]),
    "delta": model(64, 120, [layer("general_delta", delta(heads=2, dim=32))]),
    "dense": model(64, 120, [layer("mamba1", mamba1(inner=8, state=4, dt_rank=2), dense(96))]),
    "moe": model(64, 120, [layer("mamba1", mamba1(inner=8, state=4, dt_rank=2), moe(experts=6, top=2, ff=48))]),
    "depth": model(64, 120, [layer("mamba1", mamba1(inner=8, state=4, dt_rank=2), dense(16)) for _ in range(6)]),
}
