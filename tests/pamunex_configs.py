"""Small Pamunex configurations for the tests: sizes, layer orders and constants that differ from one another in every
field, and single-layer ones that show one mechanism alone."""

import copy


def blocks(heads=4, kv_heads=2, dim=24, vdim=40, size=21, rot_dims=16, base=1e4, scale=0.3):
    """The attention layer: normed queries and keys, blocks of ``size`` positions, a logit per head without a key."""
    return {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "mask": {"size": size}, "rot": {"base": base, "dims": rot_dims}, "scale": scale}


def latent(heads=3, dim=20, rot_dim=12, vdim=28, kv_rank=36, size=19, base=500.0, scale=0.25):
    """The latent attention layer: a sliding window of ``size`` positions, the same logit per head."""
    return {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "mask": {"size": size},
            "rot": {"base": base, "dims": rot_dim}, "scale": scale}


def dense(ff=136):
    return {"kind": "dense", "ff": ff}


def moe(experts=8, top=3, count=4, keep=2, ff=40):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}}}


def layer(kind, mixer, mlp=None):
    return {"type": kind, "mixer": mixer, "mlp": mlp}


def model(width, vocab, layers, eps=1e-5, logit_scale=1.5):
    return {"architecture": "Pamunex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale, "layers": copy.deepcopy(layers)}


# Both mixers, each with both kinds of feed-forward and with none; key and value sizes that differ either way, windows and
# blocks that are no multiples of a page; sizes that fit no tile.
PAMU_A = model(96, 300, [layer("attention", blocks(), dense(72)),
                         layer("latent_attention", latent(), moe()),
                         layer("attention", blocks(heads=6, kv_heads=1, dim=32, vdim=16, size=50, rot_dims=32, base=77.0, scale=0.2), None),
                         layer("latent_attention", latent(heads=5, dim=16, rot_dim=32, vdim=16, kv_rank=64, size=45, base=3e5, scale=0.3), dense()),
                         layer("attention", blocks(heads=3, kv_heads=3, dim=48, vdim=48, size=33, rot_dims=8, scale=0.15), moe(experts=9, top=2, count=3, keep=1, ff=24)),
                         layer("latent_attention", latent(size=7), None)])

# A width that is no multiple of 4; one head, one expert of one, groups of one expert, every group kept; a block and a window of
# exactly one page; head sizes and rotated parts that no vector load fits; a latent wider than the paged attention kernels take.
PAMU_B = model(50, 77, [layer("latent_attention", latent(heads=1, dim=10, rot_dim=6, vdim=9, kv_rank=270, size=16, base=33.0, scale=0.5), moe(1, 1, 1, 1, 33)),
                        layer("attention", blocks(heads=1, kv_heads=1, dim=10, vdim=6, size=16, rot_dims=6, base=33.0, scale=0.5), moe(4, 4, 4, 4, 10)),
                        layer("attention", blocks(heads=5, kv_heads=1, dim=7, vdim=11, size=37, rot_dims=2, base=7.0, scale=0.4), moe(6, 1, 6, 2, 31))],
               eps=1e-3, logit_scale=0.7)

# Blocks and a window of one position (a query sees itself and the logit without a key); heads beyond 64 and 128 elements; layers of
# one kind twice in a row; more of the widths the tiles like; a scale of the logits of one.
PAMU_C = model(128, 131, [layer("latent_attention", latent(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, size=1, scale=0.2), dense(256)),
                          layer("latent_attention", latent(heads=8, dim=16, rot_dim=16, vdim=24, kv_rank=112, size=70, base=1e4, scale=0.2), moe(16, 4, 4, 2, 64)),
                          layer("attention", blocks(heads=2, kv_heads=1, dim=80, vdim=144, size=1, rot_dims=40, base=100.0, scale=0.11), dense(64)),
                          layer("attention", blocks(heads=2, kv_heads=2, dim=160, vdim=32, size=64, rot_dims=64, scale=0.09), moe(16, 6, 2, 1, 64))],
               eps=1e-6, logit_scale=1.0)

# One mechanism each, over a width of 64.
ALONE = {
    "blocks": model(64, 120, [layer("attention", blocks(heads=4, kv_heads=2, dim=16, vdim=16, size=9))]),
    "blocks_wide_values": model(64, 120, [layer("attention", blocks(heads=2, kv_heads=1, dim=8, vdim=40, size=30, rot_dims=4))]),
    "latent": model(64, 120, [layer("latent_attention", latent(heads=4, dim=16, rot_dim=8, vdim=16, kv_rank=32, size=9, base=50.0))]),
    "latent_wide": model(64, 120, [layer("latent_attention", latent(heads=2, dim=16, rot_dim=8, vdim=16, kv_rank=300, size=30, base=50.0))]),
    "dense": model(64, 120, [layer("attention", blocks(heads=1, kv_heads=1, dim=8, vdim=8, size=4, rot_dims=2), dense(96))]),
    "moe": model(64, 120, [layer("attention", blocks(heads=1, kv_heads=1, dim=8, vdim=8, size=4, rot_dims=2), moe(12, 3, 4, 2, 56))]),
}
