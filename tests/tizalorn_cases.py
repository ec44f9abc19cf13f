"""Small Tizalorn configurations for the tests (config.json dictionaries)."""


def wkv(heads, dim):
    return "wkv", {"heads": heads, "dim": dim}


def latent(heads, dim, rot, vdim, kv_rank, q_rank, scale, base=700.0, scaling=(4.0, 60, 6.0, 0.5)):
    """``scaling``: (factor, original, fast, slow) or None."""
    r = {"base": base, "dims": rot}
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return "latent_attention", {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv_rank,
                                "q_rank": q_rank, "scale": scale, "rot": r}


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, limit, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff, "limit": limit}, "router": r}


def layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def config(layers, vocab, width, bigram=(211, 31, 7), eps=1e-5):
    """``bigram``: (buckets, multiplier of the previous token, of the current one)."""
    return {"architecture": "Tizalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers,
            "embedding": {"bigram": dict(zip(("buckets", "mul_prev", "mul_cur"), bigram))}}


_E = moe(15, 3, 80, 0.9, (5, 2))
_A = latent(4, 24, 20, 40, 72, 56, 0.35)

CASES = {
    # every mixer and feed-forward, experts in groups, frequencies on both sides of the ramp
    "plain": config([layer(wkv(3, 32), dense(200)), layer(_A, _E), layer(wkv(2, 64), _E)], 160, 128),
    # every layer different: padded sizes everywhere, no feed-forward, attention first, an eps that matters
    "mixed": config([layer(latent(5, 40, 6, 72, 130, 100, 0.11, 50.0, (2.0, 30, 3.0, 0.2)), moe(7, 2, 24, 2.0)),
                     layer(wkv(3, 72), dense(90)), layer(wkv(5, 20)), layer(latent(3, 10, 66, 17, 33, 200, 0.3, 9000.0, None)),
                     layer(wkv(1, 130), moe(12, 5, 72, 0.5, (2, 2)))], 331, 200, (1009, 1013, 5), 3e-2),
    # values that may hide a factor: one head, one expert, one group, one row for all pairs, no ramp
    "ones": config([layer(wkv(1, 64), moe(1, 1, 64, 1.0, (1, 1))),
                    layer(latent(1, 64, 2, 64, 64, 64, 1.0, 10.0, (1.0, 1, 1.0, 1.0)), moe(4, 1, 64, 1.0, (2, 1)))], 97, 64,
                   (1, 1, 1)),
    # more heads than a workgroup's rows, wide latents and states, many experts
    "wide": config([layer(wkv(2, 200), moe(70, 6, 16, 1.5, (7, 3))),
                    layer(latent(70, 16, 128, 8, 300, 40, 0.1, 300.0, (8.0, 500, 20.0, 1.0)), moe(4, 4, 96, 3.0))], 256, 96,
                   (40, 3, 40)),
    # one kind of mixer only
    "recurrent": config([layer(wkv(4, 16), moe(8, 2, 32, 1.2, (2, 1)))] * 3, 128, 136, (500, 0, 1)),
    "latent": config([layer(latent(8, 32, 16, 32, 96, 64, 0.2), dense(64 * k)) for k in (1, 3)], 120, 72, (333, 120, 1)),
}
