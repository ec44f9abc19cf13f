"""Small Funepel configurations for the tests (config.json dictionaries)."""


def mamba2(heads, vdim, state, groups, conv=4, norm_groups=1):
    return "mamba2", {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": norm_groups}


def parallel(left, right):
    return "parallel", {"left": left, "right": right}


def att(heads, kv, dim, scale, size, coef=0.4, every=32):
    return {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": dim, "scale": scale, "mask": {"size": size},
            "q_temp": {"coef": coef, "every": every}}


def ret(heads, dim, vdim, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "decay": list(decay)}


def moe(experts, top, ff, shared, groups=None):
    r = {"experts": experts, "top": top}
    if groups:
        r["groups"] = {"count": groups[0], "keep": groups[1]}
    return {"kind": "moe", "expert": {"ff": ff}, "router": r, "shared": {"ff": shared}}


def layer(mixer, mlp=None):
    return {"type": mixer[0], "mixer": mixer[1], "mlp": mlp}


def config(layers, vocab, width, eps=1e-5, loop=None, side=0):
    c = {"architecture": "Funepel", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        c["token_side"] = {"dim": side}
    return c


_M = mamba2(6, 32, 64, 3, 4, 2)
_P = parallel(att(6, 3, 32, 0.2, 40), ret(5, 64, 48, (0.9, 0.97, 0.99, 0.998, 1.0)))
_E = moe(10, 3, 80, 56, (5, 2))

CASES = {
    # both mixers, a loop over both, experts in groups
    "plain": config([layer(_M, _E), layer(_P, _E), layer(_P, _E)], 160, 128, loop=(0, 2, 3), side=16),
    # every layer different: padded sizes everywhere, windows shorter and longer than a page, taps beyond four,
    # parts of the gated norm across heads, no feed-forward, one group of experts, eps that matters
    "mixed": config([layer(parallel(att(5, 1, 72, 0.11, 7, 0.7, 9), ret(2, 200, 20, (0.5, 0.995))), moe(7, 2, 24, 40)),
                     layer(mamba2(5, 24, 20, 1, 6, 4), moe(6, 5, 40, 72, (2, 2))),
                     layer(parallel(att(4, 4, 24, 0.3, 100, 0.3, 64), ret(3, 30, 70, (0.8, 0.0, 0.999)))),
                     layer(mamba2(4, 72, 130, 2, 2, 3), moe(12, 1, 72, 24, (3, 1)))], 331, 200, eps=3e-2,
                    loop=(1, 4, 2), side=10),
    # values that may hide a factor: one head, one group, one tap, one expert, a window of one key, a loop of one pass
    "ones": config([layer(mamba2(1, 32, 32, 1, 1, 1), moe(1, 1, 64, 64, (1, 1))),
                    layer(parallel(att(1, 1, 64, 1.0, 1, 1.0, 1), ret(1, 32, 64, (1.0,))), moe(4, 1, 64, 64, (4, 1)))],
                   97, 64, loop=(1, 2, 1), side=64),
    # no loop, no token input, wide heads, many query heads over one key head, many experts
    "wide": config([layer(parallel(att(40, 1, 32, 0.18, 300), ret(2, 128, 130, (0.97, 0.99))), moe(70, 6, 16, 200, (7, 3))),
                    layer(mamba2(3, 100, 256, 3, 3, 5), moe(4, 4, 96, 32))], 256, 96),
    # recurrent layers only, the loop reaches the last one
    "recurrent": config([layer(mamba2(8, 16, 16, 4, 4, 8), moe(8, 2, 32, 32, (2, 1)))] * 3, 128, 136, loop=(1, 3, 3), side=24),
}
