"""Small Kozusun configurations for the tests (config.json dictionaries)."""


def att(heads, kv, dim, vdim, scale, size=None, keep=0):
    m = {"heads": heads, "kv_heads": kv, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        m["mask"] = {"size": size, "keep_first": keep}
    return m


def layer(mixer, ff=None):
    return {"type": "attention", "mixer": mixer, "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def config(layers, vocab, width, embed=3.0, mult=0.6, eps=1e-5, loop=None, side=0):
    c = {"architecture": "Kozusun", "vocab": vocab, "width": width, "embedding": {"scale": embed},
         "norm": {"eps": eps}, "residual_mult": mult, "layers": layers}
    if loop:
        c["loop"] = dict(zip(("start", "stop", "times"), loop))
    if side:
        c["token_side"] = {"dim": side}
    return c


CASES = {
    # every layer alike, loop in the middle
    "plain": config([layer(att(4, 2, 64, 64, 0.11, 40, 5), 192)] * 3, 160, 128, loop=(1, 2, 3), side=16),
    # every layer different: head counts and sizes, windows shorter and longer than a page, no feed-forward,
    # padded sizes everywhere, a loop from the first layer on, eps that matters
    "mixed": config([layer(att(6, 3, 24, 40, 0.2, 7, 2), 72), layer(att(5, 1, 80, 24, 0.09, 70, 65)),
                     layer(att(3, 3, 48, 100, 0.15, 64, 0), 200), layer(att(8, 2, 16, 16, 0.3, 130, 1), 40)],
                    331, 200, embed=0.7, mult=1.3, eps=3e-2, loop=(0, 3, 2), side=10),
    # all the values that may hide a factor: one query head, scale and multipliers of one, a window of one key
    "ones": config([layer(att(1, 1, 32, 32, 1.0, 1, 1), 64), layer(att(2, 2, 32, 64, 1.0, 1, 0), 64)], 97, 64,
                   embed=1.0, mult=1.0, loop=(1, 2, 1), side=64),
    # no loop, no token input, full attention, wide heads, many query heads over one key head
    "full": config([layer(att(40, 1, 32, 136, 0.18), 96), layer(att(2, 1, 200, 72, 0.07, 33, 40), 64)], 256, 96,
                   mult=0.4),
    # the loop reaches the last layer
    "tail": config([layer(att(4, 4, 40, 40, 0.16, 20, 30), 104)] * 4, 128, 136, loop=(2, 4, 3), side=24, mult=0.5),
}
