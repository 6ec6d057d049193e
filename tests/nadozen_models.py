"""Small Nadozen models for the tests: odd sizes, every branch, sharp attention (score deviations of about 3), so that one key more
or less shows in the logits."""
import copy
import math


def wkv(heads, dim, rank, ff=None):
    return {"type": "wkv", "mixer": {"heads": heads, "dim": dim}, "rank": rank, "mlp": {"kind": "dense", "ff": ff} if ff else None}


def parallel(heads, kv_heads, dim, window, ssm, ff=None, sharp=3.0, scales=(0.7, 0.8)):
    """ssm: (heads, value size, state, groups, convolution taps, norm groups)"""
    names = ("heads", "vdim", "state", "groups", "conv", "norm_groups")
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": sharp / math.sqrt(dim), "mask": {"size": window}}
    return {"type": "parallel", "mixer": {"left": left, "right": dict(zip(names, ssm)), "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def again(i, layers):
    return {**copy.deepcopy(layers[i]), "weights_of": i}


def model(layers, width, vocab, streams, eps=1e-5, logit_scale=0.6):
    layers = [again(x, layers) if isinstance(x, int) else x for x in layers]
    return {"architecture": "Nadozen", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width, "streams": streams,
            "logit_scale": logit_scale}


MODELS = {
    # every branch at sizes that are multiples of nothing; weights shared by name, also of a layer that comes later
    "odd": model([wkv(3, 13, 5, ff=37), parallel(6, 2, 14, 9, (4, 11, 7, 2, 3, 4), ff=50), 0, wkv(2, 22, 9), 1,
                  parallel(3, 3, 20, 30, (5, 6, 18, 5, 5, 3)), 3], 61, 101, 2),
    # one stream, one head, one tap, one token of window, one value per head (no norm over a single value: its sign would turn on the
    # last bit)
    "ones": model([parallel(1, 1, 8, 1, (6, 1, 1, 1, 1, 1), ff=1), wkv(1, 6, 1), parallel(2, 1, 4, 2, (1, 8, 3, 1, 2, 1))], 17, 23, 1, logit_scale=1.0),
    # whole sections of 128 rows, states of 64 and 128 keys, windows over several tiles
    "whole": model([wkv(2, 64, 32, ff=96), parallel(4, 2, 64, 100, (4, 32, 128, 1, 4, 1), ff=128), wkv(1, 128, 64), 1], 128, 131, 4),
    # larger heads and states: every tile class of the recurrences, 16 and more query heads per key head, more than four norm parts
    "large": model([wkv(2, 140, 70), parallel(18, 1, 128, 33, (3, 20, 200, 3, 4, 6), ff=64), wkv(1, 300, 16), parallel(2, 1, 200, 70, (1, 40, 300, 1, 7, 5)),
                    parallel(34, 2, 16, 65, (2, 130, 5, 1, 4, 2))], 96, 89, 3),
    # head sizes beyond the matrix-core classes, more streams than fit the small kernel
    "beyond": model([parallel(2, 1, 264, 17, (2, 17, 9, 2, 4, 1)), wkv(2, 9, 3)], 64, 71, 6),
}


def random_model(seed):
    """A design of any shape: sizes, heads, windows, layer order, shared weights and streams drawn at random."""
    import random
    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(1, 5)):
        ff = r.choice([None, r.randint(9, 150), 8 * r.randint(2, 20)])
        if layers and r.random() < 0.3:
            layers.append(r.randrange(len(layers)))
            while isinstance(layers[layers[-1]], int):
                layers[-1] = layers[layers[-1]]
        elif r.random() < 0.5:
            layers.append(wkv(r.choice([1, 2, 3, 6]), r.choice([r.randint(2, 40), 64, 128, r.randint(60, 150)]), r.choice([r.randint(1, 40), 64, 130]), ff))
        else:
            kv = r.choice([1, 2, 3])
            heads = r.choice([1, 2, 3, 6])
            vdim, groups = r.choice([r.randint(2, 40), 64]), r.choice([g for g in (1, 2, 3, 6) if heads % g == 0])
            parts = r.choice([n for n in (1, 2, 3, 4, 6, 8) if heads * vdim % n == 0])
            layers.append(parallel(kv * r.choice([1, 2, 3, 5, 8, 17]), kv, r.choice([r.randint(5, 40), 64, 32, r.randint(60, 130)]),
                                   r.choice([1, 2, r.randint(3, 30), r.randint(40, 140), 1000]),
                                   (heads, vdim, r.choice([r.randint(1, 60), 64, 128, r.randint(100, 260)]), groups, r.choice([1, 2, 4, r.randint(3, 9)]), parts),
                                   ff, sharp=r.choice([1.0, 2.0]), scales=(r.choice([1.0, 0.3]), r.choice([1.0, -0.6]))))
    return model(layers, r.choice([r.randint(20, 120), 64, 192]), r.randint(30, 300), r.choice([1, 2, 3, 4, 5]), eps=r.choice([1e-6, 1e-5, 1e-2]),
                 logit_scale=r.choice([1.0, 0.25]))


def variant(cfg, layer, delta):
    """A copy whose window of one layer (and of those that share its weights) is `delta` longer."""
    out = copy.deepcopy(cfg)
    for i, L in enumerate(out["layers"]):
        if i == layer or L.get("weights_of") == layer:
            L["mixer"]["left"]["mask"]["size"] += delta
    return out
