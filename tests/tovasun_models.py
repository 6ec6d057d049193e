"""Small Tovasun models for the tests: odd sizes, every branch, sharp attention (score deviations of about 3), so that one key
more or less shows in the logits."""
import copy
import math

YARN = {"factor": 3.0, "fast": 8.0, "original": 48, "slow": 1.0}


def attention(heads, kv_heads, dim, vdim, rot=None, window=0, keep=0, softcap=0.0, base=1000.0, sharp=3.0):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": sharp / math.sqrt(dim),
         "rot": {"base": base, "dims": dim if rot is None else rot}}
    if window:
        m["mask"] = {"size": window, "keep_first": keep}
    if softcap:
        m["softcap"] = softcap
    return m


def latent(heads, dim, rot_dim, kv_rank, vdim, window=0, yarn=YARN, base=500.0, sharp=3.0):
    m = {"heads": heads, "dim": dim, "rot_dim": rot_dim, "kv_rank": kv_rank, "vdim": vdim,
         "scale": sharp / math.sqrt(dim + rot_dim), "rot": {"base": base, "dims": rot_dim}}
    if yarn:
        m["rot"]["scaling"] = dict(yarn)
    if window:
        m["mask"] = {"size": window}
    return m


def layer(mixer, ff=None):
    return {"type": "latent_attention" if "kv_rank" in mixer else "attention", "mixer": mixer,
            "mlp": {"kind": "dense", "ff": ff} if ff else None}


def model(layers, width, vocab, loop=None, side=0, eps=1e-5):
    cfg = {"architecture": "Tovasun", "layers": layers, "norm": {"eps": eps}, "vocab": vocab, "width": width}
    if loop:
        cfg["loop"] = {"start": loop[0], "stop": loop[1], "times": loop[2]}
    if side:
        cfg["token_side"] = {"dim": side}
    return cfg


MODELS = {
    # every branch at sizes that are multiples of nothing
    "odd": model([layer(latent(3, 20, 6, 27, 13, window=9), 50), layer(attention(6, 2, 22, 14, rot=10, window=13, keep=3, softcap=8.0)),
                  layer(attention(4, 4, 18, 30), 37), layer(latent(5, 12, 10, 40, 24, yarn=None), 61)],
                 76, 101, loop=(1, 3, 2), side=11),
    # the loop starts at the first layer and covers all of them; one pass would be no loop
    "all_looped": model([layer(latent(2, 16, 8, 24, 16, window=5), 40), layer(attention(2, 1, 16, 16, window=6, keep=2), 40)],
                        48, 67, loop=(0, 2, 4), side=8),
    # no loop, no token input
    "plain": model([layer(attention(8, 2, 40, 24, window=21, keep=1, softcap=20.0), 96), layer(latent(6, 24, 16, 72, 40, window=30), 96)], 96, 131),
    # more kept positions than a tile of 64, a window over several tiles, 16 query heads on one kv head
    "wide_keep": model([layer(attention(16, 1, 128, 128, rot=64, window=100, keep=70), 64)], 128, 97),
    # more than 16 (two head tiles) and more than 32 query heads per kv head
    "many_heads": model([layer(attention(20, 1, 24, 72, rot=8, window=40, keep=5), 64), layer(attention(40, 1, 16, 16), 64),
                         layer(latent(36, 16, 8, 120, 16, window=33))], 64, 89, side=5),
    # the largest tile classes: keys of 576 and 320 in the latent step, 192 / 128 and 256 / 256 in the prompt pass
    "large_heads": model([layer(latent(4, 128, 64, 512, 128, window=50), 128), layer(latent(2, 160, 40, 200, 200)),
                          layer(latent(2, 40, 24, 264, 64, window=70)), layer(attention(4, 2, 200, 250, window=45, keep=2), 128)], 128, 103),
    # sizes beyond every tile class: the plain kernels
    "beyond_classes": model([layer(attention(2, 1, 264, 300, rot=100, window=17, keep=4), 64), layer(latent(2, 40, 16, 600, 20, window=23))], 64, 71),
}


def random_model(seed):
    """A design of any shape: sizes, heads, masks, layer order, loop and token input drawn at random."""
    import random
    r = random.Random(seed)
    layers = []
    for _ in range(r.randint(1, 5)):
        window = r.choice([0, 1, 2, r.randint(3, 30), r.randint(40, 140)])
        ff = r.choice([None, r.randint(9, 150), 8 * r.randint(2, 20)])
        if r.random() < 0.5:
            kv = r.choice([1, 2, 3])
            dim = r.choice([r.randint(5, 40), 64, 32, r.randint(60, 130)])
            mix = attention(kv * r.choice([1, 2, 3, 5, 8, 17]), kv, dim, r.choice([dim, r.randint(3, 90)]),
                            rot=2 * r.randint(1, dim // 2), window=window, keep=r.choice([0, 1, r.randint(2, 12), 80]) if window else 0,
                            softcap=r.choice([0.0, 6.0, 40.0]), base=r.choice([100.0, 1e4, 5e5]), sharp=r.choice([1.0, 2.0]))
            if r.random() < 0.3:
                mix["rot"]["scaling"] = dict(YARN)
        else:
            mix = latent(r.choice([1, 2, 5, 18]), r.randint(4, 70), 2 * r.randint(2, 20), r.choice([r.randint(8, 60), 64, r.randint(65, 300)]),
                         r.randint(4, 70), window=window, yarn=r.choice([None, YARN, {"factor": 1.7, "fast": 20.0, "slow": 2.0, "original": 700}]),
                         base=r.choice([300.0, 1e4]), sharp=r.choice([1.0, 2.0]))
        layers.append(layer(mix, ff))
    n = len(layers)
    loop = None
    if r.random() < 0.6:
        start = r.randrange(n)
        loop = (start, r.randint(start + 1, n), r.randint(1, 4))
    return model(layers, r.choice([r.randint(20, 120), 64, 192]), r.randint(30, 300), loop=loop, side=r.choice([0, 1, r.randint(2, 70)]),
                 eps=r.choice([1e-6, 1e-5, 1e-2]))


def variant(cfg, **changes):
    """A copy with mixer or mask entries of some layers changed: variant(cfg, l1_size=+1, l1_keep_first=-1)."""
    out = copy.deepcopy(cfg)
    for key, delta in changes.items():
        i, what = key[1:].split("_", 1)
        m = out["layers"][int(i)]["mixer"]
        (m["mask"] if what in ("size", "keep_first") else m)[what] += delta
    return out
