"""Small Rudazen configurations for the tests: sizes that no fast kernel's tiling suits, sizes
that suit them, and one in which much is 1 or absent (one head, blocks of one token, a window
of one position, no rotation, a residual factor of 1, a layer without a feed-forward, a layer
without blocks, a layer without a window)."""
import math
import random


def rot(dims, base=10000.0, scaling=None):
    r = {"base": base, "dims": dims}
    if scaling:
        r["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    return r


def heads_of(heads, kv_heads, dim, vdim=None, size=None, pool=None, rot_dims=None, base=10000.0,
             scaling=None, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim if vdim is None else vdim,
         "scale": scale if scale is not None else 1.0 / math.sqrt(dim),
         "rot": rot(dim if rot_dims is None else rot_dims, base, scaling)}
    if size:
        m["mask"] = {"size": size}
        if pool:
            m["mask"]["pool"] = pool
    return m


def attention(*a, **k):
    return {"type": "attention", "mixer": heads_of(*a, **k)}


def parallel(left, heads, dim, vdim):
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": heads, "dim": dim, "vdim": vdim}}}


def layer(mixer, ff):
    return dict(mixer, mlp=None if ff is None else {"kind": "dense", "ff": ff})


def model(vocab, width, eps, alpha, scale, layers):
    return {"architecture": "Rudazen", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "postln_alpha": alpha, "embedding": {"scale": scale}, "layers": layers}


def config_odd():
    sc = (3.0, 24, 4.0, 0.5)
    return model(211, 72, 1e-5, 1.7, 5.5, [
        layer(attention(6, 3, 20, size=11, pool=3, rot_dims=10, base=500.0), 40),
        layer(parallel(heads_of(6, 2, 12, 20, size=17, rot_dims=12, base=300.0, scaling=sc), 3, 12, 20), 56),
        layer(attention(3, 1, 36, size=5, pool=7, rot_dims=36), None),
        layer(parallel(heads_of(3, 3, 28, 36, size=33, rot_dims=6, base=90.0), 2, 20, 9), 24)])


def config_even():
    sc = (4.0, 64, 8.0, 1.0)
    return model(384, 128, 1e-6, 2.2, 9.0, [
        layer(parallel(heads_of(8, 2, 64, 32, size=48, rot_dims=32, scaling=sc), 4, 32, 64), 128),
        layer(attention(8, 2, 64, size=32, pool=16, base=2000.0), 192),
        layer(attention(4, 4, 32, size=40, pool=8, rot_dims=16), 64),
        layer(attention(4, 1, 128, size=24, pool=4), None),
        layer(parallel(heads_of(4, 1, 128, size=70, rot_dims=128, base=100000.0), 2, 64, 128), 96)])


def config_ones():
    return model(96, 64, 1e-5, 1.0, 1.0, [
        layer(attention(1, 1, 16, size=1, pool=1, rot_dims=2), 16),
        layer(attention(2, 1, 8, rot_dims=0), 24),
        layer(parallel(heads_of(1, 1, 8, 24, rot_dims=0), 1, 4, 8), None),
        layer(attention(2, 2, 24, size=9), 16),
        layer(attention(2, 1, 8, size=2, pool=5), 32)])


CASES = {"odd": (config_odd, 31), "even": (config_even, 32), "ones": (config_ones, 33)}


def random_config(seed: int) -> dict:
    """A seeded random configuration: sizes, head counts, kinds and order of layers, windows,
    blocks, what is absent."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 5)):
        kv = rng.choice([1, 2, 3])
        dim = rng.choice([8, 12, 16, 32, 40, 64])
        heads, size = kv * rng.choice([1, 2, 4]), rng.choice([None, 1, 3, 16, 31, 32, 40])
        common = dict(rot_dims=rng.choice([0, dim // 2 // 2 * 2, dim]), base=rng.choice([50.0, 10000.0]),
                      scale=rng.choice([None, 0.3]))
        if rng.random() < 0.6:
            pool = rng.choice([None, 1, 2, 5, 8, 16]) if size else None
            m = attention(heads, kv, dim, size=size, pool=pool, **common)
        else:
            sc = rng.choice([None, (2.0, 24, 3.0, 1.0), (8.0, 100, 16.0, 0.5), (4.0, 48, 2.0, 2.0)])
            left = heads_of(heads, kv, dim, rng.choice([8, 16, 20, 48]), size=size, scaling=sc, **common)
            m = parallel(left, rng.choice([1, 2, 3]), rng.choice([4, 8, 16, 20, 32]), rng.choice([8, 12, 16, 40]))
        layers.append(layer(m, rng.choice([None, 16, 40, 64, 96])))
    return model(rng.choice([64, 130, 300]), rng.choice([48, 64, 72, 96, 136]), rng.choice([1e-5, 1e-6]),
                 rng.choice([1.0, 1.5, 3.0]), rng.choice([1.0, 4.0, 10.0]), layers)
