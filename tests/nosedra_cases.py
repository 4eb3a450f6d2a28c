"""Small Nosedra configurations for the tests: sizes that no fast kernel's tiling suits, sizes
that suit them, and one in which much is 1 or absent (one head, one group, one tap, no rotation,
factors of 1, layers without a feed-forward, no cap on the logits)."""
import math
import random


def parallel(heads, kv_heads, dim, vdim, mem_heads, mem_dim, mem_vdim, rot_dims=None, base=10000.0, factor=None,
             scale=None, cap=10.0, scales=(1.0, 1.0)):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim,
            "scale": scale if scale is not None else 1.0 / math.sqrt(dim)}
    if rot_dims != 0:
        left["rot"] = {"base": base, "dims": dim if rot_dims is None else rot_dims}
        if factor is not None:
            left["rot"]["scaling"] = {"factor": factor}
    return {"type": "parallel", "mixer": {
        "left": left, "right": {"heads": mem_heads, "dim": mem_dim, "vdim": mem_vdim, "gate_cap": cap},
        "left_scale": scales[0], "right_scale": scales[1]}}


def mamba2(heads, vdim, state, groups=1, conv=4, norm_groups=1):
    return {"type": "mamba2", "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups,
                                        "conv": conv, "norm_groups": norm_groups}}


def layer(mixer, ff):
    return dict(mixer, mlp=None if ff is None else {"kind": "dense", "ff": ff})


def model(vocab, width, eps, side, softcap, layers):
    return {"architecture": "Nosedra", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "token_side": {"dim": side}, "logit_softcap": softcap, "layers": layers}


def config_odd():
    return model(211, 72, 1e-5, 9, 7.0, [
        layer(mamba2(6, 10, 12, groups=3, conv=3, norm_groups=4), 40),
        layer(parallel(6, 2, 20, 12, 3, 14, 9, rot_dims=10, base=500.0, factor=3.0, cap=6.0, scales=(0.7, -1.3)), 56),
        layer(mamba2(3, 7, 33, conv=5), None),
        layer(parallel(3, 3, 28, 36, 5, 6, 11, rot_dims=28, base=90.0, scale=0.4, scales=(1.6, 0.5)), 24)])


def config_even():
    return model(384, 128, 1e-6, 16, 20.0, [
        layer(parallel(8, 2, 64, 64, 4, 32, 64, rot_dims=32, factor=4.0, cap=12.0, scales=(0.9, 1.2)), 128),
        layer(mamba2(8, 32, 64, groups=2, norm_groups=2), 192),
        layer(mamba2(4, 64, 128, conv=2), 64),
        layer(parallel(4, 1, 128, 128, 2, 128, 128, base=100000.0, scales=(0.5, 0.75)), None),
        layer(parallel(4, 4, 32, 40, 8, 16, 24, rot_dims=16, factor=0.5), 96)])


def config_ones():
    return model(96, 64, 1e-5, 1, 0.0, [
        layer(mamba2(1, 16, 8, conv=1), 16),
        layer(parallel(1, 1, 8, 24, 1, 8, 8, rot_dims=0), None),
        layer(mamba2(4, 8, 1, groups=4, norm_groups=4, conv=2), None),
        layer(parallel(2, 1, 16, 16, 2, 4, 16, rot_dims=2, factor=1.0), 32)])


CASES = {"odd": (config_odd, 41), "even": (config_even, 42), "ones": (config_ones, 43)}


def alone(kind: str) -> dict:
    """A model of layers of one kind (a model of state-space layers keeps nothing in pages)."""
    if kind == "parallel":
        layers = [layer(parallel(4, 2, 40, 24, 2, 24, 32, factor=2.0), 48), layer(parallel(2, 1, 16, 16, 3, 8, 16), None)]
    else:
        layers = [layer(mamba2(4, 24, 40, groups=2), 48), layer(mamba2(2, 8, 16, conv=3), None)]
    return model(130, 96, 1e-6, 12, 15.0, layers)


def random_config(seed: int) -> dict:
    """A seeded random configuration: sizes, head counts, kinds and order of layers, what is
    absent."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 5)):
        if rng.random() < 0.55:
            kv, dim = rng.choice([1, 2, 3]), rng.choice([8, 12, 16, 32, 40, 64, 80, 128])
            m = parallel(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([8, 16, 20, 48, dim]),
                         rng.choice([1, 2, 3, 6]), rng.choice([4, 8, 16, 20, 40, 72]), rng.choice([8, 12, 16, 40, 72]),
                         rot_dims=rng.choice([0, dim // 2 // 2 * 2, dim]), base=rng.choice([50.0, 10000.0]),
                         factor=rng.choice([None, 2.0, 8.0]), scale=rng.choice([None, 0.3]),
                         cap=rng.choice([3.0, 15.0]), scales=rng.choice([(1.0, 1.0), (0.6, 1.4), (2.0, -0.5)]))
        else:
            groups = rng.choice([1, 2, 3])
            heads = groups * rng.choice([1, 2, 4])
            vdim = rng.choice([4, 8, 16, 24, 64])
            m = mamba2(heads, vdim, rng.choice([4, 8, 16, 20, 40, 64, 136]), groups, rng.choice([1, 2, 3, 4, 6]),
                       rng.choice([1, 2, heads]) if vdim % 2 == 0 else 1)
        layers.append(layer(m, rng.choice([None, 16, 40, 64, 96])))
    return model(rng.choice([64, 130, 300]), rng.choice([48, 64, 72, 96, 136]), rng.choice([1e-5, 1e-6]),
                 rng.choice([3, 8, 16, 40]), rng.choice([0.0, 5.0, 30.0]), layers)
