"""Small Lifesun configurations that differ from each other in every size, constant and option."""
import random

import torch


def _attention(heads, kv_heads, dim, vdim, scale, size):
    d = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale}
    if size is not None:
        d["mask"] = {"size": size}
    return d


def _unit(width, blocks, conv):
    return {"width": width, "blocks": blocks, "conv": conv}


def _retention(heads, dim, vdim, base, dims, decay):
    return {"heads": heads, "dim": dim, "vdim": vdim, "rot": {"base": base, "dims": dims}, "decay": decay}


def _chunked(left, right, scales, ff=None):
    return {"type": "parallel", "mixer": {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _capped(left, cap, base, dims, right, scales, ff=None):
    left = dict(left, softcap=cap, rot={"base": base, "dims": dims})
    return {"type": "parallel_2", "mixer": {"left": left, "right": right, "left_scale": scales[0], "right_scale": scales[1]},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff}}


def _top(vocab, width, eps, logit_scale, layers, loop=None):
    d = {"architecture": "Lifesun", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
         "layers": layers}
    if loop is not None:
        d["loop"] = dict(zip(("start", "stop", "times"), loop))
    return d


LIFESUN = {
    # both mixers, grouped and single kv heads, values smaller and larger than keys, partly turned heads, a stretch run
    # three times, a layer without a feed-forward
    "LA": dict(seed=3, **_top(300, 64, 1e-5, 0.6, [
        _chunked(_attention(4, 2, 16, 24, 0.4, 24), _unit(48, 3, 3), (0.8, 1.2), 40),
        _capped(_attention(6, 3, 16, 8, 0.3, 33), 3.0, 500.0, 8, _retention(3, 16, 20, 900.0, 12, [0.5, 0.97, 0.999]),
                (1.1, 0.7), 24),
        _capped(_attention(4, 4, 24, 16, 0.35, 17), 5.0, 3000.0, 24, _retention(2, 8, 24, 50.0, 8, [0.9, 1.0]), (0.6, 0.9)),
        _chunked(_attention(6, 1, 8, 16, 0.5, 40), _unit(80, 5, 5), (1.3, 0.5), 56),
    ], loop=(1, 3, 3))),
    # sizes that fit no fast path (a width that is no multiple of 4, heads of 6 and 10 elements, blocks of 5 and 7, a
    # prime vocabulary), a loop from the first layer on that runs once, one block, one tap, one head, no masks, a
    # window of one token, a decay of zero
    "LB": dict(seed=5, **_top(257, 54, 1e-3, 1.7, [
        _capped(_attention(3, 1, 10, 6, 0.5, 1), 2.0, 30.0, 2, _retention(2, 6, 10, 7.0, 4, [0.0, 0.8]), (0.5, 1.0), 22),
        _chunked(_attention(2, 2, 6, 10, 0.6, 5), _unit(35, 7, 1), (1.0, 1.0), 30),
        _chunked(_attention(1, 1, 10, 3, 0.4, None), _unit(21, 3, 6), (-0.7, 0.4)),
        _capped(_attention(4, 2, 6, 7, 0.7, None), 1.5, 9000.0, 6, _retention(1, 5, 3, 100.0, 2, [0.95]), (0.9, -1.1), 18),
        _chunked(_attention(5, 5, 3, 9, 0.5, 1), _unit(13, 1, 2), (0.3, 1.6), 14),
    ], loop=(0, 2, 1))),
    # sharp scores: a key just inside a window or a chunk, or one where a page ends, carries most of a query's weight
    "LS": dict(seed=13, **_top(128, 32, 1e-5, 1.0, [
        _chunked(_attention(2, 1, 16, 16, 1.0, 48), _unit(32, 2, 4), (1.0, 0.3), 32),
        _capped(_attention(2, 2, 16, 16, 0.8, 48), 12.0, 10000.0, 16, _retention(2, 16, 16, 10000.0, 16, [0.99, 0.7]),
                (1.0, 0.3), 48),
    ])),
}

# with the sizes the vector and matrix-core paths need (GPU tests)
LIFESUN_FAST = {
    "LF": dict(seed=9, **_top(1000, 192, 1e-6, 0.4, [
        _capped(_attention(8, 2, 64, 64, 0.125, 80), 20.0, 20000.0, 48,
                _retention(3, 64, 128, 5000.0, 64, [0.96875, 0.998, 0.6]), (0.9, 0.8), 128),
        _chunked(_attention(4, 4, 64, 32, 0.15, 112), _unit(256, 2, 4), (0.7, 1.0), 320),
        _chunked(_attention(8, 4, 40, 64, 0.2, 70), _unit(192, 12, 2), (1.2, 0.6)),
        _capped(_attention(4, 2, 128, 128, 0.09, 100), 8.0, 700.0, 128, _retention(2, 96, 40, 60.0, 32, [0.99, 0.999]),
                (0.5, 1.0), 64),
        _chunked(_attention(6, 3, 128, 96, 0.1, 130), _unit(384, 3, 3), (1.0, 1.0), 96),
    ], loop=(2, 4, 2))),
    # wide enough for several pieces of a row a thread, the streaming layout of the pass product, long keys and values
    "LW": dict(seed=11, **_top(512, 1280, 1e-5, 1.3, [
        _chunked(_attention(10, 5, 128, 128, 0.09, 90), _unit(1024, 4, 4), (0.9, 0.8), 512),
        _capped(_attention(4, 1, 256, 256, 0.0625, 75), 15.0, 30000.0, 200,
                _retention(2, 256, 512, 10000.0, 256, [0.98, 0.9995]), (0.7, 0.9), 256),
    ], loop=(0, 2, 2))),
}


def lifesun_config_json(name: str) -> dict:
    return {k: v for k, v in {**LIFESUN, **LIFESUN_FAST}[name].items() if k != "seed"}


def write_lifesun(name: str, out_dir: str, dtype=torch.float32) -> str:
    from jax_llm_examples_amd.config import get_architecture
    from jax_llm_examples_amd.weights import write_random_model

    top = lifesun_config_json(name)
    arch = get_architecture(top["architecture"])
    return write_random_model(arch, arch.parse_config(top), out_dir, {**LIFESUN, **LIFESUN_FAST}[name]["seed"], dtype)


def draw_lifesun(seed: int):
    """A configuration drawn at random: ``(config.json, page size, request lengths)``."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(1, 4)):
        kv = rng.choice([1, 2, 3])
        dim = rng.choice([8, 12, 16, 32, 64, 96, 128])
        left = _attention(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([8, 10, 16, 40, 64, 128]), rng.choice([0.1, 0.3]),
                          rng.choice([None, 1, 5, 16, 31, 64, 100]))
        scales = (rng.choice([0.5, 0.9, 1.0]), rng.choice([0.4, 1.0, 1.2]))
        ff = rng.choice([None, 16, 40, 64, 192])
        if rng.random() < 0.5:
            blocks = rng.choice([1, 2, 3, 4, 8])
            layers.append(_chunked(left, _unit(blocks * rng.choice([1, 4, 9, 16, 32, 64, 128, 144]), blocks,
                                               rng.choice([1, 2, 4, 5])), scales, ff))
        else:
            heads, rdim = rng.choice([1, 2, 3]), rng.choice([4, 8, 20, 32, 64, 72, 128, 160])
            layers.append(_capped(left, rng.choice([2.0, 15.0, 50.0]), rng.choice([100.0, 250000.0]),
                                  rng.choice([d for d in (2, 4, 8, 16, 32, 64, 96, 128) if d <= dim]),
                                  _retention(heads, rdim, rng.choice([4, 10, 16, 64, 80, 128, 136, 256]),
                                             rng.choice([50.0, 1e6]), rng.choice([2, 4, rdim]),
                                             [rng.choice([0.5, 0.9, 0.984375, 0.9995, 1.0]) for _ in range(heads)]),
                                  scales, ff))
    n = len(layers)
    start = rng.randint(0, n - 1)
    loop = rng.choice([None, (start, rng.randint(start + 1, n), rng.choice([1, 2, 3]))])
    top = _top(rng.choice([97, 257, 300, 512, 1001]), rng.choice([56, 62, 64, 72, 100, 128, 192, 256, 264]),
               rng.choice([1e-5, 1e-6, 1e-3]), rng.choice([0.2, 1.0, 1.5]), layers, loop)
    lengths = [rng.choice([1, 2, 17, 33, 64, 65, 97, 130, 200]) for _ in range(rng.randint(2, 5))]
    return top, rng.choice([16, 16, 32, 64]), lengths
