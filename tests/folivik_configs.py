"""Small Folivik configurations that differ from each other in every size, constant and option."""
import random

import torch


def _latent(heads, dim, rot_dim, vdim, kv_rank, q_rank, scale, base, mlp=None):
    return {"type": "latent_attention", "mlp": mlp,
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "scale": scale, "rot": {"base": base, "dims": rot_dim}}}


def _window(heads, kv_heads, dim, vdim, scale, size, mlp=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": scale,
                      "mask": {"size": size}}}


def _mamba(heads, vdim, state, groups, conv, norm_groups, mlp=None):
    return {"type": "mamba2", "mlp": mlp,
            "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "conv": conv,
                      "norm_groups": norm_groups}}


def _moe(experts, top, ff, groups=None, keep=None, identity=0, scale=1.0, shared=None):
    router = {"experts": experts, "top": top, "scale": scale}
    if groups is not None:
        router["groups"] = {"count": groups, "keep": keep}
    if identity:
        router["identity"] = identity
    d = {"kind": "moe", "router": router, "expert": {"ff": ff}}
    if shared is not None:
        d["shared"] = {"ff": shared}
    return d


def _top(vocab, width, eps, layers):
    return {"architecture": "Folivik", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


FOLIVIK = {
    # every mixer, grouped kv heads, values smaller and larger than keys, a window shorter than a prompt, identity
    # experts that fill a group of their own or part of one, shared experts wider and narrower than the routed ones,
    # a layer without a feed-forward
    "FA": dict(seed=3, **_top(300, 64, 1e-5, [
        _mamba(4, 12, 20, 2, 3, 2, _moe(6, 3, 24, groups=4, keep=2, identity=2, scale=1.7, shared=40)),
        _window(4, 2, 16, 24, 0.3, 24, _moe(4, 2, 16, identity=1, scale=0.8)),
        _latent(4, 12, 8, 20, 24, 40, 0.22, 5000.0, _moe(8, 2, 32, groups=2, keep=1, scale=2.0, shared=32)),
        _mamba(6, 8, 16, 3, 4, 1, None),
        _window(6, 6, 24, 8, 0.25, 33, _moe(5, 4, 16, groups=4, keep=3, identity=3, scale=1.3, shared=8)),
    ])),
    # sizes that fit no fast path (a width that is no multiple of 4, heads of 6 and 10 elements, a prime vocabulary),
    # one kv head, one group of experts, groups of one expert, every expert chosen, only identity experts beside one
    # expert, a convolution of one tap, one head, a state of one number, a window of one token
    "FB": dict(seed=5, **_top(257, 54, 1e-3, [
        _mamba(3, 7, 5, 1, 1, 3, _moe(2, 2, 20, groups=1, keep=1, scale=1.5)),
        _latent(3, 6, 2, 10, 9, 7, 0.4, 30.0, _moe(3, 2, 18, groups=4, keep=3, identity=1, shared=10)),
        _window(3, 1, 10, 6, 0.5, 1, _moe(1, 2, 22, identity=3, scale=0.7, shared=22)),
        _mamba(1, 9, 1, 1, 6, 1, _moe(3, 3, 12)),
        _window(2, 2, 6, 10, 0.6, 7, None),
        _latent(1, 10, 6, 6, 12, 20, 0.3, 900.0, _moe(5, 1, 14, scale=3.0)),
    ])),
    # sharp scores: a key just inside a window, or one where a page ends, carries most of a query's weight
    "FS": dict(seed=13, **_top(128, 32, 1e-5, [
        _window(2, 1, 16, 16, 1.5, 48, _moe(4, 2, 16, groups=3, keep=2, identity=2, scale=1.2, shared=16)),
        _latent(2, 16, 8, 16, 32, 24, 1.2, 10000.0, _moe(4, 2, 16, identity=2)),
        _mamba(2, 16, 16, 1, 4, 1, None),
    ])),
}

# with the sizes the vector and matrix-core paths need (GPU tests)
FOLIVIK_FAST = {
    "FF": dict(seed=9, **_top(1000, 256, 1e-6, [
        _mamba(8, 64, 128, 2, 4, 4, _moe(8, 2, 128, groups=5, keep=3, identity=2, scale=2.0, shared=128)),
        _window(8, 2, 64, 64, 0.125, 80, _moe(16, 4, 64, groups=4, keep=2, scale=1.5, shared=256)),
        _latent(8, 32, 32, 64, 96, 160, 0.125, 20000.0, _moe(6, 3, 64, identity=6)),
        _mamba(4, 96, 64, 4, 4, 1, _moe(6, 1, 64, scale=1.1)),
        _window(4, 2, 128, 128, 0.09, 100, None),
        _mamba(2, 40, 200, 1, 2, 2, None),
    ])),
    # wide enough for the launch that norms, routes and groups in one, and for experts in the streaming layout
    "FW": dict(seed=11, **_top(512, 1280, 1e-5, [
        _window(8, 4, 128, 96, 0.09, 70, _moe(8, 3, 256, groups=4, keep=3, identity=4, scale=2.5, shared=256)),
        _mamba(8, 64, 64, 1, 4, 2, _moe(70, 6, 128, groups=6, keep=4, identity=2, scale=1.6, shared=256)),
        _latent(4, 64, 32, 64, 128, 256, 0.1, 10000.0, _moe(12, 2, 256, scale=1.2)),
    ])),
}


def folivik_config_json(name: str) -> dict:
    return {k: v for k, v in {**FOLIVIK, **FOLIVIK_FAST}[name].items() if k != "seed"}


def write_folivik(name: str, out_dir: str, dtype=torch.float32) -> str:
    from jax_llm_examples_amd.config import get_architecture
    from jax_llm_examples_amd.weights import write_random_model

    top = folivik_config_json(name)
    arch = get_architecture(top["architecture"])
    return write_random_model(arch, arch.parse_config(top), out_dir, {**FOLIVIK, **FOLIVIK_FAST}[name]["seed"], dtype)


def draw_folivik(seed: int):
    """A configuration drawn at random: ``(config.json, page size, request lengths)``."""
    rng = random.Random(seed)

    def moe():
        experts, identity = rng.choice([1, 2, 4, 6, 7, 12]), rng.choice([0, 0, 1, 2, 4])
        outputs = experts + identity
        groups = rng.choice([None] + [g for g in (1, 2, 3, 4, 5) if outputs % g == 0])
        keep = None if groups is None else rng.randint(1, groups)
        most = outputs if groups is None else keep * (outputs // groups)
        return _moe(experts, rng.randint(1, min(most, 5)), rng.choice([16, 20, 24, 64, 96]), groups, keep, identity,
                    rng.choice([1.0, 0.6, 2.2]), rng.choice([None, 16, 48, 64]))

    layers = []
    for _ in range(rng.randint(1, 4)):
        mlp = rng.choice([None, moe(), moe()])
        kind = rng.choice(["mamba", "window", "latent"])
        if kind == "mamba":
            groups = rng.choice([1, 2, 3])
            heads = groups * rng.choice([1, 2, 4])
            vdim = rng.choice([4, 8, 12, 16, 40, 64, 80, 128])
            norm_groups = rng.choice([g for g in (1, 2, 3, 4) if heads * vdim % g == 0])
            layers.append(_mamba(heads, vdim, rng.choice([3, 8, 16, 40, 64, 100, 128, 160]), groups,
                                 rng.choice([1, 2, 4, 5]), norm_groups, mlp))
        elif kind == "window":
            kv = rng.choice([1, 2, 3])
            layers.append(_window(kv * rng.choice([1, 2, 4]), kv, rng.choice([8, 12, 16, 32, 64, 128]),
                                  rng.choice([8, 10, 16, 40, 64, 128]), rng.choice([0.1, 0.3]),
                                  rng.choice([1, 5, 16, 31, 64, 100]), mlp))
        else:
            layers.append(_latent(rng.choice([1, 2, 4, 6]), rng.choice([8, 10, 16, 32, 64]), rng.choice([2, 4, 8, 16, 32]),
                                  rng.choice([8, 12, 16, 40, 64]), rng.choice([8, 20, 32, 64, 128]),
                                  rng.choice([8, 18, 32, 96]), rng.choice([0.1, 0.25]), rng.choice([100.0, 250000.0]), mlp))
    top = _top(rng.choice([97, 257, 300, 512, 1001]), rng.choice([56, 64, 72, 100, 128, 192, 256, 264]),
               rng.choice([1e-5, 1e-6, 1e-3]), layers)
    lengths = [rng.choice([1, 2, 17, 33, 64, 65, 97, 130]) for _ in range(rng.randint(2, 5))]
    return top, rng.choice([16, 16, 32, 64]), lengths
