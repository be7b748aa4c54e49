"""Small Vizonex models with random weights for tests/test_vizonex*.py."""
import torch

from mirage.mpk.models.vizonex.builder import VizonexConfig


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, count, keep, ff, shared, scale=1.7, limit=2.0, shared_limit=1.2):
    return {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": count, "keep": keep}, "scale": scale}, "expert": {"ff": ff, "limit": limit},
            "shared": None if shared is None else {"ff": shared, "limit": shared_limit}}


def chunked(heads, kv_heads, dim, vdim, size, mlp, scale=None):
    return {"type": "attention", "mlp": mlp, "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 1.3 / dim ** 0.5 if scale is None else scale, "mask": {"size": size}}}


def dual(heads, vdim, state, groups, norm_groups, conv, mlp):
    return {"type": "mamba2", "mlp": mlp, "mixer": {"heads": heads, "vdim": vdim, "state": state, "groups": groups, "norm_groups": norm_groups, "conv": conv}}


def config(layers, width, vocab, eps=1e-5, taps=4, positions=600):
    return {"architecture": "Vizonex", "vocab": vocab, "width": width, "norm": {"eps": eps}, "canon": {"taps": taps}, "max_positions": positions, "layers": layers}


# sizes that are powers of two; sizes that nothing divides, values of another size than keys, layers that differ from each other, layers
# without a feed-forward or without a shared expert; wide heads and states, many experts, one tap
CONFIGS = {
    "even": config([chunked(4, 2, 32, 32, 64, dense(128)), dual(4, 32, 64, 2, 4, 4, moe(8, 2, 4, 2, 64, 64))], 128, 320),
    "odd": config([dual(3, 25, 11, 1, 5, 3, None), chunked(6, 2, 20, 28, 33, moe(6, 3, 3, 2, 20, 37)), dual(6, 14, 37, 3, 2, 6, dense(75)), chunked(3, 3, 24, 10, 70, None),
                   chunked(5, 1, 44, 36, 2, moe(9, 4, 3, 2, 50, None, scale=0.8)), dual(2, 45, 6, 2, 1, 2, moe(5, 1, 1, 1, 33, 20, limit=0.7))], 84, 133, taps=3),
    "wide": config([chunked(4, 1, 160, 200, 130, moe(72, 6, 9, 4, 33, 100)), dual(3, 100, 130, 1, 3, 2, dense(192)), chunked(4, 2, 96, 64, 0, dense(70)), dual(5, 64, 200, 5, 10, 1, None)],
                   320, 257, eps=1e-3, taps=1),
    "taps": config([dual(2, 33, 20, 2, 3, 9, dense(40)), chunked(2, 1, 16, 16, 48, None)], 60, 70, taps=7),
}


def weights(cfg, seed=None):
    """bf16-valued weights under their checkpoint names; norm weights, factors and offsets away from their neutral values.  (The "odd" model's seed is
    one whose routers have next to no near ties on the tests' prompts: a choice that rounding turns changes a request for good.)"""
    seed = (17 if cfg is CONFIGS["odd"] else 0) if seed is None else seed
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in VizonexConfig.from_dict(cfg).tensor_shapes().items():
        t = torch.randn(shape, generator=g)
        if name.endswith(".A_log"):
            t = 0.5 * t  # rates around one: with the small steps below a state that remembers
        elif name.endswith(".dt_bias"):
            t = t - 3.0
        elif name.endswith((".conv.b", ".sink")):
            t = 0.5 * t
        elif name.endswith(".correction"):
            t = 0.4 * t - 0.6  # most choice scores are negative
        elif name.endswith(".router"):
            t = 3.0 * t / shape[1] ** 0.5  # choices that rounding does not change
        elif name.endswith((".conv", ".canon1")):
            t = t / shape[1] ** 0.5
        elif len(shape) == 2:
            t = t if name == "embed" else 0.5 * t if name == "pos" else t / shape[1] ** 0.5
        else:
            t = 1.0 + 0.3 * t
        out[name] = t.to(torch.bfloat16)
    return out


def prompt(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
