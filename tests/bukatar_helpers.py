"""Small Bukatar models with random weights for tests/test_bukatar*.py."""
import torch

from mirage.mpk.models.bukatar.builder import BukatarConfig


def dense(ff):
    return {"kind": "dense", "ff": ff}


def moe(experts, top, ff, shared):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": {"ff": shared}}


def window(heads, kv_heads, dim, rot, size, keep_first, mlp, base=700.0, scale=None):
    return {"type": "attention", "mlp": mlp,
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": base, "dims": rot}, "scale": 1.5 / dim ** 0.5 if scale is None else scale,
                      "mask": {"size": size, "keep_first": keep_first}}}


def latent(heads, dim, rot, vdim, kv_rank, mlp, base=3000.0, scale=None, kv_from=None):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot}, "scale": 2.0 / (dim + rot) ** 0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": mlp}


def scan(inner, state, conv, dt_rank, mlp):
    return {"type": "mamba1", "mixer": {"inner": inner, "state": state, "conv": conv, "dt_rank": dt_rank}, "mlp": mlp}


def config(layers, width, vocab, eps=1e-5):
    return {"architecture": "Bukatar", "vocab": vocab, "width": width, "norm": {"eps": eps}, "layers": layers}


# sizes that are powers of two; sizes that nothing divides, layers that differ from each other, layers without a feed-forward, one latent
# read by several layers; wide heads, latents and states, many experts
CONFIGS = {
    "even": config([window(4, 2, 32, 16, 48, 8, dense(128)), scan(128, 16, 4, 16, moe(8, 2, 64, 64)), latent(4, 32, 16, 32, 64, dense(128))], 128, 320),
    "odd": config([scan(75, 11, 3, 5, None), latent(5, 24, 12, 20, 44, moe(5, 3, 20, 37)), window(6, 2, 20, 12, 33, 5, dense(75), base=90.0), window(3, 3, 24, 24, 70, 0, None),
                   latent(3, 16, 12, 28, 44, dense(50), kv_from=1, scale=0.4), scan(90, 37, 6, 33, moe(6, 1, 50, 18)), window(5, 1, 28, 4, 2, 1, moe(3, 3, 40, 70))], 84, 133),
    "wide": config([window(4, 1, 160, 96, 130, 40, moe(70, 6, 33, 100)), latent(3, 160, 96, 136, 320, dense(192)), scan(200, 70, 2, 70, dense(64)), latent(2, 96, 96, 200, 320, None, kv_from=1),
                    scan(64, 200, 1, 8, None)], 320, 257, eps=1e-3),
}


def weights(cfg, seed=0):
    """bf16-valued weights under their checkpoint names; norm weights and offsets away from their neutral values."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in BukatarConfig.from_dict(cfg).tensor_shapes().items():
        t = torch.randn(shape, generator=g)
        if name.endswith(".A_log"):
            t = 0.5 * t  # rates around one: with the small steps below a state that remembers
        elif name.endswith(".dt.b"):
            t = t - 4.0
        elif name.endswith(".b"):
            t = 0.3 * t
        elif name.endswith(".router"):
            t = 3.0 * t / shape[1] ** 0.5  # choices that rounding does not change
        elif len(shape) == 2:
            t = t / shape[1] ** 0.5 if name != "embed" else t
        else:
            t = 1.0 + 0.3 * t
        out[name] = t.to(torch.bfloat16)
    return out


def prompt(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
