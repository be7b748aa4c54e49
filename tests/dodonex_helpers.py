"""Small Dodonex models with random weights for tests/test_dodonex*.py."""
import torch

from mirage.mpk.models.dodonex.builder import DodonexConfig


def latent(heads, dim, rot, vdim, q_rank, kv_rank, ff, base=3000.0, scale=None, kv_from=None, limit=1.2):
    m = {"heads": heads, "dim": dim, "rot_dim": rot, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank, "rot": {"base": base, "dims": rot},
         "scale": 2.0 / (dim + rot) ** 0.5 if scale is None else scale}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "latent_attention", "mixer": m, "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def delta(heads, dim, low_rank, ff, limit=0.8):
    return {"type": "general_delta", "mixer": {"heads": heads, "dim": dim, "low_rank": low_rank},
            "mlp": None if ff is None else {"kind": "dense", "ff": ff, "limit": limit}}


def config(layers, width, vocab, groups=4, mult=0.7, eps=1e-4, emb=3.0, logit=0.6, side=20):
    return {"architecture": "Dodonex", "vocab": vocab, "width": width, "norm": {"eps": eps, "groups": groups}, "residual_mult": mult, "embedding": {"scale": emb},
            "logit_scale": logit, "token_side": {"dim": side}, "layers": layers}


# sizes that are powers of two; sizes that nothing divides, layers that differ from each other, layers without a feed-forward,
# one latent read by several layers; wide heads and latents
CONFIGS = {
    "even": config([latent(4, 32, 16, 32, 64, 64, 128), delta(4, 32, 32, 128)], 128, 320, groups=1),
    "odd": config([delta(3, 20, 12, 75), latent(5, 24, 12, 20, 44, 36, None), delta(2, 72, 40, None), latent(9, 40, 12, 28, 30, 36, 50, kv_from=1, scale=0.5),
                   latent(2, 16, 6, 8, 17, 22, 90, base=90.0)], 84, 133, groups=3, mult=1.3, emb=1.0, logit=2.0, side=7),
    "wide": config([latent(3, 160, 96, 136, 200, 320, 192), delta(2, 128, 96, 64), latent(2, 96, 96, 200, 96, 320, 64, kv_from=0)], 320, 257, groups=5, side=70),
    "deep_state": config([delta(1, 200, 33, 64), delta(5, 64, 20, None)], 192, 99, groups=2, mult=1.0, logit=1.0, side=33),
}


def weights(cfg, seed=0):
    """bf16-valued weights under their checkpoint names; norm weights and offsets away from their neutral values."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in DodonexConfig.from_dict(cfg).tensor_shapes().items():
        t = torch.randn(shape, generator=g)
        if len(shape) == 2:
            t = t / shape[1] ** 0.5 if name not in ("embed", "side.embed") else t
        elif name.endswith(".w0"):
            t = t - 3.0  # slow decay: a state that remembers
        elif name.endswith(".a.b"):
            t = 0.5 * t
        else:
            t = 1.0 + 0.3 * t
        out[name] = t.to(torch.bfloat16)
    return out


def prompt(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()
