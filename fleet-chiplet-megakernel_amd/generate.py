"""Greedy generation with any registered model, from a checkpoint directory or with random weights of a named shape.

    python generate.py --model-path DIR --prompt-ids 5,17,3 --prompt-ids 8,9 --max-new-tokens 32
    python generate.py --random suborax-8b --layers 4 --batch 8 --prompt-length 80 --max-new-tokens 64

The model class is chosen by the checkpoint's config.json.  `--engine offline` (default) runs the whole generation in one
persistent launch with the on-GPU scheduler; `--engine serving` runs the host loop of mirage.mpk.ServingSession.
"""
import argparse
import json
import os
import time

import torch

from mirage.mpk import MPK, MirageModelConfig, MPKMetadata, ServingSession
from mirage.mpk.models import bukatar, dodonex, suborax, vizonex


def suborax_shape(width=4096, heads=32, kv_heads=8, dim=128, vdim=128, ff=12288, layers=36, vocab=151936) -> dict:
    """A Suborax config.json of the given sizes, every layer alike, half of each head rotated."""
    layer = {"type": "attention", "mlp": {"kind": "dense", "ff": ff},
             "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5, "softcap": 50.0,
                       "rot": {"base": 5e5, "dims": dim // 2, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 8192}}}}
    return {"architecture": "Suborax", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "postln_alpha": 1.5, "embedding": {"scale": 1.0},
            "layers": [layer] * layers}


def dodonex_shape(width=4096, heads=32, dim=128, rot_dim=64, vdim=128, q_rank=1536, kv_rank=512, delta_heads=32, delta_dim=128, low_rank=128, ff=12288, side=256, layers=36,
                  vocab=151936) -> dict:
    """A Dodonex config.json of the given sizes, latent attention and delta rule by turns."""
    mlp = {"kind": "dense", "ff": ff, "limit": 7.0}
    latent = {"type": "latent_attention", "mlp": mlp, "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "q_rank": q_rank, "kv_rank": kv_rank,
                                                               "rot": {"base": 5e5, "dims": rot_dim}, "scale": (dim + rot_dim) ** -0.5}}
    delta = {"type": "general_delta", "mlp": mlp, "mixer": {"heads": delta_heads, "dim": delta_dim, "low_rank": low_rank}}
    return {"architecture": "Dodonex", "vocab": vocab, "width": width, "norm": {"eps": 1e-6, "groups": 4}, "residual_mult": 1.0, "embedding": {"scale": 1.0}, "logit_scale": 1.0,
            "token_side": {"dim": side}, "layers": [delta if i % 2 else latent for i in range(layers)]}


def bukatar_shape(width=4096, heads=32, kv_heads=8, dim=128, window=1024, keep_first=64, rot_dim=64, vdim=128, kv_rank=512, inner=8192, state=16, dt_rank=256, ff=12288, experts=64,
                  top=8, expert_ff=1536, layers=36, vocab=151936) -> dict:
    """A Bukatar config.json of the given sizes: windowed attention, latent attention and two scans by turns, dense and expert
    feed-forwards by turns."""
    dense = {"kind": "dense", "ff": ff}
    moe = {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": expert_ff}, "shared": {"ff": expert_ff}}
    att = {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "rot": {"base": 5e5, "dims": dim // 2}, "scale": dim ** -0.5,
                                          "mask": {"size": window, "keep_first": keep_first}}}
    lat = {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "rot": {"base": 5e5, "dims": rot_dim},
                                                 "scale": (dim + rot_dim) ** -0.5}}
    ssm = {"type": "mamba1", "mixer": {"inner": inner, "state": state, "conv": 4, "dt_rank": dt_rank}}
    cycle = [dict(att, mlp=dense), dict(lat, mlp=moe), dict(ssm, mlp=dense), dict(ssm, mlp=moe)]
    return {"architecture": "Bukatar", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "layers": [cycle[i % 4] for i in range(layers)]}


def vizonex_shape(width=4096, heads=32, kv_heads=8, dim=128, chunk=1024, dual_heads=64, dual_dim=128, state=128, groups=8, ff=12288, experts=64, top=8, expert_groups=8, expert_groups_kept=4,
                  expert_ff=1536, layers=36, vocab=151936, positions=32768) -> dict:
    """A Vizonex config.json of the given sizes: chunked attention and recurrence by turns, dense and expert feed-forwards by turns."""
    dense = {"kind": "dense", "ff": ff}
    moe = {"kind": "moe", "router": {"experts": experts, "top": top, "groups": {"count": expert_groups, "keep": expert_groups_kept}, "scale": 2.5},
           "expert": {"ff": expert_ff, "limit": 7.0}, "shared": {"ff": expert_ff, "limit": 7.0}}
    att = {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5, "mask": {"size": chunk}}}
    ssm = {"type": "mamba2", "mixer": {"heads": dual_heads, "vdim": dual_dim, "state": state, "groups": groups, "norm_groups": groups, "conv": 4}}
    cycle = [dict(att, mlp=dense), dict(ssm, mlp=moe), dict(ssm, mlp=dense), dict(att, mlp=moe)]
    return {"architecture": "Vizonex", "vocab": vocab, "width": width, "norm": {"eps": 1e-6}, "canon": {"taps": 4}, "max_positions": positions, "layers": [cycle[i % 4] for i in range(layers)]}


# name -> (config.json of a shape, its sizes)
SHAPES = {"suborax-8b": (suborax_shape, {}), "suborax-2k": (suborax_shape, dict(width=2048, heads=32, kv_heads=4, ff=6144)),
          "dodonex-8b": (dodonex_shape, {}), "dodonex-2k": (dodonex_shape, dict(width=2048, heads=16, q_rank=768, delta_heads=32, delta_dim=64, low_rank=64, ff=6144)),
          "bukatar-8b": (bukatar_shape, {}), "bukatar-2k": (bukatar_shape, dict(width=2048, heads=16, kv_heads=4, inner=4096, dt_rank=128, ff=6144, experts=128, expert_ff=768)),
          "vizonex-8b": (vizonex_shape, {}), "vizonex-2k": (vizonex_shape, dict(width=2048, heads=16, kv_heads=4, dual_heads=32, ff=6144, experts=128, expert_ff=768))}


def random_model(config: dict):
    """(MirageModelConfig with random-init weights, the reader's form of the config) of a parsed config.json."""
    kind, module = {"Suborax": (suborax.SuboraxConfig, suborax), "Dodonex": (dodonex.DodonexConfig, dodonex), "Bukatar": (bukatar.BukatarConfig, bukatar),
                    "Vizonex": (vizonex.VizonexConfig, vizonex)}[config["architecture"]]
    sizes = kind.from_dict(config)
    return MirageModelConfig(architecture=config, state_dict=module.random_state_dict(sizes)), sizes


class Generator:
    """An MPK in offline mode with its request table: `generate(prompts)` runs every prompt to its new tokens (or EOS)."""

    def __init__(self, max_seq_length: int, model_path: str = None, model_config: MirageModelConfig = None, batch: int = 1, max_num_batched_tokens: int = None,
                 max_tokens_per_request: int = None, page_size: int = 4096, total_requests: int = None, eos_token_id: int = None, dtype=torch.bfloat16,
                 **meta):
        pages_per_req = -(-max_seq_length // page_size)
        self.max_seq = max_seq_length
        self.model = MPK(MPKMetadata(
            mode="offline", total_num_requests=total_requests or batch, max_seq_length=max_seq_length, max_num_batched_requests=batch,
            max_num_batched_tokens=max_num_batched_tokens or batch, max_num_pages=batch * pages_per_req, page_size=page_size,
            weight_from_model=model_path is not None, model_path=model_path, model_config=model_config, eos_token_id=eos_token_id,
            max_tokens_per_request=max_tokens_per_request, dtype=dtype, tokens=torch.zeros(total_requests or batch, max_seq_length, dtype=torch.int64, device="cuda"),
            **meta))
        self.model.build()
        self.model.compile()
        self.mpk = self.model.persistent_kernel
        self.meta = self.mpk.meta_tensors

    def load_prompts(self, prompts):
        assert len(prompts) <= self.mpk.total_num_requests
        tokens = torch.zeros(self.mpk.total_num_requests, self.max_seq, dtype=torch.int64)
        lengths = torch.zeros(self.mpk.total_num_requests, dtype=torch.int32)
        for i, p in enumerate(prompts):
            assert 0 < len(p) < self.max_seq
            tokens[i, :len(p)] = torch.as_tensor(p)
            lengths[i] = len(p)
        self.meta["tokens"].copy_(tokens)
        self.meta["prompt_lengths"].copy_(lengths)
        torch.cuda.synchronize()
        self.mpk.init_request_resources()

    def generate(self, prompts, max_new_tokens: int = None):
        self.load_prompts(prompts)
        self.model()
        torch.cuda.synchronize()
        steps, tokens = self.meta["step"].tolist(), self.meta["tokens"].cpu()
        limit = lambda p: self.max_seq if max_new_tokens is None else len(p) + max_new_tokens
        return [tokens[i, :min(steps[i] + 1, limit(p))].tolist() for i, p in enumerate(prompts)]

    def logits(self):
        return self.model.model_builder.logits.to_torch()

    def finalize(self):
        self.model.finalize()


def main(argv=None):
    ap = argparse.ArgumentParser(description="Greedy generation on the MI355X persistent megakernel")
    src = ap.add_mutually_exclusive_group(required=True)
    src.add_argument("--model-path", help="checkpoint directory (config.json + *.safetensors)")
    src.add_argument("--random", choices=sorted(SHAPES), help="random-init weights of this shape")
    ap.add_argument("--layers", type=int, default=None, help="with --random: number of layers")
    ap.add_argument("--dtype", choices=["bfloat16", "float32"], default="bfloat16")
    ap.add_argument("--engine", choices=["offline", "serving"], default="offline")
    ap.add_argument("--prompt-ids", action="append", default=[], help="token ids with commas between them; once per prompt")
    ap.add_argument("--batch", type=int, default=None, help="live requests (default: one per prompt, at most 64)")
    ap.add_argument("--prompt-length", type=int, default=80, help="length of the random prompts used when no --prompt-ids are given")
    ap.add_argument("--max-new-tokens", type=int, default=32)
    ap.add_argument("--max-num-batched-tokens", type=int, default=None, help="token rows per iteration (default 64, or 1 for a single request of one token)")
    ap.add_argument("--page-size", type=int, default=64)
    ap.add_argument("--eos-token-id", type=int, default=None)
    args = ap.parse_args(argv)
    dtype = getattr(torch, args.dtype)
    if args.model_path:
        with open(os.path.join(args.model_path, "config.json")) as f:
            cfg = json.load(f)
        vocab, source = cfg.get("vocab") or cfg["vocab_size"], dict(model_path=args.model_path)
    else:
        make, shape = SHAPES[args.random]
        cfg = make(**shape, **({"layers": args.layers} if args.layers else {}))
        vocab, source = cfg["vocab"], dict(model_config=random_model(cfg)[0])
    prompts = [[int(x) for x in p.split(",")] for p in args.prompt_ids]
    if not prompts:
        prompts = [torch.randint(0, vocab, (args.prompt_length,), generator=torch.Generator().manual_seed(r)).tolist() for r in range(args.batch or 1)]
    batch = min(args.batch or len(prompts), 64)
    longest = max(len(p) for p in prompts) + args.max_new_tokens
    rows = args.max_num_batched_tokens or 64
    if args.engine == "serving":
        pages = -(-longest // args.page_size)
        s = ServingSession.open(dtype=dtype, max_tokens=batch * pages * args.page_size, max_requests=batch, page_size=args.page_size, max_rows=rows, **source)
        t0 = time.perf_counter()
        out = s.generate(prompts, args.max_new_tokens, -1 if args.eos_token_id is None else args.eos_token_id)
        what = "host-driven passes"
    else:
        s = Generator(longest + 1, batch=batch, max_num_batched_tokens=rows, max_tokens_per_request=min(rows, 64), page_size=args.page_size,
                      total_requests=len(prompts), eos_token_id=args.eos_token_id, dtype=dtype, **source)
        torch.cuda.synchronize()
        t0 = time.perf_counter()
        out = s.generate(prompts, args.max_new_tokens)
        what = f"{s.mpk.stats()['iterations']} iterations in one launch"
    dt = time.perf_counter() - t0
    for i, ids in enumerate(out):
        print(f"{i}: " + " ".join(str(t) for t in ids[len(prompts[i]):]))
    n = sum(len(o) - len(p) for o, p in zip(out, prompts))
    print(f"{n} new tokens for {len(prompts)} prompts in {dt * 1e3:.1f} ms ({what})")
    s.finalize()


if __name__ == "__main__":
    main()
