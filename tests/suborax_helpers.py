"""Small Suborax models with random weights, and a paged-attention rig, for tests/test_suborax*.py."""
import torch

import mirage as mi
from helpers import make_meta
from mirage.mpk.models.checkpoint import rotary_tables_f32
from mirage.mpk.models.suborax.builder import SuboraxConfig
from mirage.mpk.persistent_kernel import flex_cache_dims

SCALING = {"factor": 4.0, "low": 1.0, "high": 3.0, "original": 256}


def layer(heads, kv_heads, dim, vdim, rot, ff, base=5000.0, scaling=SCALING, scale=None, softcap=15.0):
    return {"type": "attention", "mlp": None if ff is None else {"kind": "dense", "ff": ff},
            "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 2.5 / dim ** 0.5 if scale is None else scale, "softcap": softcap,
                      "rot": {"base": base, "dims": rot, **({"scaling": scaling} if scaling else {})}}}


def config(layers, width, vocab, alpha=1.7, eps=1e-5, emb=0.7):
    return {"architecture": "Suborax", "vocab": vocab, "width": width, "norm": {"eps": eps}, "postln_alpha": alpha, "embedding": {"scale": emb}, "layers": layers}


# sizes that are powers of two, sizes that nothing divides, and layers that differ from each other
CONFIGS = {
    "even": config([layer(8, 2, 64, 64, 32, 192), layer(8, 2, 64, 64, 32, 192)], 128, 320),
    "odd": config([layer(5, 1, 40, 24, 12, 75, scaling=None), layer(6, 3, 72, 88, 72, None, softcap=4.0), layer(20, 1, 16, 8, 2, 33, base=100.0)], 84, 133, alpha=0.9, emb=3.0),
    "wide_heads": config([layer(2, 2, 160, 200, 64, 64), layer(4, 1, 256, 144, 10, 100)], 320, 257, alpha=1.0, emb=1.0),
    "one_layer": config([layer(7, 7, 32, 48, 32, 130, scale=1.0, softcap=30.0)], 70, 99, alpha=3.0, eps=1e-3),
}


def weights(cfg, seed=0):
    """bf16-valued weights under their checkpoint names; norm weights and sinks away from their neutral values."""
    g = torch.Generator().manual_seed(seed)
    out = {}
    for name, shape in SuboraxConfig.from_dict(cfg).tensor_shapes().items():
        t = torch.randn(shape, generator=g)
        if len(shape) == 2:
            t = t / shape[1] ** 0.5 if name != "embed" else t
        elif name.endswith("sink"):
            t = 5.0 + t
        else:
            t = 0.3 * t
        out[name] = t.to(torch.bfloat16)
    return out


def prompt(cfg, n, seed=0):
    return torch.randint(0, cfg["vocab"], (n,), generator=torch.Generator().manual_seed(seed)).tolist()



class AttentionRig:
    """A graph of one flex_attention_layer over caller-written q/k/v rows, with page tables the test chooses."""

    def __init__(self, H, G, D, DV, rot, scale, softcap, unit_norm=True, sink=None, dtype=torch.bfloat16, rows=64, slots=4, pages=24, page=32, base=1000.0, scaling=SCALING,
                 eps=1e-5):
        self.dims, self.dtype, self.page, self.rows = (H, G, D, DV), dtype, page, rows
        self.max_seq = pages * page
        meta = make_meta(slots, self.max_seq, rows, slots, pages)
        self.pk = pk = mi.PersistentKernel(
            mode="onepass", world_size=1, mpi_rank=0, num_workers=mi.get_configurations_from_gpu(0)[0], num_local_schedulers=0, num_remote_schedulers=0,
            max_seq_length=self.max_seq, max_num_batched_requests=slots, max_num_batched_tokens=rows, max_num_pages=pages, page_size=page, meta_tensors=meta,
            max_tokens_per_request=min(rows, 64))
        self.meta = meta
        cols = H * D + G * (D + DV)
        self.qkv = torch.zeros(rows, cols, dtype=dtype, device="cuda")
        self.out = torch.zeros(rows, H * DV, dtype=dtype, device="cuda")
        dk, dv = flex_cache_dims(D, DV, dtype)
        # a cache full of garbage: nothing of it may show
        self.k = torch.full((pages, page, G, dk), 3.0e4, dtype=dtype, device="cuda")
        self.v = torch.full((pages, page, G, dv), float("nan"), dtype=dtype, device="cuda")
        if dk != D:
            self.k.zero_()  # (padding dims are part of the operands and start out as zeros)
        if dv != DV:
            self.v.zero_()
        E = mi.bfloat16 if dtype == torch.bfloat16 else mi.float32
        a = pk.attach_input
        cos = sin = None
        if rot:
            c, s = rotary_tables_f32(rot, base, scaling, self.max_seq)
            self.keep = (c, s)
            cos, sin = a(c, "cos"), a(s, "sin")
        self.sink = sink
        pk.flex_attention_layer(a(self.qkv, "qkv"), a(self.k, "k"), a(self.v, "v"), cos, sin, None if sink is None else a(sink.cuda(), "sink"),
                                pk.new_tensor((rows, H * dk), dtype=E, name="qw"), a(self.out, "out"), H, G, D, DV, rot, scale, softcap, unit_norm, eps)
        pk.compile()
        self.args = dict(rot={"dims": rot, "base": base, **({"scaling": scaling} if scaling else {})}, scale=scale, cap=softcap, unit_norm=unit_norm, eps=eps)
        self.tables = {}

    def run(self, entries):
        """entries: (slot, first position, rows [n, cols] on the CPU, page list).  Returns the output rows of each entry."""
        idx, ptr, slots, pos, at = [], [0], [], [], 0
        for i, (slot, p0, rows, pages) in enumerate(entries):
            self.qkv[at:at + len(rows)] = rows.to(self.dtype).cuda()
            idx += pages
            ptr.append(len(idx))
            slots += [i] * len(rows)
            pos += list(range(p0, p0 + len(rows)))
            at += len(rows)
        self.meta["paged_kv_indices_buffer"][:len(idx)] = torch.tensor(idx, dtype=torch.int32, device="cuda")
        self.meta["paged_kv_indptr_buffer"][:len(ptr)] = torch.tensor(ptr, dtype=torch.int32, device="cuda")
        self.out.fill_(7.0)
        self.pk.run_once(slots, pos)
        got, out, at = self.out.cpu().double(), [], 0
        for _, _, rows, _ in entries:
            out.append(got[at:at + len(rows)])
            at += len(rows)
        return out

    def reference(self, rows):
        """The oracle's attention over all rows of one request (float64, fed with the rows as the kernel stores them)."""
        from oracle.suborax_ref import attention_core, rms_divide, rotate
        H, G, D, DV = self.dims
        x = rows.to(self.dtype).double()
        T = len(x)
        pos = torch.arange(T)
        q, k, v = x[:, :H * D].view(T, H, D), x[:, H * D:(H + G) * D].view(T, G, D), x[:, (H + G) * D:].view(T, G, DV)
        if self.args["rot"]["dims"]:
            q, k = rotate(q, pos, self.args["rot"]), rotate(k, pos, self.args["rot"])
        if self.args["unit_norm"]:
            q, k = rms_divide(q, self.args["eps"]), rms_divide(k, self.args["eps"])
        r = lambda t: t.to(self.dtype).double()
        sink = torch.full((H,), float("-inf"), dtype=torch.float64) if self.sink is None else self.sink.double()
        return attention_core(r(q), r(k), v, pos, sink, self.args["scale"], self.args["cap"]).reshape(T, H * DV)

    def close(self):
        self.pk.finalize()
