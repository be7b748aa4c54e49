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
                   latent(2, 16, 6, 8, 17, 22, 90, base=90.0)], 84, 133, groups=3, mult=1.3, emb=1.0, logit=2.0, side=23),
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


class LatentRig:
    """latent_prep_layer (appends the caller's rows) and latent_attention_layer over caller-written queries."""

    def __init__(self, H, R, rot, dtype, rows=64, slots=4, pages=14, page=64, base=500.0, scale=None, eps=1e-5):
        import mirage as mi
        from helpers import make_meta
        from mirage.mpk.models.checkpoint import rotary_tables_f32
        from mirage.mpk.persistent_kernel import latent_row_dim, operand_row
        kw = operand_row(dtype)
        self.H, self.R, self.rot, self.dtype, self.page, self.eps, self.base, self.scale = H, R, rot, dtype, page, eps, base, scale or 1.5 / (R + rot) ** 0.5
        self.Rp = -(-R // kw) * kw
        self.meta = make_meta(slots, pages * page, rows, slots, pages)
        self.pk = pk = mi.PersistentKernel(
            mode="onepass", world_size=1, mpi_rank=0, num_workers=mi.get_configurations_from_gpu(0)[0], num_local_schedulers=0, num_remote_schedulers=0,
            max_seq_length=pages * page, max_num_batched_requests=slots, max_num_batched_tokens=rows, max_num_pages=pages, page_size=page, meta_tensors=self.meta,
            max_tokens_per_request=min(rows, 64))
        up = lambda n, m: -(-n // m) * m
        self.qc, self.cc, self.rc = 8, 8 + 24, 8 + 24 + up(R, 16)
        new = lambda c: torch.zeros(rows, c, dtype=dtype, device="cuda")
        self.rows_in, self.cq, self.q, self.ql, self.out = new(self.rc + up(rot, 16)), new(32), new(H * (8 + up(rot, 8))), new(H * self.Rp), new(H * self.Rp)
        self.hs = 8 + up(rot, 8)
        self.cache = torch.full((pages, page, latent_row_dim(R, rot, dtype)), float("nan"), dtype=dtype, device="cuda")  # nothing of it may show
        g = torch.Generator().manual_seed(9)
        self.wq, self.wc = 1 + 0.2 * torch.randn(20, generator=g), 1 + 0.2 * torch.randn(R, generator=g)
        pad4 = lambda v: torch.nn.functional.pad(v, (0, -len(v) % 4)).cuda()
        a, cos, sin = pk.attach_input, None, None
        if rot:
            self.tables = rotary_tables_f32(rot, base, None, pages * page)
            cos, sin = a(self.tables[0], "cos"), a(self.tables[1], "sin")
        cache, q = a(self.cache, "cache"), a(self.q, "q")
        self.keep = (pad4(self.wq), pad4(self.wc))
        pk.latent_prep_layer(a(self.rows_in, "rows"), a(self.keep[0], "wq"), a(self.cq, "cq"), self.qc, 20, eps, cache=cache, latent_weight=a(self.keep[1], "wc"), cos=cos,
                             sin=sin, latent_column=self.cc, latent_rank=R, rot_column=self.rc, rot_dims=rot)
        pk.latent_attention_layer(q, a(self.ql, "ql"), cache, cos, sin, a(self.out, "out"), H, R, rot, self.hs, 8, self.scale)
        pk.compile()

    def data(self, n, seed):
        """(query latents [n, H, R], rotated query parts [n, H, rot], key latents [n, R], rotated key parts [n, rot], query latent rows [n, 20])."""
        g = torch.Generator().manual_seed(seed)
        return [torch.randn(n, *s, generator=g).to(self.dtype).double() for s in ((self.H, self.R), (self.H, self.rot), (self.R,), (self.rot,), (20,))]

    def run(self, entries):
        """entries: (slot, first position, data rows, page list).  Returns (attention rows, query latents) of each entry."""
        idx, ptr, slots, pos, at = [], [0], [], [], 0
        self.out.fill_(7.0)
        for i, (_, p0, (ql, qr, c, kr, cq), pages) in enumerate(entries):
            n = len(c)
            put = lambda dst, lo, src: dst[at:at + n, lo:lo + src.shape[1]].copy_(src.to(self.dtype))
            put(self.rows_in, self.qc, cq)
            put(self.rows_in, self.cc, c)
            put(self.rows_in, self.rc, kr)
            for h in range(self.H):
                put(self.ql, h * self.Rp, ql[:, h])
                put(self.q, h * self.hs + 8, qr[:, h])
            idx += pages
            ptr.append(len(idx))
            slots += [i] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.meta["paged_kv_indices_buffer"][:len(idx)] = torch.tensor(idx, dtype=torch.int32, device="cuda")
        self.meta["paged_kv_indptr_buffer"][:len(ptr)] = torch.tensor(ptr, dtype=torch.int32, device="cuda")
        self.pk.run_once(slots, pos)
        o, cq, out, at = self.out.cpu().double().view(-1, self.H, self.Rp)[:, :, :self.R], self.cq.cpu().double()[:, :20], [], 0
        for _, _, d, _ in entries:
            out.append((o[at:at + len(d[2])], cq[at:at + len(d[2])]))
            at += len(d[2])
        return out

    def reference(self, d):
        from oracle.dodonex_ref import latent_attention_core, rms_norm, rotate_half
        ql, qr, c, kr, cq = d
        r = lambda t: t.to(self.dtype).double()
        pos, eye = torch.arange(len(c)), torch.eye(self.R, dtype=torch.float64).expand(self.H, -1, -1)
        if self.rot:
            qr, kr = rotate_half(qr, pos, self.base), rotate_half(kr, pos, self.base)
        cn = r(rms_norm(c, self.wc.double(), self.eps))
        return latent_attention_core(ql, r(qr), cn, r(kr), eye, eye, pos, self.scale), rms_norm(cq, self.wq.double(), self.eps)


class DeltaRig:
    """general_delta_layer over caller-written rows; state slots are the batch slots unless the caller permutes them."""

    def __init__(self, H, D, rank, dtype, rows=64, slots=4, eps=1e-5, w0=-3.0):
        import mirage as mi
        from helpers import make_meta
        from mirage.mpk.persistent_kernel import operand_row, operand_tiles
        kw = operand_row(dtype)
        self.H, self.D, self.rank, self.dtype, self.eps = H, D, rank, dtype, eps
        self.Dp, self.rp = -(-D // 16) * 16, -(-rank // kw) * kw
        n = H * self.Dp
        self.meta = make_meta(slots, 512, rows, slots, 8 * slots)
        self.pk = pk = mi.PersistentKernel(
            mode="onepass", world_size=1, mpi_rank=0, num_workers=mi.get_configurations_from_gpu(0)[0], num_local_schedulers=0, num_remote_schedulers=0,
            max_seq_length=512, max_num_batched_requests=slots, max_num_batched_tokens=rows, max_num_pages=8 * slots, page_size=64, meta_tensors=self.meta,
            max_tokens_per_request=min(rows, 64))
        g = torch.Generator().manual_seed(H * D)
        self.w2 = (torch.randn(H, D, rank, generator=g) / rank ** 0.5).to(dtype)
        self.w0, self.ab, self.nw = w0 + torch.randn(H, D, generator=g), 0.5 * torch.randn(H, D, generator=g), 1 + 0.3 * torch.randn(H, D, generator=g)
        pad = lambda t: torch.nn.functional.pad(t, (0, self.Dp - D)).reshape(-1).cuda()
        self.rows_in = torch.zeros(rows, 5 * n + self.rp + 16, dtype=dtype, device="cuda")
        self.out = torch.zeros(rows, n, dtype=dtype, device="cuda")
        self.state = torch.full((slots, H, self.Dp, self.Dp), float("nan"), device="cuda")  # a request begins from zero whatever is there
        self.state_slots = torch.arange(slots, dtype=torch.int32, device="cuda")
        a = pk.attach_input
        self.keep = [operand_tiles(torch.nn.functional.pad(self.w2, (0, 0, 0, self.Dp - D)).reshape(1, n, rank)).cuda(), pad(self.w0), pad(self.ab), pad(self.nw)]
        pk.general_delta_layer(a(self.rows_in, "rows"), *(a(t, f"w{i}") for i, t in enumerate(self.keep)), a(self.state, "state"), a(self.state_slots, "slots"),
                               pk.new_tensor((rows, 2 * n), dtype=mi.float32, name="work"), a(self.out, "out"), H, D, self.rp, tuple(i * n for i in range(6)), eps)
        pk.compile()

    def data(self, n, seed):
        """Rows r, k, v, gate, a [n, H, D] and the low-rank projection [n, rank].  (r leans towards k: the norm behind the
        recurrence would magnify the rounding of an output that cancels to nearly nothing.)"""
        g = torch.Generator().manual_seed(seed)
        d = [torch.randn(n, self.H, self.D, generator=g) for _ in range(5)] + [torch.randn(n, self.rank, generator=g)]
        d[0] += d[1]
        return [t.to(self.dtype).double() for t in d]

    def run(self, entries):
        """entries: (batch slot, first position, data rows).  Returns the output rows of each entry."""
        slots, pos, at = [], [], 0
        for slot, p0, d in entries:
            n = len(d[0])
            for i in range(5):
                self.rows_in[at:at + n, i * self.H * self.Dp:(i + 1) * self.H * self.Dp].view(n, self.H, self.Dp)[:, :, :self.D] = d[i].to(self.dtype).cuda()
            self.rows_in[at:at + n, 5 * self.H * self.Dp:5 * self.H * self.Dp + self.rank] = d[5].to(self.dtype).cuda()
            slots += [slot] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.out.fill_(7.0)
        self.pk.run_once(slots, pos)
        o, out, at = self.out.cpu().double().view(-1, self.H, self.Dp)[:, :, :self.D], [], 0
        for _, _, d in entries:
            out.append(o[at:at + len(d[0])])
            at += len(d[0])
        return out

    def reference(self, d):
        from oracle.dodonex_ref import decay, delta_scan, rms_norm
        r, k, v, gate, a, low = d
        n = len(r)
        w = decay(torch.einsum("tr,hdr->thd", torch.tanh(low), self.w2.double()) + self.w0.double())
        S, o = delta_scan(torch.zeros(self.H, self.D, self.D, dtype=torch.float64), r, w, torch.sigmoid(a + self.ab.double()), k, v)
        return rms_norm(o, torch.ones(self.D, dtype=torch.float64), self.eps) * self.nw.double() * torch.sigmoid(gate)

    def close(self):
        self.pk.finalize()
