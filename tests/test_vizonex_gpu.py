"""Vizonex on the GPU against the plain oracle: every mechanism alone, whole models of several sizes in bf16 and in 32 bits, prompts
against single tokens, portions, mixed batches, pages and state slots used again, chunk edges, long decoding, and greedy generation
through the framework's own entry points.  Expected values come from oracle/vizonex_ref.py in float64."""
import json

import pytest
import torch

pytestmark = pytest.mark.gpu

F64 = torch.float64
BOTH = pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])


def _session(cfg, w, dtype, max_tokens=512, **kw):
    from mirage.mpk import MirageModelConfig, ServingSession
    return ServingSession.open(model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in w.items()}), dtype=dtype, max_tokens=max_tokens, **kw)


def _oracle_logits(cfg, w, toks):
    from oracle.vizonex_ref import VizonexOracle
    orc = VizonexOracle(cfg, w)
    return orc.forward(toks, orc.new_state(), 0)


def _feed(s, rid, toks, cuts):
    """All logits of `toks`, fed to request `rid` in portions of the given sizes."""
    out, at = [], 0
    for n in cuts:
        lg, _ = s.step([(rid, toks[at:at + n])], [list(range(n))])
        out.append(lg.cpu().double())
        at += n
    assert at == len(toks)
    return torch.cat(out)


def _close(got, want, dtype, what="", bf16_outliers=0.05):
    """Logits per position.  In bf16 a router's near tie may fall the other way: a small share of positions may be off by more."""
    err = ((got - want) - (got - want).mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()
    limit = 0.04 if dtype == torch.bfloat16 else 1e-5
    over = (err > limit).nonzero().flatten()
    allowed = int(bf16_outliers * len(err)) if dtype == torch.bfloat16 else 0
    assert len(over) <= allowed and err.isfinite().all(), f"{what}: {len(over)} positions over {limit}, worst {int(err.argmax())} with {float(err.max())}; first: {over[:8].tolist()}"


def _graph(rows, slots=None, seq=64, page=64, pages=None):
    import mirage as mi
    from helpers import make_meta
    R = slots or rows
    pages = pages or 2 * R
    meta = make_meta(R, seq, rows, R, pages)
    pk = mi.PersistentKernel(mode="onepass", world_size=1, mpi_rank=0, num_workers=mi.get_configurations_from_gpu(0)[0], num_local_schedulers=0, num_remote_schedulers=0, max_seq_length=seq,
                             max_num_batched_requests=R, max_num_batched_tokens=rows, max_num_pages=pages, page_size=page, meta_tensors=meta, max_tokens_per_request=min(rows, 64))
    return pk, meta


def _tol(dtype):
    return dict(rtol=1.6e-2, atol=1.6e-2) if dtype == torch.bfloat16 else dict(rtol=2e-5, atol=2e-5)


def _E(dtype):
    import mirage as mi
    return mi.bfloat16 if dtype == torch.bfloat16 else mi.float32


# ---------------------------------------------------------------- mechanisms alone
@BOTH
def test_embedding_adds_the_position(dtype):
    pk, _ = _graph(8, 8, seq=512)
    g = torch.Generator().manual_seed(0)
    for cols in (64, 70):
        pk, _ = _graph(8, 8, seq=512)
        table, pos = torch.randn(50, cols, generator=g).to(dtype), torch.randn(300, cols, generator=g).to(dtype)
        ids, where = torch.tensor([3, 49, 0, 7, -1, 12, 3, 3]), [0, 299, 5, 63, 64, 65, 298, 1]
        up = -(-cols // 4) * 4
        t = dict(ids=ids[:, None].cuda(), table=table.cuda(), pos=pos.cuda(), r=torch.zeros(8, up, device="cuda"), o=torch.zeros(8, up, dtype=dtype, device="cuda"))
        a = {k: pk.attach_input(v, k) for k, v in t.items()}
        pk.embed_scaled_layer(a["ids"], a["table"], a["r"], a["o"], scale=1.5, positions=a["pos"])
        pk.compile()
        pk.run_once(list(range(8)), where)
        want = 1.5 * table[ids.clamp(min=0)].double() * (ids >= 0)[:, None] + pos[where].double()
        torch.testing.assert_close(t["r"][:, :cols].cpu().double(), want, rtol=1e-6, atol=1e-6)
        torch.testing.assert_close(t["o"][:, :cols].cpu().double(), want, **_tol(dtype))
        pk.finalize()


@BOTH
@pytest.mark.parametrize("rows", [1, 2, 7, 16, 40, 64])
@pytest.mark.parametrize("n,k", [(64, 64), (192, 192), (512, 2048), (256, 4096)])
def test_gelu_gated_linear(dtype, rows, n, k):
    from oracle.vizonex_ref import gelu_tanh
    g = torch.Generator().manual_seed(rows * n)
    x, w = torch.randn(rows, k, generator=g).to(dtype), [(2 * torch.randn(n, k, generator=g) / k ** 0.5).to(dtype) for _ in range(2)]
    pk, _ = _graph(64, 64)
    rows_in = torch.zeros(64, k, dtype=dtype, device="cuda")
    rows_in[:rows] = x.cuda()
    out = torch.zeros(64, n, dtype=dtype, device="cuda")
    keep = [t.cuda() for t in w]
    both = pk.shuffle_tensors(inputs=[pk.attach_input(t, f"w{i}") for i, t in enumerate(keep)], shuffled_dim=0, num_groups=1, name="w")
    mid = pk.new_tensor((64, 2 * n), dtype=_E(dtype), name="mid")
    pk.linear_layer(pk.attach_input(rows_in, "x"), both, mid, (1, 1, 1), (256, 1, 1))
    pk.gelu_mul_layer(mid, pk.attach_input(out, "o"))
    pk.compile()
    pk.run_once(list(range(rows)), [0] * rows)
    want = gelu_tanh(x.double() @ w[0].double().T) * (x.double() @ w[1].double().T)
    torch.testing.assert_close(out[:rows].cpu().double(), want, **_tol(dtype))
    assert not out[rows:].any()
    pk.finalize()


class JoinRig:
    """residual_prenorm with two summands, their factors and places, the convolution behind it and (fused) a linear."""

    def __init__(self, width, slots, taps, dtype, fused, second=True, rows=64):
        self.W, self.S, self.taps, self.dtype, self.second = width, max(slots, 1), taps, dtype, second
        self.ld = ld = -(-width // 64) * 64
        g = torch.Generator().manual_seed(width + slots + taps)
        rnd = lambda *s: torch.randn(*s, generator=g)
        self.s1, self.s2, self.w = 1 + 0.3 * rnd(width), 1 + 0.3 * rnd(width), 1 + 0.3 * rnd(width)
        self.cw, self.wl = (rnd(width, max(taps, 1)) / max(taps, 1) ** 0.5).to(dtype), (rnd(48, width) / width ** 0.5).to(dtype)
        self.pk, self.meta = pk, _ = _graph(rows, min(rows, 4), seq=256, pages=16)
        R = min(rows, 4)
        z = lambda *s, dt=dtype: torch.zeros(*s, dtype=dt, device="cuda")
        pad = lambda t: torch.nn.functional.pad(t, (0, ld - width)).cuda()
        t = dict(x=z(rows, ld, dt=torch.float32), y=z(rows, ld), y2=z(rows, self.S * ld), f=z(rows, 12, dt=torch.float32), s1=pad(self.s1), s2=pad(self.s2), w=pad(self.w), nx=z(rows, ld, dt=torch.float32),
                 h=z(rows, ld), m=z(rows, ld), lo=z(rows, 48), wl=pad(self.wl), cw=pad(self.cw.T.contiguous()), ring=z(R, max(taps, 1), ld).fill_(float("nan")),
                 slots=torch.arange(R, dtype=torch.int32, device="cuda"))
        self.t, a = t, {k: pk.attach_input(v, k) for k, v in t.items()}
        kw = dict(input2=a["y2"], factor2=a["s2"], **(dict(slot_weights=a["f"], slots=slots, slot_columns=ld) if slots else {})) if second else {}
        pk.residual_prenorm_layer(a["y"], a["x"], a["nx"], a["h"], weight=a["w"], width=width, eps=1e-4, factor=a["s1"], **kw)
        if taps:
            pk.ring_conv_layer(a["h"], a["cw"], a["ring"], a["slots"], a["m"], identity=True)
        if fused:
            pk.linear_layer(a["m"] if taps else a["h"], a["wl"], a["lo"], (1, 1, 1), (256, 1, 1))
        pk.compile()
        self.slots, self.fused = slots, fused

    def data(self, n, seed):
        g = torch.Generator().manual_seed(seed)
        rnd = lambda *s: torch.randn(*s, generator=g)
        return rnd(n, self.W), rnd(n, self.W).to(self.dtype), rnd(n, self.S, self.W).to(self.dtype), rnd(n, self.S)

    def reference(self, d):
        from oracle.vizonex_ref import causal_conv, rms_norm
        x, y, y2, f = (t.double() for t in d)
        v = x + self.s1.double() * y
        if self.second:
            v = v + self.s2.double() * ((y2 * f[..., None]).sum(1) if self.slots else y2[:, 0])
        h = rms_norm(v, self.w.double(), 1e-4)
        m = h
        if self.taps:
            hr = h.to(self.dtype).double()
            m = hr + causal_conv(hr, torch.zeros(self.taps - 1, self.W, dtype=F64), self.cw.double())[0]
        return v, h, m, m.to(self.dtype).double() @ self.wl.double().T

    def run(self, entries):
        """entries: (slot, first position, rows of data)"""
        slots, pos, at, W, ld = [], [], 0, self.W, self.ld
        for slot, p0, (x, y, y2, f) in entries:
            n = len(x)
            self.t["x"][at:at + n, :W], self.t["y"][at:at + n, :W] = x.cuda(), y.cuda()
            self.t["y2"].view(-1, self.S, ld)[at:at + n, :, :W], self.t["f"][at:at + n, :self.S] = y2.cuda(), f.cuda()
            slots += [slot] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.pk.run_once(slots, pos)
        names = ["nx", "h"] + (["m"] if self.taps and not (self.fused and at == 1 and self.dtype == torch.bfloat16) else [])  # (a single token's convolved row stays on the chip)
        return {k: self.t[k][:at, :W].cpu().double() for k in names} | ({"lo": self.t["lo"][:at].cpu().double()} if self.fused else {})


@BOTH
@pytest.mark.parametrize("fused", [False, True])
@pytest.mark.parametrize("width,slots,taps,second", [(64, 0, 4, True), (84, 3, 3, True), (84, 0, 0, False), (200, 9, 1, True), (320, 5, 7, True), (2048, 9, 4, True), (4096, 1, 4, True), (4096, 0, 2, False),
                                                     (6000, 3, 4, True)])
def test_sum_norm_and_convolution(dtype, fused, width, slots, taps, second):
    """Single tokens, portions shorter than the convolution and longer ones, mixtures; slots that are used again (their rings hold NaN at first)."""
    rig = JoinRig(width, slots, taps, dtype, fused, second)
    lens = [90, 33, 20, 7]
    data = [rig.data(n, 10 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    at, slot = [0] * 4, [2, 0, 3, 0]
    plan = [[(0, 1)], [(0, 1)], [(0, 2), (1, 1)], [(0, 1), (1, 1), (2, 1)], [(0, 40), (1, 2), (2, 3)], [(1, 1)], [(0, 1), (1, 1)], [(2, 14), (1, 27), (0, 3)], [(0, 1)], [(3, 1)], [(3, 1), (0, 1), (2, 1)],
            [(3, 5), (0, 32)], [(2, 1)]]
    for step in plan:
        got = rig.run([(slot[r], at[r], [t[at[r]:at[r] + n] for t in data[r]]) for r, n in step])
        o = 0
        for r, n in step:
            for name, g in got.items():
                w = want[r][{"nx": 0, "h": 1, "m": 2, "lo": 3}[name]][at[r]:at[r] + n]
                tol = dict(rtol=3e-5, atol=3e-5) if name == "nx" else _tol(dtype) if name == "h" else dict(rtol=3e-2, atol=4e-2) if dtype == torch.bfloat16 else dict(rtol=1e-4, atol=1e-4)
                torch.testing.assert_close(g[o:o + n], w, msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **tol)
            o, at[r] = o + n, at[r] + n
    assert at[0] == 83 and at[1:] == [33, 20, 7]
    rig.pk.finalize()


@BOTH
@pytest.mark.parametrize("fused", [False, True])
@pytest.mark.parametrize("width,groups", [(64, 1), (84, 3), (90, 6), (96, 4), (480, 5), (4096, 8), (8192, 8), (10000, 2), (4096, 64)])
def test_norm_in_parts_of_wide_rows(dtype, fused, width, groups):
    """Rows that are only normalised, in equal parts (of whole quads or not), alone and in front of a linear."""
    from oracle.vizonex_ref import rms_norm_parts
    g = torch.Generator().manual_seed(width)
    ld = -(-width // 64) * 64
    x, w, wl = torch.randn(20, width, generator=g), 1 + 0.3 * torch.randn(width, generator=g), (torch.randn(80, width, generator=g) / width ** 0.5).to(dtype)
    x *= torch.exp(torch.randn(20, groups, generator=g)).repeat_interleave(width // groups, 1)  # parts of different size
    want = rms_norm_parts(x.double(), w.double(), 1e-4, groups)
    pad = lambda t, rows=None: torch.nn.functional.pad(t, (0, ld - width)).cuda()
    for rows in (1, 20):
        pk, _ = _graph(20, 20)
        t = dict(x=pad(x), w=pad(w), o=torch.zeros(20, ld, dtype=dtype, device="cuda"), wl=pad(wl), lo=torch.zeros(20, 80, dtype=dtype, device="cuda"))
        a = {k: pk.attach_input(v, k) for k, v in t.items()}
        pk.residual_prenorm_layer(None, a["x"], None, a["o"], weight=a["w"], width=width, groups=groups, eps=1e-4)
        if fused:
            pk.linear_layer(a["o"], a["wl"], a["lo"], (1, 1, 1), (256, 1, 1))
        pk.compile()
        pk.run_once(list(range(rows)), [0] * rows)
        torch.testing.assert_close(t["o"][:rows, :width].cpu().double(), want[:rows], **_tol(dtype))
        if fused:
            torch.testing.assert_close(t["lo"][:rows].cpu().double(), want[:rows] @ wl.double().T, rtol=3e-2 if dtype == torch.bfloat16 else 1e-4, atol=3e-2 if dtype == torch.bfloat16 else 1e-4)
        pk.finalize()


class ChunkRig:
    """flex_attention_layer with chunks, norms over all heads of a row, score factors and a sink, over caller-written rows."""

    def __init__(self, H, G, D, E, size, dtype, pages=12, scale=None):
        from mirage.mpk.persistent_kernel import flex_cache_dims
        self.H, self.G, self.D, self.E, self.size, self.dtype, self.scale = H, G, D, E, size, dtype, scale or 1.3 / D ** 0.5
        self.pk, self.meta = pk, _ = _graph(64, 4, seq=pages * 64, pages=pages)
        dk, dv = flex_cache_dims(D, E, dtype)
        old = lambda d, v: torch.full((pages, 64, G, d), v, dtype=dtype, device="cuda")  # nothing of it may show
        g = torch.Generator().manual_seed(5)
        rnd = lambda *s: torch.randn(*s, generator=g)
        self.qn, self.kn, self.temp, self.sink = 1 + 0.3 * rnd(H * D), 1 + 0.3 * rnd(G * D), 1 + 0.4 * rnd(H), 0.7 * rnd(H)
        self.cols = H * D + G * (D + E)
        t = dict(qkv=torch.zeros(64, -(-self.cols // 16) * 16, dtype=dtype, device="cuda"), kc=old(dk, 3e4), vc=old(dv, float("nan")), sink=self.sink.cuda(), temp=self.temp.cuda(), qn=self.qn.cuda(),
                 kn=self.kn.cuda(), qws=torch.zeros(64, H * dk, dtype=dtype, device="cuda"), out=torch.zeros(64, H * E, dtype=dtype, device="cuda"))
        self.t, a = t, {k: pk.attach_input(v, k) for k, v in t.items()}
        pk.flex_attention_layer(a["qkv"], a["kc"], a["vc"], None, None, a["sink"], a["qws"], a["out"], H, G, D, E, 0, self.scale, eps=1e-4, chunk=size, q_row_weight=a["qn"], k_row_weight=a["kn"],
                                score_factors=a["temp"])
        pk.compile()

    def data(self, n, seed):
        return torch.randn(n, self.cols, generator=torch.Generator().manual_seed(seed)).to(self.dtype).double()

    def run(self, entries):
        """entries: (first position, rows, page list)"""
        idx, ptr, slots, pos, at = [], [0], [], [], 0
        self.t["out"].fill_(7.0)
        for i, (p0, d, pages) in enumerate(entries):
            n = len(d)
            self.t["qkv"][at:at + n, :self.cols] = d.to(self.dtype).cuda()
            idx += pages
            ptr.append(len(idx))
            slots += [i] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.meta["paged_kv_indices_buffer"][:len(idx)] = torch.tensor(idx, dtype=torch.int32, device="cuda")
        self.meta["paged_kv_indptr_buffer"][:len(ptr)] = torch.tensor(ptr, dtype=torch.int32, device="cuda")
        self.pk.run_once(slots, pos)
        return list(self.t["out"][:at].cpu().double().view(at, self.H, self.E).split([len(d) for _, d, _ in entries]))

    def heads(self, d):
        from oracle.vizonex_ref import rms_norm
        nq, nk, r = self.H * self.D, self.G * self.D, lambda t: t.to(self.dtype).double()
        q, k = r(rms_norm(d[:, :nq], self.qn.double(), 1e-4)), r(rms_norm(d[:, nq:nq + nk], self.kn.double(), 1e-4))
        return q.view(-1, self.H, self.D), k.view(-1, self.G, self.D), d[:, nq + nk:].reshape(-1, self.G, self.E)

    def reference(self, d):
        from oracle.vizonex_ref import chunk_attention_core
        return chunk_attention_core(*self.heads(d), torch.arange(len(d)), self.scale, self.temp.double(), self.sink.double(), self.size)


CHUNKS = {"even": (4, 2, 32, 32, 64), "odd": (6, 2, 20, 28, 33), "one": (3, 3, 24, 10, 1), "two": (5, 1, 44, 36, 2), "wide": (4, 1, 160, 200, 130), "all": (4, 2, 128, 64, 0), "long": (8, 1, 64, 64, 250),
          "odd_columns": (3, 1, 23, 17, 50), "many_heads": (32, 4, 128, 128, 96)}


@BOTH
@pytest.mark.parametrize("name", CHUNKS)
def test_chunked_attention_alone(name, dtype):
    """Portions, single tokens and mixtures on a cache full of garbage; pages out of order."""
    rig = ChunkRig(*CHUNKS[name], dtype)
    lens = [330, 100, 70]
    data = [rig.data(n, 30 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    pages, at = [[7, 2, 9, 0, 11, 4], [5, 1], [3, 8]], [0, 0, 0]
    plan = [[(0, 64)], [(0, 2), (1, 31), (2, 3)], [(0, 62)], [(0, 1), (1, 1), (2, 1)], [(0, 40), (2, 2)], [(0, 24)], [(0, 33), (1, 3), (2, 20)], [(0, 1)], [(0, 1), (1, 60)], [(0, 64)], [(0, 3), (2, 40)]]
    plan += [[(0, 1), (1, 1), (2, 1)]] * 4 + [[(0, 1), (1, 1)]] + [[(0, 1)]] * 30
    for step in plan:
        got = rig.run([(at[r], data[r][at[r]:at[r] + n], pages[r]) for r, n in step])
        for (r, n), o in zip(step, got):
            torch.testing.assert_close(o, want[r][at[r]:at[r] + n], msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **_tol(dtype))
            at[r] += n
    assert at == lens
    rig.pk.finalize()


@BOTH
@pytest.mark.parametrize("size", [33, 64, 100, 31, 128])
def test_chunk_edges_alone(size, dtype):
    """One key per query stands out: the chunk's first position and the last one of the chunk before, tile and page borders, the newest key; in
    single tokens and in portions."""
    rig = ChunkRig(4, 2, 32, 32, size, dtype, scale=2.0)
    rig.qn.fill_(1.0), rig.kn.fill_(1.0), rig.temp.fill_(1.0)
    for k in ("qn", "kn", "temp"):
        rig.t[k].fill_(1.0)
    n, base, D, nq = 300, 230, 32, 128
    data = rig.data(n, 3)
    shown = 0
    for p in range(base, n):
        c0 = p // size * size
        j = [c0, c0 - 1, c0 + 1, p, p - 1, p // 32 * 32, p // 64 * 64, p // 64 * 64 - 1, c0 + size // 2][p % 9]
        j = min(max(j, 0), p)
        shown += c0 <= j
        for h in range(4):  # the query of every head points along that position's key
            data[p, h * D:(h + 1) * D] = 3.0 * data[j, nq + (h // 2) * D:nq + (h // 2 + 1) * D]
    assert 20 < shown < n - base
    data = data.to(dtype).double()
    want, perm = rig.reference(data), [3, 0, 4, 1, 2]
    for p0, p1 in ((0, 64), (64, 128), (128, 192), (192, base)):
        torch.testing.assert_close(rig.run([(p0, data[p0:p1], perm)])[0], want[p0:p1], **_tol(dtype))
    for p in range(base, n):
        torch.testing.assert_close(rig.run([(p, data[p:p + 1], perm)])[0], want[p:p + 1], msg=lambda m: f"query {p}: {m}", **_tol(dtype))
    for lo, hi in ((230, 232), (232, 263), (263, 300)):
        torch.testing.assert_close(rig.run([(lo, data[lo:hi], perm)])[0], want[lo:hi], msg=lambda m: f"queries {lo}..{hi}: {m}", **_tol(dtype))
    rig.pk.finalize()


class DualRig:
    """ring_conv (with steps) and dual_scan over caller-written rows; rings and states hold NaN at first."""

    def __init__(self, heads, vdim, state, groups, taps, dtype, slots=4, bias=-2.5):
        self.H, self.V, self.N, self.G, self.taps, self.dtype = heads, vdim, state, groups, taps, dtype
        up = lambda a, m: -(-a // m) * m
        I, Np = heads * vdim, up(state, 4)
        self.I, self.Np, self.Ip = I, Np, up(I, 4)
        n, Hp = self.Ip + 2 * groups * Np, up(heads, 4)
        self.pk, self.meta = pk, _ = _graph(64, slots, seq=512, pages=8 * slots)
        g = torch.Generator().manual_seed(I + state)
        rnd = lambda *s: torch.randn(*s, generator=g)
        C = I + 2 * groups * state
        self.w, self.b, self.bd = (rnd(C, taps) / taps ** 0.5).to(dtype), 0.3 * rnd(C), bias + rnd(heads)
        self.A, self.D = -torch.exp(0.5 * rnd(heads)), rnd(heads)
        z = lambda *s, dt=dtype: torch.zeros(*s, dtype=dt, device="cuda")
        self.at = torch.cat([torch.arange(I), self.Ip + (torch.arange(2 * groups)[:, None] * Np + torch.arange(state)).flatten()])  # where a channel of the model lies
        t = dict(rows=z(64, up(self.Ip + n + heads, 16)), conv=z(64, n), steps=z(64, 2 * Hp, dt=torch.float32), out=z(64, self.Ip, dt=torch.float32), cw=z(taps, n), cb=z(n, dt=torch.float32), bd=self.bd.cuda(),
                 A=(self.A / 0.6931471805599453).cuda(), D=self.D.cuda(), state=z(slots, heads, vdim, Np, dt=torch.float32).fill_(float("nan")), ring=z(slots, taps, n).fill_(float("nan")),
                 slots=torch.arange(slots, dtype=torch.int32, device="cuda"))
        t["cw"][:, self.at], t["cb"][self.at] = self.w.T.cuda(), self.b.cuda()
        self.t, a = t, {k: pk.attach_input(v, k) for k, v in t.items()}
        pk.ring_conv_layer(a["rows"], a["cw"], a["ring"], a["slots"], a["conv"], bias=a["cb"], column=self.Ip, silu=True, heads=heads, step_column=self.Ip + n, decay_column=Hp, step_bias=a["bd"], rates=a["A"],
                           steps=a["steps"])
        pk.dual_scan_layer(a["rows"], a["conv"], a["steps"], a["D"], a["state"], a["slots"], a["out"], heads, vdim, state, groups, 0, 0, self.Ip, self.Ip + groups * Np, Hp)
        pk.compile()
        self.dt_col = self.Ip + n

    def data(self, n, seed):
        """z [n, inner], x and B and C [n, channels], step input [n, heads]."""
        g = torch.Generator().manual_seed(seed)
        return [torch.randn(n, c, generator=g).to(self.dtype).double() for c in (self.I, len(self.at), self.H)]

    def run(self, entries):
        slots, pos, at = [], [], 0
        for slot, p0, (z, xbc, dt) in entries:
            n = len(z)
            self.t["rows"][at:at + n, :self.I] = z.to(self.dtype).cuda()
            self.t["rows"][at:at + n, self.Ip + self.at] = xbc.to(self.dtype).cuda()
            self.t["rows"][at:at + n, self.dt_col:self.dt_col + self.H] = dt.to(self.dtype).cuda()
            slots += [slot] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.t["out"].fill_(7.0)
        self.pk.run_once(slots, pos)
        return list(self.t["out"][:at, :self.I].cpu().double().split([len(d[0]) for _, _, d in entries]))

    def reference(self, d):
        from oracle.vizonex_ref import causal_conv, dual_scan, silu, softplus
        z, xbc, dt = d
        T, GN = len(z), self.G * self.N
        c, _ = causal_conv(xbc, torch.zeros(self.taps - 1, xbc.shape[1], dtype=F64), self.w.double(), self.b.double())
        x, B, C = silu(c).to(self.dtype).double().split([self.I, GN, GN], dim=1)
        _, y = dual_scan(torch.zeros(self.H, self.N, self.V, dtype=F64), softplus(dt + self.bd.double()), x.reshape(T, self.H, self.V), self.A.double(), B.reshape(T, self.G, self.N),
                         C.reshape(T, self.G, self.N), self.D.double())
        return y.reshape(T, self.I) * silu(z)


DUALS = {"tiny": (3, 5, 3, 1, 2), "odd": (6, 14, 37, 3, 6), "even": (4, 32, 64, 2, 4), "states16": (4, 64, 16, 4, 4), "states20": (2, 45, 20, 1, 3), "states100": (3, 130, 100, 1, 4), "states256": (2, 48, 256, 2, 9),
         "one_tap": (5, 16, 8, 5, 1), "one_value": (7, 1, 12, 7, 4), "many": (32, 128, 128, 8, 4)}


@BOTH
@pytest.mark.parametrize("name", DUALS)
def test_recurrence_alone(name, dtype):
    """Portions, single tokens and mixtures; a slot that is used again starts from zero whatever it holds (NaN at first); portions
    shorter than the convolution."""
    rig = DualRig(*DUALS[name], dtype)
    lens = [101, 38, 40, 5, 30]
    data = [rig.data(n, 20 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    at, slot = [0] * 5, [2, 0, 3, 1, 1]
    plan = [[(0, 64)], [(0, 2), (1, 31), (2, 3)], [(0, 8), (1, 1), (3, 2)], [(1, 1), (2, 30), (0, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 1)], [(2, 3), (0, 3)],
            [(0, 1), (2, 1), (3, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 17)], [(4, 1), (1, 1), (2, 1)], [(4, 17), (1, 4), (0, 1)], [(4, 1)], [(4, 11), (0, 1)]]
    tol = dict(rtol=2e-2, atol=4e-2) if dtype == torch.bfloat16 else dict(rtol=3e-5, atol=1e-4)
    for step in plan:
        got = rig.run([(slot[r], at[r], [t[at[r]:at[r] + n] for t in data[r]]) for r, n in step])
        for (r, n), o in zip(step, got):
            torch.testing.assert_close(o, want[r][at[r]:at[r] + n], msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **tol)
            at[r] += n
    assert at == lens
    rig.pk.finalize()


@pytest.mark.parametrize("heads,vdim,state", [(8, 100, 64), (16, 128, 128), (4, 64, 200)])
def test_recurrence_of_many_requests(heads, vdim, state):
    """64 requests of one token each: several units per workgroup, the states of the next ones in flight."""
    rig = DualRig(heads, vdim, state, 2, 4, torch.float32, slots=64)
    data = [rig.data(3, 100 + i) for i in range(64)]
    want = [rig.reference(d) for d in data]
    for t in range(3):
        for r, o in enumerate(rig.run([((5 * r) % 64, t, [x[t:t + 1] for x in data[r]]) for r in range(64)])):
            torch.testing.assert_close(o[0], want[r][t], rtol=3e-5, atol=1e-4)
    rig.pk.finalize()


def test_recurrence_remembers_a_first_token():
    """A first token that is still there after 300 others, through portions and single tokens."""
    rig = DualRig(2, 32, 8, 1, 4, torch.float32, bias=-7.0)  # (small steps: slow decay)
    n = 300
    d = rig.data(n, 7)
    d[2] *= 0.1
    d[1][0], d[1][4:, :64] = 3.0 * d[1][0].abs() + 2.0, 0.01 * d[1][4:, :64]
    d[2][0] = 7.0  # (a step of its own)
    want, without = rig.reference(d), rig.reference([torch.cat([x[:1] * 0, x[1:]]) if i == 1 else x for i, x in enumerate(d)])
    at = 0
    for m in [64, 2, 1, 64, 1, 1, 40, 64] + [1] * 63:
        o = rig.run([(3, at, [x[at:at + m] for x in d])])[0]
        at += m
    assert at == n
    torch.testing.assert_close(o[0], want[-1], rtol=3e-5, atol=1e-4)
    assert (want[-1] - without[-1]).norm() > 0.05 * want[-1].norm()
    rig.pk.finalize()


@BOTH
@pytest.mark.parametrize("rows", [1, 3, 17, 64])
@pytest.mark.parametrize("E,top,count,keep,ff,shared,width", [(6, 3, 3, 2, 20, 37, 84), (12, 2, 1, 1, 80, 144, 160), (7, 1, 7, 3, 50, None, 64), (200, 8, 10, 3, 64, 64, 256), (1, 1, 1, 1, 40, 24, 64),
                                                              (64, 16, 8, 4, 33, 100, 320), (256, 16, 128, 20, 32, None, 64), (96, 5, 2, 1, 32, 48, 64)])
def test_experts_alone(dtype, rows, E, top, count, keep, ff, shared, width):
    """Router, choice among groups, both expert linears with the clamped activation and the shared expert through the builder's own stages:
    shares and the places' outputs."""
    from mirage.mpk.models.vizonex.builder import VizonexBuilder, VizonexConfig
    from oracle.vizonex_ref import clamped_gate, route_groups
    from vizonex_helpers import chunked, config, moe, weights
    layer = moe(E, top, count, keep, ff, shared, limit=0.9, shared_limit=0.5)
    cfg = config([chunked(1, 1, 16, 16, 9, layer)], width, 40)
    w = weights(cfg, seed=E)
    pk, _ = _graph(64, 64)
    b = VizonexBuilder(pk)
    b.set_dtype(dtype)
    b.config = VizonexConfig.from_dict(cfg)
    b._begin(b.config, {k: v.cuda() for k, v in w.items()}, True)
    x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(dtype)
    h = torch.zeros(64, b._W, dtype=dtype, device="cuda")
    h[:rows, :width] = x.cuda()
    parts = b._experts(0, "l0.mlp.", b.config.layers[0].ff, pk.attach_input(h, "h"))
    pk.compile()
    wd = {k[7:]: v.double() for k, v in w.items() if k.startswith("l0.mlp.")}
    expert = lambda t, name, lim: clamped_gate(t @ wd[name + ".gate"].T, t @ wd[name + ".up"].T, lim) @ wd[name + ".down"].T
    tol = dict(rtol=3e-2, atol=3e-2) if dtype == torch.bfloat16 else dict(rtol=3e-5, atol=3e-5)
    for _ in range(2):  # the lists of the first run are gone in the second
        pk.run_once(list(range(rows)), [0] * rows)
        f, y = parts["slot_weights"].to_torch()[:rows].cpu().double(), parts["input2"].to_torch()[:rows].cpu().double().view(rows, parts["slots"], b._W)[:, :, :width]
        for t in range(rows):
            xt = x[t].double()
            idx, share = route_groups(xt @ wd["router"].T, wd["correction"], top, count, keep, 1.7)
            torch.testing.assert_close(f[t, :top], share, rtol=2e-4 if dtype == torch.bfloat16 else 2e-5, atol=1e-6)
            for s, e in enumerate(idx.tolist()):
                torch.testing.assert_close(y[t, s], expert(xt, f"e{e}", 0.9), msg=lambda m: f"token {t} place {s} expert {e}: {m}", **tol)
            if shared is not None:
                assert f[t, top] == 1.0
                torch.testing.assert_close(y[t, top], expert(xt, "shared", 0.5), **tol)
    pk.finalize()


# ---------------------------------------------------------------- whole models
@BOTH
@pytest.mark.parametrize("name", ["even", "odd", "wide", "taps"])
def test_prompt_portions_and_decoding_agree_with_the_oracle(name, dtype):
    from vizonex_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS[name]
    w, toks = weights(cfg), prompt(cfg, 150)
    want = _oracle_logits(cfg, w, toks)
    s = _session(cfg, w, dtype)
    for cuts in ([150], [1] * 40 + [110], [2, 3, 1, 40, 64, 1, 1, 1, 37], [17] * 8 + [2] * 7, [130] + [1] * 20):
        _close(_feed(s, "r", toks, cuts), want, dtype, f"{name} {cuts[:4]}")
        s.end("r")
    s.finalize()


@BOTH
def test_mixed_batches_pages_and_slots_used_again(dtype):
    """Unequal requests together, pausing and going on, ending and making room: the logits of every position are those of the
    request alone.  The pool is too small for all requests at once and there are four state slots for seven requests."""
    from vizonex_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    lens = {"a": 200, "b": 65, "c": 1, "d": 130, "e": 90, "f": 64, "g": 37}
    toks = {r: prompt(cfg, n, seed=i) for i, (r, n) in enumerate(lens.items())}
    want = {r: _oracle_logits(cfg, w, t) for r, t in toks.items()}
    s = _session(cfg, w, dtype, max_tokens=384)
    at, got, live = dict.fromkeys(lens, 0), {r: [] for r in lens}, []
    waiting, g, used, slots = list(lens), torch.Generator().manual_seed(4), set(), set()
    pages = lambda r: -(-lens[r] // 64)
    while waiting or live:
        while waiting and len(live) < 4 and sum(map(pages, live)) + pages(waiting[0]) <= 6:
            live.append(waiting.pop(0))
        step = []
        for r in live:
            n = min([0, 1, 1, 2, 3, 17, 40, 64][int(torch.randint(0, 8, (1,), generator=g))], lens[r] - at[r])
            if n:
                step.append((r, n))
        if not step:
            continue
        lg, _ = s.step([(r, toks[r][at[r]:at[r] + n]) for r, n in step], [list(range(n)) for _, n in step])
        o = 0
        for r, n in step:
            got[r].append(lg[o:o + n].cpu().double())
            o, at[r] = o + n, at[r] + n
            used.update(s.requests[r].pages)
            slots.add(s.requests[r].slot)
            if at[r] == lens[r]:
                s.end(r)
                live.remove(r)
    assert len(s.pool) == 6 and used == set(range(6)) and len(s.slots) == 4 and slots <= set(range(4))
    for r in lens:
        _close(torch.cat(got[r]), want[r], dtype, r, bf16_outliers=0.08)
    s.finalize()


@BOTH
def test_long_decoding(dtype):
    """Hundreds of single tokens across page and chunk borders."""
    from vizonex_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["even"]
    w, toks = weights(cfg), prompt(cfg, 420)
    s = _session(cfg, w, dtype, max_tokens=448)
    _close(_feed(s, "r", toks, [3] + [1] * 417), _oracle_logits(cfg, w, toks), dtype)
    s.finalize()


def test_wide_model_takes_the_tuned_linears():
    """A width of 2048: sums, norms and convolutions folded into the single-token streaming form, the staged matrix-core form at 1, 2, 8,
    40 and 64 rows, recurrences of 2048 and of 4096 values, norms in several parts."""
    from vizonex_helpers import chunked, config, dense, dual, moe, prompt, weights
    cfg = config([chunked(16, 4, 128, 128, 100, dense(2048)), dual(16, 128, 40, 4, 8, 4, moe(16, 4, 4, 2, 256, 256)), dual(32, 128, 12, 1, 2, 4, dense(4096))], 2048, 1000)
    w, toks = weights(cfg), prompt(cfg, 140)
    want = _oracle_logits(cfg, w, toks)
    s = _session(cfg, w, torch.bfloat16, max_tokens=256)
    for cuts in ([140], [64, 40, 8, 2, 2, 8] + [1] * 16):
        _close(_feed(s, "r", toks, cuts), want, torch.bfloat16, str(cuts[:4]))
        s.end("r")
    for r in range(4):
        s.step([(r, toks[:50 - r])])
    lg, _ = s.step([(r, toks[50 - r:51 - r]) for r in range(4)], [[0]] * 4)
    _close(lg.cpu().double(), torch.stack([want[50 - r] for r in range(4)]), torch.bfloat16)
    s.finalize()


def test_single_weight_copy():
    """Linear weights kept once, in tile order: iterations of one token take the matrix-core forms, their norms and convolutions the stages."""
    from generate import Generator
    from mirage.mpk import MirageModelConfig
    from vizonex_helpers import chunked, config, dense, dual, moe, prompt, weights
    cfg = config([chunked(4, 2, 64, 64, 50, dense(256)), dual(4, 64, 32, 2, 4, 4, moe(8, 2, 4, 2, 64, 64))], 256, 320)  # (reductions in whole tiles)
    w, p = weights(cfg), prompt(cfg, 40)
    g = Generator(80, model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in w.items()}), batch=1, max_num_batched_tokens=16, max_tokens_per_request=16, page_size=64,
                  eos_token_id=-1, single_weight_copy=True)
    ids = g.generate([p])[0]
    lg = _oracle_logits(cfg, w, ids[:-1])
    off = [t for t in range(39, 79) if not lg[t, ids[t + 1]] > lg[t].max() - 0.15 * lg.std()]
    assert len(off) <= 1, off
    g.finalize()


def test_sessions_keep_requests_within_the_position_table():
    from vizonex_helpers import CONFIGS, prompt, weights
    cfg = dict(CONFIGS["even"], max_positions=70)
    w, toks = weights(cfg), prompt(cfg, 70)
    s = _session(cfg, w, torch.float32, max_tokens=256)
    _close(_feed(s, "r", toks, [64, 5, 1]), _oracle_logits(cfg, w, toks), torch.float32)
    with pytest.raises(ValueError, match="max_seq_length=70"):
        s.step([("r", toks[:1])])
    with pytest.raises(ValueError, match="max_seq_length=70"):
        s.generate([toks[:60]], 12)
    s.end("r")
    assert len(s.generate([toks[:60]], 11)[0]) == 71
    s.finalize()


# ---------------------------------------------------------------- generation through the framework's entry points
def _checkpoint(tmp_path, cfg, w):
    from safetensors.torch import save_file
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    return str(tmp_path)


def test_greedy_generation_from_a_checkpoint(tmp_path, capsys):
    """32-bit, so that the tokens are the oracle's: the offline engine with two and with three batch slots for five requests (the
    on-GPU schedulers move requests, and with them their states, between slots), the serving session, the command line."""
    import generate
    from generate import Generator
    from mirage.mpk import ServingSession
    from vizonex_helpers import CONFIGS, prompt, weights
    from oracle.vizonex_ref import VizonexOracle
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    path = _checkpoint(tmp_path, cfg, w)
    prompts = [prompt(cfg, n, seed=20 + n) for n in (70, 3, 1, 33, 64)]
    orc = VizonexOracle(cfg, w)
    want = [orc.generate(p, 20) for p in prompts]
    for batch in (2, 3):
        g = Generator(70 + 20 + 1, model_path=path, batch=batch, max_num_batched_tokens=16, max_tokens_per_request=16, page_size=64, total_requests=5, eos_token_id=-1,
                      dtype=torch.float32)
        for _ in range(2):  # the same handle serves again
            assert g.generate(prompts, 20) == want
        assert sorted(g.model.model_builder.state_slots.tolist()) == list(range(batch))
        g.finalize()
    s = ServingSession.open(model_path=path, dtype=torch.float32, max_tokens=256, max_requests=3)
    assert s.generate(prompts, 20) == want
    assert len(s.pool) == s.pool.num_pages and len(s.slots) == 3
    s.finalize()
    ids = [",".join(map(str, p)) for p in prompts[:2]]
    for engine in ("offline", "serving"):
        capsys.readouterr()
        generate.main(["--model-path", path, "--dtype", "float32", "--prompt-ids", ids[0], "--prompt-ids", ids[1], "--max-new-tokens", "20", "--engine", engine])
        lines = capsys.readouterr().out.splitlines()
        assert [int(t) for t in lines[0].split(":")[1].split()] == want[0][70:] and [int(t) for t in lines[1].split(":")[1].split()] == want[1][3:]


def test_generation_in_bf16_is_greedy_on_its_own_logits():
    """Offline engine in bf16, single-token kernel and batched one: every sampled token is the argmax of near-oracle logits."""
    from generate import Generator
    from mirage.mpk import MirageModelConfig
    from vizonex_helpers import CONFIGS, prompt, weights
    for name in ("even", "wide"):
        cfg = CONFIGS[name]
        w = weights(cfg)
        for rows, batch in ((1, 1), (8, 4)):
            g = Generator(80, model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in w.items()}), batch=batch, max_num_batched_tokens=rows,
                          page_size=64, eos_token_id=-1)
            prompts = [prompt(cfg, 9 + i, seed=i) for i in range(batch)]
            for p, ids in zip(prompts, g.generate(prompts)):
                assert len(ids) == 80 and ids[:len(p)] == p
                lg = _oracle_logits(cfg, w, ids[:-1])
                off = [t for t in range(len(p) - 1, 79) if not lg[t, ids[t + 1]] > lg[t].max() - 0.15 * lg.std()]
                assert len(off) <= 2, off
            g.finalize()


def test_trace_replay(tmp_path, monkeypatch, capsys):
    """bin/trace_run on a checkpoint of its own: files, order of the rows, and the `done` lines."""
    import io
    import os
    import sys
    from importlib.machinery import SourceFileLoader

    import numpy as np

    from conftest import ROOT
    from vizonex_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["odd"]
    w, toks = weights(cfg), prompt(cfg, 80)
    path = _checkpoint(tmp_path, cfg, w)
    out = tmp_path / "out"
    out.mkdir()
    steps = [{"step": 0, "entries": [{"id": "p", "tokens": toks[:70], "want": [69, 3]}, {"id": "q", "tokens": toks[:1], "want": []}], "end": []},
             {"step": 1, "entries": [{"id": "q", "tokens": toks[1:3], "want": []}], "end": ["q"]},
             {"step": 2, "entries": [{"id": "z", "tokens": toks[:2], "want": [1]}, {"id": "p", "tokens": toks[70:71], "want": [0]}], "end": ["z", "p"]}]
    trace_run = SourceFileLoader("trace_run", os.path.join(ROOT, "bin", "trace_run")).load_module()
    monkeypatch.setattr(sys, "stdin", io.StringIO("".join(json.dumps(s) + "\n" for s in steps)))
    trace_run.main(["--model", path, "--dtype", "float32", "--out", str(out), "--max-tokens", "192"])
    assert [l for l in capsys.readouterr().out.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    want = _oracle_logits(cfg, w, toks)
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"])).double()
    _close(read(0), want[[69, 3]], torch.float32)
    _close(read(2), want[[1, 70]], torch.float32)
