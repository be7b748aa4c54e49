"""Bukatar on the GPU against the plain oracle: every mechanism alone, whole models of several sizes in bf16 and in 32 bits, prompts
against single tokens, portions, mixed batches, pages and state slots used again, window edges, long decoding, and greedy generation
through the framework's own entry points.  Expected values come from oracle/bukatar_ref.py in float64."""
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
    from oracle.bukatar_ref import BukatarOracle
    orc = BukatarOracle(cfg, w)
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


def _close(got, want, dtype, what="", bf16_outliers=0.02):
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


# ---------------------------------------------------------------- mechanisms alone
@BOTH
@pytest.mark.parametrize("rows", [1, 2, 5, 16, 40, 64])
@pytest.mark.parametrize("n,k", [(70, 64), (200, 192), (512, 2048), (300, 4096)])
def test_relu_squared_linear(dtype, rows, n, k):
    import mirage as mi
    from oracle.bukatar_ref import relu_squared
    g = torch.Generator().manual_seed(rows * n)
    x, w = torch.randn(rows, k, generator=g).to(dtype).cuda(), (torch.randn(n, k, generator=g) / k ** 0.5).to(dtype).cuda()
    pk, _ = _graph(64, 64)
    rows_in = torch.zeros(64, k, dtype=dtype, device="cuda")
    rows_in[:rows] = x
    out = torch.zeros(64, n, dtype=dtype, device="cuda")
    E = mi.bfloat16 if dtype == torch.bfloat16 else mi.float32
    up = pk.new_tensor((64, n), dtype=E, name="up")
    pk.linear_layer(pk.attach_input(rows_in, "x"), pk.attach_input(w, "w"), up, (1, 1, 1), (256, 1, 1))
    pk.relu_squared_layer(up, pk.attach_input(out, "o"))
    # (a flex stage tells the graph its kernel family by itself: the activation is enough)
    pk.compile()
    pk.run_once(list(range(rows)), [0] * rows)
    torch.testing.assert_close(out[:rows].cpu().double(), relu_squared(x.cpu().double() @ w.cpu().double().T), **_tol(dtype))
    assert not out[rows:].any()
    pk.finalize()


@BOTH
@pytest.mark.parametrize("width,ld,slots", [(64, 64, 0), (84, 128, 0), (84, 128, 4), (200, 256, 9), (2048, 2048, 9), (4096, 4096, 1), (6000, 6016, 3)])
def test_prenorm_with_bias_and_places(dtype, width, ld, slots):
    """The summand plus a bias, or the weighted sum of a token's places, normalised, into the stream; as a stage and in a linear."""
    import mirage as mi
    from oracle.bukatar_ref import rms_norm
    g = torch.Generator().manual_seed(width + slots)
    rnd = lambda *s: torch.randn(*s, generator=g)
    S = max(slots, 1)
    x, y, f = rnd(5, width), rnd(5, S, width).to(dtype), rnd(5, S)
    b, yw, w = rnd(width), 1 + 0.3 * rnd(width), 1 + 0.3 * rnd(width)
    wl = (rnd(48, width) / width ** 0.5).to(dtype)
    pad = torch.nn.functional.pad
    summand = (y.double() * f.double()[..., None]).sum(1) if slots else y[:, 0].double() + b.double()
    v = x.double() + rms_norm(summand, yw.double(), 1e-3)
    h = rms_norm(v, w.double(), 1e-4)
    for fused in (False, True):
        for rows in (1, 5):
            pk, _ = _graph(8, 8)
            put = lambda t, cols, dt, name: pk.attach_input(keep.setdefault(name, pad(t.reshape(t.shape[0], -1), (0, cols - t.reshape(t.shape[0], -1).shape[1], 0, 8 - t.shape[0])).to(dt).cuda()), name)
            vec = lambda t, name: pk.attach_input(keep.setdefault(name, pad(t, (0, ld - width)).cuda()), name)
            keep = {}
            yp = torch.zeros(5, S, ld, dtype=dtype)
            yp[:, :, :width] = y
            kw = dict(slot_weights=put(f, 12, torch.float32, "f"), slots=slots, slot_columns=ld) if slots else dict(input_bias=vec(b, "b"))
            new_x, out, lo = torch.zeros(8, ld, device="cuda"), torch.zeros(8, ld, dtype=dtype, device="cuda"), torch.zeros(8, 48, dtype=dtype, device="cuda")
            o = pk.attach_input(out, "o")
            pk.residual_prenorm_layer(put(yp, S * ld, dtype, "y"), put(x, ld, torch.float32, "x"), pk.attach_input(new_x, "nx"), o, weight=vec(w, "w"), input_weight=vec(yw, "yw"), width=width,
                                      eps=1e-4, input_eps=1e-3, **kw)
            if fused:
                keep["wl"] = pad(wl, (0, ld - width)).contiguous().cuda()
                pk.linear_layer(o, pk.attach_input(keep["wl"], "wl"), pk.attach_input(lo, "lo"), (1, 1, 1), (256, 1, 1))
            pk.compile()
            pk.run_once(list(range(rows)), [0] * rows)
            torch.testing.assert_close(new_x[:rows, :width].cpu().double(), v[:rows], rtol=3e-5, atol=3e-5)
            torch.testing.assert_close(out[:rows, :width].cpu().double(), h[:rows], **_tol(dtype))
            if fused:
                torch.testing.assert_close(lo[:rows].cpu().double(), h[:rows] @ wl.double().T, rtol=3e-2 if dtype == torch.bfloat16 else 1e-4, atol=3e-2 if dtype == torch.bfloat16 else 1e-4)
            pk.finalize()


class WindowRig:
    """flex_attention_layer with a window, kept first positions, biases, a unit sink and values from keys, over caller-written rows."""

    def __init__(self, H, G, D, rot, size, keep, dtype, pages=12, scale=None):
        from mirage.mpk.models.checkpoint import rotary_tables_f32
        from mirage.mpk.persistent_kernel import flex_cache_dims, pairs_to_halves
        self.H, self.G, self.D, self.rot, self.size, self.keep, self.dtype = H, G, D, rot, size, keep, dtype
        self.scale, self.order = scale or 1.5 / D ** 0.5, pairs_to_halves(D, rot)
        self.pk, self.meta = pk, _ = _graph(64, 4, seq=pages * 64, pages=pages)
        dk, dv = flex_cache_dims(D, D, dtype)
        old = lambda d, v: torch.full((pages, 64, G, d), v, dtype=dtype, device="cuda")  # nothing of it may show
        g = torch.Generator().manual_seed(5)
        self.bias = 0.3 * torch.randn(H + G, D, generator=g)
        t = dict(qk=torch.zeros(64, (H + G) * D, dtype=dtype, device="cuda"), kc=old(dk, 3e4), vc=old(dv, float("nan")), sink=torch.zeros(H, device="cuda"), b=self.bias[:, self.order].reshape(-1).cuda(),
                 qws=torch.zeros(64, H * dk, dtype=dtype, device="cuda"), out=torch.zeros(64, H * D, dtype=dtype, device="cuda"))
        if rot:
            t["cos"], t["sin"] = rotary_tables_f32(rot, 500.0, None, pages * 64)
        self.t, a = t, {k: pk.attach_input(v, k) for k, v in t.items()}
        pk.flex_attention_layer(a["qk"], a["kc"], a["vc"], a.get("cos"), a.get("sin"), a["sink"], a["qws"], a["out"], H, G, D, D, rot, self.scale, window=size, keep_first=keep,
                                values_from_keys=True, input_bias=a["b"])
        pk.compile()

    def data(self, n, seed):
        g = torch.Generator().manual_seed(seed)
        return torch.randn(n, self.H + self.G, self.D, generator=g).to(self.dtype).double()

    def run(self, entries):
        """entries: (first position, rows, page list)"""
        idx, ptr, slots, pos, at = [], [0], [], [], 0
        self.t["out"].fill_(7.0)
        for i, (p0, d, pages) in enumerate(entries):
            n = len(d)
            self.t["qk"][at:at + n] = d[..., self.order].reshape(n, -1).to(self.dtype).cuda()
            idx += pages
            ptr.append(len(idx))
            slots += [i] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.meta["paged_kv_indices_buffer"][:len(idx)] = torch.tensor(idx, dtype=torch.int32, device="cuda")
        self.meta["paged_kv_indptr_buffer"][:len(ptr)] = torch.tensor(ptr, dtype=torch.int32, device="cuda")
        self.pk.run_once(slots, pos)
        o = torch.empty(at, self.H, self.D, dtype=F64)
        o[..., self.order] = self.t["out"][:at].cpu().double().view(at, self.H, self.D)
        return list(o.split([len(d) for _, d, _ in entries]))

    def reference(self, d):
        from oracle.bukatar_ref import rotate_pairs, window_attention_core
        r, pos, x = lambda t: t.to(self.dtype).double(), torch.arange(len(d)), d + self.bias.double()
        turn = lambda t: r(rotate_pairs(t, pos, self.rot, 500.0))
        q, k = x[:, :self.H], x[:, self.H:]
        return window_attention_core(turn(q), turn(k), r(k), pos, self.scale, self.size or None, self.keep)


WINDOWS = {"even": (4, 2, 32, 16, 48, 8), "odd": (6, 1, 20, 12, 33, 5), "one": (3, 3, 24, 24, 1, 0), "nothing_kept": (5, 1, 40, 0, 100, 0), "kept_tile": (2, 2, 64, 32, 64, 64),
           "wide": (4, 1, 160, 96, 130, 40), "all": (4, 2, 128, 64, 0, 0), "many_kept": (8, 1, 64, 16, 20, 170), "tiles": (16, 2, 128, 128, 256, 32)}


@BOTH
@pytest.mark.parametrize("name", WINDOWS)
def test_window_attention_alone(name, dtype):
    """Portions, single tokens and mixtures on a cache full of garbage; pages out of order."""
    rig = WindowRig(*WINDOWS[name], dtype)
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
@pytest.mark.parametrize("size,keep", [(42, 18), (64, 0), (33, 1), (100, 64), (31, 33)])
def test_window_edges_alone(size, keep, dtype):
    """One key per query stands out: just inside and just outside the window, the last kept position and the next, tile and page
    borders; in single tokens and in portions."""
    rig = WindowRig(4, 2, 32, 0, size, keep, dtype, scale=2.0)
    n, base = 300, 250
    data = 0.2 * rig.data(n, 3)
    offsets = [0, 1, size - 2, size - 1, size, size + 1, size + 31, size + 32, size + 63]
    for i in range(n - base):
        p = base + i
        j = max(0, [p - o for o in offsets][i % 9] if i % 3 else [0, keep - 1, keep, keep + 1, 31, 32, 63, 64, 65, 127, 128][(i // 3) % 11])
        data[p, :4] = (3.0 * (data[j, 4:] + rig.bias[4:].double())).repeat_interleave(2, 0) - rig.bias[:4].double()
    data = data.to(dtype).double()
    want, perm = rig.reference(data), [3, 0, 4, 1, 2]
    for p0, p1 in ((0, 64), (64, 128), (128, 192), (192, 250)):
        torch.testing.assert_close(rig.run([(p0, data[p0:p1], perm)])[0], want[p0:p1], **_tol(dtype))
    for p in range(base, n):
        torch.testing.assert_close(rig.run([(p, data[p:p + 1], perm)])[0], want[p:p + 1], msg=lambda m: f"query {p}: {m}", **_tol(dtype))
    for lo, hi in ((250, 252), (252, 283), (283, 300)):
        torch.testing.assert_close(rig.run([(lo, data[lo:hi], perm)])[0], want[lo:hi], msg=lambda m: f"queries {lo}..{hi}: {m}", **_tol(dtype))
    rig.pk.finalize()


class ScanRig:
    """short_conv, scan_step and selective_scan over caller-written rows; slots hold NaN at first."""

    def __init__(self, inner, state, taps, dt_rank, dtype, slots=4, bias=-3.0):
        import mirage as mi
        from mirage.mpk.persistent_kernel import operand_row, operand_tiles
        self.n, self.N, self.taps, self.R, self.dtype = inner, state, taps, dt_rank, dtype
        up = lambda a, m: -(-a // m) * m
        I, Np, K = up(inner, 64), up(state, 4), up(dt_rank, operand_row(dtype))
        self.I, self.Kc, self.s = I, up(K, 16), up(state, 16)
        self.pk, self.meta = pk, _ = _graph(64, slots, seq=512, pages=8 * slots)
        g = torch.Generator().manual_seed(inner + state)
        rnd = lambda *s: torch.randn(*s, generator=g)
        self.w, self.b, self.wd, self.bd = rnd(inner, taps) / taps ** 0.5, 0.3 * rnd(inner), (rnd(inner, dt_rank) / dt_rank ** 0.5).to(dtype), bias + rnd(inner)
        self.A, self.D = -torch.exp(0.5 * rnd(inner, state)), rnd(inner)
        pad = torch.nn.functional.pad
        z = lambda *s, dt=dtype: torch.zeros(*s, dtype=dt, device="cuda")
        t = dict(xz=z(64, 2 * I), dbc=z(64, self.Kc + 2 * self.s), x=z(64, I), step=z(64, I, dt=torch.float32), out=z(64, I), cw=z(taps, I, dt=torch.float32),
                 cb=pad(self.b, (0, I - inner)).cuda(), wd=operand_tiles(pad(self.wd, (0, K - dt_rank, 0, I - inner))[None]).cuda(), bd=pad(self.bd, (0, I - inner)).cuda(),
                 A=(pad(self.A, (0, Np - state, 0, I - inner)) / 0.6931471805599453).cuda(), D=pad(self.D, (0, I - inner)).cuda(),
                 state=z(slots, I, Np, dt=torch.float32).fill_(float("nan")), tail=z(slots, max(taps - 1, 1), I).fill_(float("nan")), slots=torch.arange(slots, dtype=torch.int32, device="cuda"))
        t["cw"][:, :inner] = self.w.T.cuda()
        self.t, a = t, {k: pk.attach_input(v, k) for k, v in t.items()}
        pk.short_conv_layer(a["xz"], a["cw"], a["cb"], a["tail"], a["slots"], a["x"])
        pk.scan_step_layer(a["dbc"], a["wd"], a["bd"], a["step"], I, K)
        pk.selective_scan_layer(a["xz"], a["x"], a["step"], a["dbc"], a["A"], a["D"], a["state"], a["tail"], a["slots"], a["out"], state, taps, 0, I, self.Kc, self.Kc + self.s)
        pk.compile()

    def data(self, n, seed):
        """x, z [n, inner], step input [n, rank], B, C [n, states]."""
        g = torch.Generator().manual_seed(seed)
        return [torch.randn(n, c, generator=g).to(self.dtype).double() for c in (self.n, self.n, self.R, self.N, self.N)]

    def run(self, entries):
        slots, pos, at = [], [], 0
        for slot, p0, (x, z, d, B, C) in entries:
            n = len(x)
            for name, col, src in (("xz", 0, x), ("xz", self.I, z), ("dbc", 0, d), ("dbc", self.Kc, B), ("dbc", self.Kc + self.s, C)):
                self.t[name][at:at + n, col:col + src.shape[1]] = src.to(self.dtype).cuda()
            slots += [slot] * n
            pos += list(range(p0, p0 + n))
            at += n
        self.t["out"].fill_(7.0)
        self.pk.run_once(slots, pos)
        return list(self.t["out"][:at, :self.n].cpu().double().split([len(d[0]) for _, _, d in entries]))

    def reference(self, d):
        from oracle.bukatar_ref import causal_conv, selective_scan, silu, softplus
        x, z, dt, B, C = d
        xc, _ = causal_conv(x, torch.zeros(self.taps - 1, self.n, dtype=F64), self.w.double(), self.b.double())
        xc = silu(xc).to(self.dtype).double()
        _, y = selective_scan(torch.zeros(self.n, self.N, dtype=F64), softplus(dt @ self.wd.double().T + self.bd.double()), xc, self.A.double(), B, C, self.D.double())
        return y * silu(z)


SCANS = {"tiny": (5, 3, 2, 4), "odd": (75, 11, 3, 5), "even": (128, 16, 4, 16), "states32": (300, 32, 4, 40), "states37": (90, 37, 6, 33), "states100": (130, 100, 4, 8), "states256": (64, 256, 9, 64),
         "one_tap": (64, 8, 1, 8), "wide": (4096, 16, 4, 128)}


@BOTH
@pytest.mark.parametrize("name", SCANS)
def test_scan_alone(name, dtype):
    """Portions, single tokens and mixtures; a slot that is used again starts from zero whatever it holds (NaN at first); portions
    shorter than the convolution."""
    rig = ScanRig(*SCANS[name], dtype)
    lens = [101, 38, 40, 5, 30]
    data = [rig.data(n, 20 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    at, slot = [0] * 5, [2, 0, 3, 1, 1]
    plan = [[(0, 64)], [(0, 2), (1, 31), (2, 3)], [(0, 8), (1, 1), (3, 2)], [(1, 1), (2, 30), (0, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 1)], [(2, 3), (0, 3)],
            [(0, 1), (2, 1), (3, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 17)], [(4, 1), (1, 1), (2, 1)], [(4, 17), (1, 4), (0, 1)], [(4, 1)], [(4, 11), (0, 1)]]
    tol = dict(rtol=2e-2, atol=3e-2) if dtype == torch.bfloat16 else dict(rtol=2e-5, atol=5e-5)
    for step in plan:
        got = rig.run([(slot[r], at[r], [t[at[r]:at[r] + n] for t in data[r]]) for r, n in step])
        for (r, n), o in zip(step, got):
            torch.testing.assert_close(o, want[r][at[r]:at[r] + n], msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **tol)
            at[r] += n
    assert at == lens
    rig.pk.finalize()


def test_scan_many_requests_and_long_memory():
    """64 requests of one token each (several units per workgroup), and a first token that is still there after 300 others."""
    rig = ScanRig(2048, 16, 4, 32, torch.float32, slots=64)
    data = [rig.data(3, 100 + i) for i in range(64)]
    want = [rig.reference(d) for d in data]
    for t in range(3):
        for r, o in enumerate(rig.run([((5 * r) % 64, t, [x[t:t + 1] for x in data[r]]) for r in range(64)])):
            torch.testing.assert_close(o[0], want[r][t], rtol=2e-5, atol=5e-5)
    rig.pk.finalize()
    rig = ScanRig(64, 8, 4, 8, torch.float32, bias=-6.0)  # (small steps: slow decay)
    n = 300
    d = rig.data(n, 7)
    d[2] *= 0.1
    d[3][0], d[3][1:] = 40.0, d[3][1:] * 0.01
    want, without = rig.reference(d), rig.reference([x if i != 3 else torch.cat([x[:1] * 0, x[1:]]) for i, x in enumerate(d)])
    at = 0
    for m in [64, 2, 1, 64, 1, 1, 40, 64] + [1] * 63:
        o = rig.run([(3, at, [x[at:at + m] for x in d])])[0]
        at += m
    assert at == n
    torch.testing.assert_close(o[0], want[-1], rtol=3e-5, atol=5e-5)
    assert (want[-1] - without[-1]).norm() > 0.05 * want[-1].norm()
    rig.pk.finalize()


@BOTH
@pytest.mark.parametrize("rows", [1, 3, 17, 64])
@pytest.mark.parametrize("E,top,ff,shared,width", [(5, 3, 20, 37, 84), (12, 2, 80, 144, 160), (7, 1, 50, None, 64), (200, 8, 64, 64, 256), (1, 1, 40, 24, 64), (64, 16, 33, 100, 320)])
def test_experts_alone(dtype, rows, E, top, ff, shared, width):
    """Router, choice, both expert linears and the shared expert through the builder's own stages: shares and the places' outputs."""
    import mirage as mi
    from mirage.mpk.models.bukatar.builder import BukatarBuilder, BukatarConfig, ExpertFF
    from oracle.bukatar_ref import route, silu
    from bukatar_helpers import config, moe, weights, window
    layer = moe(E, top, ff, shared or 1)
    if shared is None:
        del layer["shared"]
    cfg = config([window(1, 1, 16, 0, 9, 1, layer)], width, 40)
    w = weights(cfg, seed=E)
    pk, _ = _graph(64, 64)
    b = BukatarBuilder(pk)
    b.set_dtype(dtype)
    b.config = BukatarConfig.from_dict(cfg)
    b._shapes, b._state, b._acts = b.config.tensor_shapes(), {k: v.cuda() for k, v in w.items()}, {}
    b._E, b._W = mi.bfloat16 if dtype == torch.bfloat16 else mi.float32, -(-width // 64) * 64
    x = torch.randn(rows, width, generator=torch.Generator().manual_seed(rows)).to(dtype)
    h = torch.zeros(64, b._W, dtype=dtype, device="cuda")
    h[:rows, :width] = x.cuda()
    parts = b._experts(0, "l0.mlp.", b.config.layers[0].ff, pk.attach_input(h, "h"))
    pk.compile()
    for _ in range(2):  # the lists of the first run are gone in the second
        pk.run_once(list(range(rows)), [0] * rows)
        f, y = parts["slot_weights"].to_torch()[:rows].cpu().double(), parts["input"].to_torch()[:rows].cpu().double().view(rows, parts["slots"], b._W)[:, :, :width]
        wd = {k[7:]: v.double() for k, v in w.items() if k.startswith("l0.mlp.")}
        expert = lambda t, name: (silu(t @ wd[name + ".gate"].T) * (t @ wd[name + ".up"].T)) @ wd[name + ".down"].T
        tol = dict(rtol=3e-2, atol=3e-2) if dtype == torch.bfloat16 else dict(rtol=3e-5, atol=3e-5)
        for t in range(rows):
            xt = x[t].double()
            idx, share = route(xt @ wd["router"].T, top)
            torch.testing.assert_close(f[t, :top], share, rtol=2e-4 if dtype == torch.bfloat16 else 2e-5, atol=1e-6)
            for s, e in enumerate(idx.tolist()):
                torch.testing.assert_close(y[t, s], expert(xt, f"e{e}"), msg=lambda m: f"token {t} place {s} expert {e}: {m}", **tol)
            if shared is not None:
                torch.testing.assert_close(f[t, top], torch.sigmoid(xt @ wd["shared.sg"].T)[0], rtol=2e-4, atol=1e-6)
                torch.testing.assert_close(y[t, top], expert(xt, "shared"), **tol)
    pk.finalize()


# ---------------------------------------------------------------- whole models
@BOTH
@pytest.mark.parametrize("name", ["even", "odd", "wide"])
def test_prompt_portions_and_decoding_agree_with_the_oracle(name, dtype):
    from bukatar_helpers import CONFIGS, prompt, weights
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
    from bukatar_helpers import CONFIGS, prompt, weights
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
        _close(torch.cat(got[r]), want[r], dtype, r, bf16_outliers=0.04)
    s.finalize()


@BOTH
def test_long_decoding(dtype):
    """Hundreds of single tokens across page, window and chunk borders."""
    from bukatar_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["even"]
    w, toks = weights(cfg), prompt(cfg, 420)
    s = _session(cfg, w, dtype, max_tokens=448)
    _close(_feed(s, "r", toks, [3] + [1] * 417), _oracle_logits(cfg, w, toks), dtype)
    s.finalize()


def test_wide_model_takes_the_tuned_linears():
    """A width of 2048: norms, biases and places folded into the single-token streaming form, the staged matrix-core form at 1, 2, 8,
    40 and 64 rows, a latent of 512, a scan of 4096 channels."""
    from bukatar_helpers import config, dense, latent, moe, prompt, scan, weights, window
    cfg = config([window(16, 4, 128, 64, 100, 16, dense(2048)), latent(16, 128, 64, 128, 512, moe(16, 4, 256, 256)), scan(4096, 16, 4, 128, dense(4096))], 2048, 1000)
    w, toks = weights(cfg), prompt(cfg, 160)
    want = _oracle_logits(cfg, w, toks)
    s = _session(cfg, w, torch.bfloat16, max_tokens=256)
    for cuts in ([160], [64, 40, 8, 2, 2, 8] + [1] * 36):
        _close(_feed(s, "r", toks, cuts), want, torch.bfloat16, str(cuts[:4]))
        s.end("r")
    for r in range(4):
        s.step([(r, toks[:50 - r])])
    lg, _ = s.step([(r, toks[50 - r:51 - r]) for r in range(4)], [[0]] * 4)
    _close(lg.cpu().double(), torch.stack([want[50 - r] for r in range(4)]), torch.bfloat16)
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
    from bukatar_helpers import CONFIGS, prompt, weights
    from oracle.bukatar_ref import BukatarOracle
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    path = _checkpoint(tmp_path, cfg, w)
    prompts = [prompt(cfg, n, seed=20 + n) for n in (70, 3, 1, 33, 64)]
    orc = BukatarOracle(cfg, w)
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
    from bukatar_helpers import CONFIGS, prompt, weights
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
                assert len(off) <= 1, off
            g.finalize()


def test_models_without_a_scan_may_speculate():
    """Rejected guesses overwrite cached rows; tokens stay those of plain greedy decoding."""
    import mirage as mi
    from generate import Generator
    from mirage.mpk import MirageModelConfig
    from bukatar_helpers import config, dense, latent, moe, prompt, weights, window
    spec = lambda: mi.mpk.spec_decode_class("promptlookup", ngram_size=2, spec_length=4)
    cfg = config([latent(4, 16, 8, 16, 32, dense(60)), window(4, 2, 24, 8, 20, 4, moe(6, 2, 24, 24))], 64, 90)
    make = lambda **kw: Generator(90, model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in weights(cfg).items()}), batch=1, max_num_batched_tokens=8,
                                  page_size=64, eos_token_id=-1, dtype=torch.float32, **kw)
    p = (prompt(cfg, 6) * 6)[:33]
    plain = make()
    want = plain.generate([p])
    plain.finalize()
    guess = make(spec_decode_config=spec())
    assert guess.generate([p]) == want
    guess.finalize()


def test_trace_replay(tmp_path, monkeypatch, capsys):
    """bin/trace_run on a checkpoint of its own: files, order of the rows, and the `done` lines."""
    import io
    import os
    import sys
    from importlib.machinery import SourceFileLoader

    import numpy as np

    from conftest import ROOT
    from bukatar_helpers import CONFIGS, prompt, weights
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
