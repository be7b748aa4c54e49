"""Dodonex on the GPU against the plain oracle: every mechanism alone, whole models of several sizes in bf16 and in 32 bits,
prompts against single tokens, portions, mixed batches, pages and state slots used again, long decoding, and greedy
generation through the framework's own entry points.  Expected values come from oracle/dodonex_ref.py in float64."""
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
    from oracle.dodonex_ref import DodonexOracle
    orc = DodonexOracle(cfg, w)
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


def _close(got, want, dtype, what=""):
    err = ((got - want) - (got - want).mean(-1, keepdim=True)).pow(2).mean(-1).sqrt() / want.std()
    limit = 0.04 if dtype == torch.bfloat16 else 1e-5
    worst = int(err.argmax())
    assert err.max() < limit, f"{what}: position {worst} is {float(err.max())} off (limit {limit}); first over: {(err > limit).nonzero().flatten()[:8].tolist()}"


def _graph(rows, slots=None, page=64):
    from helpers import make_meta, make_mpk
    R = slots or rows
    return make_mpk(make_meta(R, 64, rows, R, 2 * R), 64, rows, R, 2 * R, page, mode="onepass")


def _tol(dtype):
    return dict(rtol=1.6e-2, atol=1.6e-2) if dtype == torch.bfloat16 else dict(rtol=2e-5, atol=2e-5)


# ---------------------------------------------------------------- mechanisms alone
@BOTH
@pytest.mark.parametrize("width,ld,groups,with_y,with_yw,with_w", [(64, 64, 1, True, False, True), (204, 256, 3, True, True, True), (4096, 4096, 8, True, True, True),
                                                                   (130, 192, 13, False, False, True), (6000, 6016, 5, True, True, True), (96, 128, 1, True, False, False)])
def test_residual_prenorm(dtype, width, ld, groups, with_y, with_yw, with_w):
    """Several rows and one row; parts that end inside a 16-byte word; the summand normalised or not; no norm at all."""
    from oracle.dodonex_ref import group_rms_norm, rms_norm
    pk = _graph(8)
    pad = lambda t: torch.nn.functional.pad(t, (0, ld - width))
    x, y = pad(torch.randn(8, width, device="cuda") * 3), pad(torch.randn(8, width, device="cuda")).to(dtype)
    x[:, :width // 2] *= 5.0  # parts of very different size
    w, yw = pad(torch.randn(width, device="cuda")), pad(torch.randn(width, device="cuda"))
    xo, o = torch.zeros(8, ld, device="cuda"), torch.zeros(8, ld, device="cuda", dtype=dtype)
    a = pk.attach_input
    pk.residual_prenorm_layer(a(y, "y") if with_y else None, a(x, "x"), a(xo, "xo"), a(o, "o"), weight=a(w, "w") if with_w else None,
                              input_weight=a(yw, "yw") if with_yw else None, width=width, groups=groups, alpha=0.7, eps=1e-3, input_eps=1e-2)
    pk.compile()
    for M in (8, 1, 3):
        xo.zero_(), o.zero_()
        pk.run_once(list(range(M)), [0] * M)
        v, s = x[:M, :width].double(), y[:M, :width].double()
        if with_y:
            v = v + 0.7 * (rms_norm(s, yw[:width].double(), 1e-2) if with_yw else s)
        n = group_rms_norm(v, w[:width].double(), 1e-3, groups) if with_w else v
        torch.testing.assert_close(xo[:M, :width].double(), v, rtol=3e-6, atol=3e-6)
        torch.testing.assert_close(o[:M, :width].double(), n.to(dtype).double(), rtol=8e-3 if dtype == torch.bfloat16 else 3e-6, atol=3e-6)
        assert not xo[:, width:].any() and not o[:, width:].any() and not o[M:].any()
    pk.finalize()


@pytest.mark.parametrize("width,n,groups", [(192, 80, 3), (1024, 300, 2), (2048, 512, 8), (4096, 700, 4), (4096, 130, 32), (1536, 90, 1)])
def test_norm_folded_into_a_single_token_linear(width, n, groups):
    """One token: the linear forms sum and norm itself (by the control wavefront or by the workgroup); several: two stages."""
    from oracle.dodonex_ref import group_rms_norm, rms_norm
    pk = _graph(16)
    x, y = torch.randn(16, width, device="cuda"), torch.randn(16, width, device="cuda").bfloat16()
    w, yw, W = torch.randn(width, device="cuda"), torch.randn(width, device="cuda"), (torch.randn(n, width, device="cuda") / width ** 0.5).bfloat16()
    xo, o, z = torch.zeros(16, width, device="cuda"), torch.zeros(16, width, device="cuda").bfloat16(), torch.zeros(16, n, device="cuda").bfloat16()
    a = pk.attach_input
    oo = a(o, "o")
    pk.residual_prenorm_layer(a(y, "y"), a(x, "x"), a(xo, "xo"), oo, weight=a(w, "w"), input_weight=a(yw, "yw"), groups=groups, alpha=1.6, eps=1e-5, input_eps=1e-4)
    pk.linear_layer(oo, a(W, "W"), a(z, "z"), (1, 1, 1), (256, 1, 1))
    pk.compile()
    for M in (1, 2, 5, 16):
        for t in (xo, o, z):
            t.zero_()
        pk.run_once(list(range(M)), [0] * M)
        v = x[:M].double() + 1.6 * rms_norm(y[:M].double(), yw.double(), 1e-4)
        torch.testing.assert_close(xo[:M].double(), v, rtol=3e-6, atol=3e-6)
        torch.testing.assert_close(o[:M].double(), group_rms_norm(v, w.double(), 1e-5, groups), rtol=8e-3, atol=1e-5)
        torch.testing.assert_close(z[:M].double(), o[:M].double() @ W.double().T, rtol=1e-2, atol=1.5e-2)
    pk.finalize()


@pytest.mark.parametrize("k,n", [(64, 70), (256, 2048), (448, 36), (1536, 300), (2048, 256), (6144, 515), (12288, 130), (16384, 2000)])
def test_linear_joins_the_stream(k, n):
    """One token: the linear adds its result to the residual stream; several: two stages.  All reduction lengths."""
    pk, ld = _graph(8), -(-n // 64) * 64
    x, W = torch.randn(8, k, device="cuda").bfloat16(), (torch.randn(n, k, device="cuda") / k ** 0.5).bfloat16()
    res = torch.nn.functional.pad(torch.randn(8, n, device="cuda"), (0, ld - n))
    y, xo, o = torch.zeros(8, ld, device="cuda").bfloat16(), torch.zeros(8, ld, device="cuda"), torch.zeros(8, ld, device="cuda").bfloat16()
    a = pk.attach_input
    yy = a(y, "y")
    pk.linear_layer(a(x, "x"), a(W, "W"), yy, (1, 1, 1), (256, 1, 1))
    pk.residual_prenorm_layer(yy, a(res, "res"), a(xo, "xo"), a(o, "o"), width=n, alpha=0.5)
    pk.compile()
    assert "[multi-token only]" in pk.describe_program()
    for M in (1, 2, 8):
        xo.zero_(), o.zero_()
        pk.run_once(list(range(M)), [0] * M)
        want = res[:M, :n].double() + 0.5 * (x[:M].double() @ W.double().T)
        torch.testing.assert_close(xo[:M, :n].double(), want, rtol=1e-5 if M == 1 else 1e-2, atol=1e-5 if M == 1 else 1e-2)
        assert torch.equal(o[:M], xo[:M].bfloat16()) and not xo[:, n:].any()
    pk.finalize()


@BOTH
@pytest.mark.parametrize("heads,n,k,extra_in,extra_out", [(1, 20, 64, 0, 0), (7, 40, 96, 32, 3), (3, 24, 512, 0, 8), (40, 128, 128, 64, 0), (2, 300, 32, 0, 1)])
def test_head_linear(dtype, heads, n, k, extra_in, extra_out):
    from mirage.mpk.persistent_kernel import operand_tiles
    pk = _graph(64)
    i, o = k + extra_in, n + extra_out
    x, W = torch.randn(64, heads * i, device="cuda").to(dtype), (torch.randn(heads, n, k, device="cuda") / k ** 0.5).to(dtype)
    out = torch.zeros(64, heads * o, device="cuda", dtype=dtype)
    a = pk.attach_input
    pk.head_linear_layer(a(x, "x"), a(operand_tiles(W), "W"), a(out, "o"), heads, n, k, i, o)
    pk.compile()
    for M in (1, 5, 17, 64):
        out.zero_()
        pk.run_once(list(range(M)), [0] * M)
        want = torch.einsum("thk,hnk->thn", x[:M].view(M, heads, i)[:, :, :k].cpu().double(), W.cpu().double())
        torch.testing.assert_close(out[:M].view(M, heads, o)[:, :, :n].cpu().double(), want, rtol=1e-2 if dtype == torch.bfloat16 else 1e-4, atol=1e-2 if dtype == torch.bfloat16 else 1e-5)
        assert not out[:M].view(M, heads, o)[:, :, n:].any() and not out[M:].any()
    pk.finalize()


@BOTH
@pytest.mark.parametrize("n,k,column", [(7, 64, 3), (24, 448, 0), (256, 2048, 256), (200, 192, 40)])
def test_gelu_times_a_table_row(dtype, n, k, column):
    from mirage.mpk.persistent_kernel import operand_tiles
    from oracle.dodonex_ref import gelu_tanh
    pk, V, ld = _graph(64), 11, -(-n // 64) * 64
    x, W, table = torch.randn(64, k, device="cuda").to(dtype), (2 * torch.randn(1, n, k, device="cuda") / k ** 0.5).to(dtype), torch.randn(V, column + n + 5, device="cuda").to(dtype)
    out, ids = torch.zeros(64, ld, device="cuda", dtype=dtype), pk.meta_tensors["input_tokens"]
    ids[:, 0] = torch.arange(64) % V
    ids[4, 0] = -1  # no token: nothing joins
    a = pk.attach_input
    pk.head_linear_layer(a(x, "x"), a(operand_tiles(W), "W"), a(out, "o"), 1, n, k, 0, 0, ids=a(ids, "ids"), table=a(table, "t"), table_column=column)
    pk.compile()
    for M in (1, 6, 64):
        out.zero_()
        pk.run_once(list(range(M)), [0] * M)
        e = torch.where(ids[:M] >= 0, table[ids[:M, 0].clamp(min=0), column:column + n].float(), 0.0).double()
        torch.testing.assert_close(out[:M, :n].double(), gelu_tanh(x[:M].double() @ W[0].double().T) * e, rtol=1e-2 if dtype == torch.bfloat16 else 1e-4,
                                   atol=1e-2 if dtype == torch.bfloat16 else 2e-5)
        assert not out[:, n:].any()
    pk.finalize()


@BOTH
@pytest.mark.parametrize("limit", [0.3, 2.0, 50.0])
def test_gated_activation(dtype, limit):
    """Beside the query latent: gate and up clamped on their own sides, values on both sides of the limit."""
    from oracle.dodonex_ref import clamped_glu
    pk, F, q = _graph(64), 1100, 300
    x = torch.zeros(64, q + 2 * F + 12, device="cuda").to(dtype)
    x[:, q:] = 3 * torch.randn(64, 2 * F + 12, device="cuda")
    x[:, :q] = torch.randn(64, q, device="cuda")
    cq, act, wq = torch.zeros(64, q, device="cuda", dtype=dtype), torch.zeros(64, F + 64, device="cuda", dtype=dtype), torch.ones(q, device="cuda")
    a = pk.attach_input
    pk.latent_prep_layer(a(x, "x"), a(wq, "wq"), a(cq, "cq"), 0, q, 1e-6, glu=(a(act, "act"), 64, F, q + 8, q + F + 12, limit, 1.702, 1.0))
    pk.compile()
    for M in (1, 33, 64):
        act.zero_()
        pk.run_once(list(range(M)), [0] * M)
        want = clamped_glu(x[:M, q + 8:q + 8 + F].double(), x[:M, q + F + 12:q + 12 + 2 * F].double(), limit)
        torch.testing.assert_close(act[:M, 64:].double(), want, rtol=1e-2 if dtype == torch.bfloat16 else 1e-5, atol=1e-5)
        assert not act[:, :64].any() and not act[M:].any()
    pk.finalize()


LATENTS = {"one_head": (1, 16, 8), "odd": (5, 36, 12), "wide": (20, 128, 64), "no_rotation": (3, 48, 0), "large": (9, 512, 64), "largest": (33, 500, 128)}


@BOTH
@pytest.mark.parametrize("name", LATENTS)
def test_latent_attention_alone(name, dtype):
    """Portions, single tokens and mixtures of both, four requests on scattered pages; cache garbage never shows."""
    from dodonex_helpers import LatentRig
    rig = LatentRig(*LATENTS[name], dtype)
    lens = [210, 33, 70, 5]
    perm = torch.randperm(14, generator=torch.Generator().manual_seed(1)).tolist()
    pages = [perm[0:4], perm[4:5], perm[5:7], perm[7:8]]
    data = [rig.data(n, 10 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    at = [0, 0, 0, 0]
    plan = [[(0, 64)], [(0, 2), (1, 31), (2, 3)], [(0, 60), (1, 1), (3, 2)], [(1, 1), (2, 30), (0, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 1)], [(2, 33), (0, 2)],
            [(0, 1), (2, 1), (3, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 17)], [(2, 1)], [(0, 60)]]
    for step in plan:
        got = rig.run([(r, at[r], [t[at[r]:at[r] + n] for t in data[r]], pages[r]) for r, n in step])
        for (r, n), (o, cq) in zip(step, got):
            torch.testing.assert_close(o, want[r][0][at[r]:at[r] + n], msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **_tol(dtype))
            torch.testing.assert_close(cq, want[r][1][at[r]:at[r] + n], **_tol(dtype))
            at[r] += n
    assert at == lens
    rig.pk.finalize()


@BOTH
@pytest.mark.parametrize("name", ["odd", "large"])
def test_far_latents_and_page_borders(name, dtype):
    """One latent per query stands out (the query is a multiple of it), at tile, page and chunk borders, the first positions and
    the newest ones; single tokens and portions."""
    from dodonex_helpers import LatentRig
    H, R, rot = LATENTS[name]
    rig, n = LatentRig(H, R, rot, dtype, scale=8.0 / R), 700
    data = rig.data(n, 3)
    from oracle.dodonex_ref import rms_norm
    cn = rms_norm(data[2], rig.wc.double(), rig.eps)
    targets, base = [0, 1, 2, 15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 255, 256, 300, 511, 512, 513, 600, 639, 640], 650
    for i, j in enumerate(targets):
        data[0][base + i] = (1.5 * cn[j]).to(dtype).double()
    want = rig.reference(data)[0]
    part = lambda lo, hi: [t[lo:hi] for t in data]
    perm = torch.randperm(14, generator=torch.Generator().manual_seed(2)).tolist()
    for p0 in range(0, 640, 64):
        rig.run([(0, p0, part(p0, p0 + 64), perm)])
    rig.run([(0, 640, part(640, base), perm)])
    for i, j in enumerate(targets):
        p = base + i
        got = rig.run([(0, p, part(p, p + 1), perm)])[0][0]
        torch.testing.assert_close(got[0], want[p], msg=lambda m: f"query {p}, key {j}: {m}", **_tol(dtype))
        assert (got[0, 0] - cn[j]).norm() < 0.25 * cn[j].norm(), (p, j)  # what comes out is the latent asked for, nearly alone
    for lo, hi in ((650, 652), (652, 660), (660, 673)):
        torch.testing.assert_close(rig.run([(0, lo, part(lo, hi), perm)])[0][0], want[lo:hi], **_tol(dtype))
    rig.pk.finalize()


DELTAS = {"tiny": (2, 8, 4), "odd": (3, 20, 12), "even": (6, 64, 32), "pad": (5, 72, 40), "wide": (4, 128, 100), "widest": (2, 200, 33), "many": (40, 32, 16), "full": (1, 256, 64)}


@BOTH
@pytest.mark.parametrize("name", DELTAS)
def test_delta_rule_alone(name, dtype):
    """Portions, single tokens and mixtures; a slot that is used again starts from zero whatever it holds (NaN at first)."""
    from dodonex_helpers import DeltaRig
    rig = DeltaRig(*DELTAS[name], dtype)
    lens = [101, 38, 40, 5, 30]
    data = [rig.data(n, 20 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    at, slot = [0] * 5, [2, 0, 3, 1, 1]
    plan = [[(0, 64)], [(0, 2), (1, 31), (2, 3)], [(0, 8), (1, 1), (3, 2)], [(1, 1), (2, 30), (0, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 1)], [(2, 3), (0, 3)],
            [(0, 1), (2, 1), (3, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 17)], [(4, 1), (1, 1), (2, 1)], [(4, 17), (1, 4), (0, 1)], [(4, 1)], [(4, 11), (0, 1)]]
    for step in plan:
        got = rig.run([(slot[r], at[r], [t[at[r]:at[r] + n] for t in data[r]]) for r, n in step])
        for (r, n), o in zip(step, got):
            torch.testing.assert_close(o, want[r][at[r]:at[r] + n], msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **_tol(dtype))
            at[r] += n
    assert at == lens
    rig.close()


def test_delta_rule_many_requests_and_long_memory():
    """64 requests of one token each (several units per workgroup), and a first token that is still there after 300 others."""
    from dodonex_helpers import DeltaRig
    rig = DeltaRig(6, 64, 32, torch.float32, slots=64, w0=-30.0)  # (decay one)
    data = [rig.data(3, 100 + i) for i in range(64)]
    want = [rig.reference(d) for d in data]
    for t in range(3):
        for r, o in enumerate(rig.run([((5 * r) % 64, t, [x[t:t + 1] for x in data[r]]) for r in range(64)])):
            torch.testing.assert_close(o[0], want[r][t], **_tol(torch.float32))
    n = 300
    d = rig.data(n, 7)
    d[4] -= 40.0  # nothing is removed ...
    d[1][1:] *= 0.02  # ... and the later keys are faint
    d[0][-1] = d[1][0]  # the last query is the first key
    want, at = rig.reference(d), 0
    for m in [64, 2, 1, 64, 1, 1, 40, 64] + [1] * 63:
        o = rig.run([(3, at, [x[at:at + m] for x in d])])[0]
        at += m
    assert at == n
    torch.testing.assert_close(o[0], want[-1], **_tol(torch.float32))
    bare = (d[2][0] * torch.sigmoid(d[3][-1])) * rig.nw.double()
    assert (torch.nn.functional.cosine_similarity(o[0], bare, dim=-1) > 0.9).all()
    rig.close()


# ---------------------------------------------------------------- whole models
@BOTH
@pytest.mark.parametrize("name", ["even", "odd", "wide", "deep_state"])
def test_prompt_portions_and_decoding_agree_with_the_oracle(name, dtype):
    from dodonex_helpers import CONFIGS, prompt, weights
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
    from dodonex_helpers import CONFIGS, prompt, weights
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
        _close(torch.cat(got[r]), want[r], dtype, r)
    for r in range(4):
        s.step([(r, toks["a"][:2])])
    with pytest.raises(RuntimeError, match="state slots"):
        s.step([("one too many", [1])])
    s.finalize()


@BOTH
def test_long_decoding(dtype):
    """Hundreds of single tokens across page and chunk borders."""
    from dodonex_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["even"]
    w, toks = weights(cfg), prompt(cfg, 420)
    s = _session(cfg, w, dtype, max_tokens=448)
    _close(_feed(s, "r", toks, [3] + [1] * 417), _oracle_logits(cfg, w, toks), dtype)
    s.finalize()


def test_wide_model_takes_the_tuned_linears():
    """A width of 2048: norms folded into the single-token streaming form, joined linears, the staged matrix-core form at 1, 2, 8,
    40 and 64 rows, a latent of 512."""
    from dodonex_helpers import config, delta, latent, prompt, weights
    cfg = config([latent(16, 128, 64, 128, 768, 512, 2048), delta(32, 64, 64, 2048)], 2048, 1000, side=256)
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
    cfg = json.loads(json.dumps(cfg))
    for l in cfg["layers"]:
        l["mixer"].pop("low_rank", None)  # the weights say it
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    return str(tmp_path)


def test_greedy_generation_from_a_checkpoint(tmp_path, capsys):
    """32-bit, so that the tokens are the oracle's: the offline engine with two and with three batch slots for five requests (the
    on-GPU schedulers move requests, and with them their states, between slots), the serving session, the command line."""
    import generate
    from generate import Generator
    from mirage.mpk import ServingSession
    from dodonex_helpers import CONFIGS, prompt, weights
    from oracle.dodonex_ref import DodonexOracle
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    path = _checkpoint(tmp_path, cfg, w)
    prompts = [prompt(cfg, n, seed=20 + n) for n in (70, 3, 1, 33, 64)]
    orc = DodonexOracle(cfg, w)
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
    stop = want[0][75]
    cut = s.generate([prompts[0]], 20, eos_token_id=stop)[0]
    assert cut == want[0][:70 + want[0][70:].index(stop) + 1]
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
    from dodonex_helpers import CONFIGS, prompt, weights
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
                for t in range(len(p) - 1, 79):
                    assert lg[t, ids[t + 1]] > lg[t].max() - 0.15 * lg.std(), t
            g.finalize()


def test_speculation_is_refused_and_latent_models_may_speculate():
    """Rejected guesses cannot leave a recurrent state; a model of latent attention alone keeps plain greedy tokens."""
    import mirage as mi
    from generate import Generator
    from mirage.mpk import MirageModelConfig
    from dodonex_helpers import CONFIGS, config, latent, prompt, weights
    spec = lambda: mi.mpk.spec_decode_class("promptlookup", ngram_size=2, spec_length=4)
    make = lambda cfg, **kw: Generator(90, model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in weights(cfg).items()}), batch=1,
                                       max_num_batched_tokens=8, page_size=64, eos_token_id=-1, dtype=torch.float32, **kw)
    with pytest.raises(NotImplementedError, match="recurrent"):
        make(CONFIGS["even"], spec_decode_config=spec())
    cfg = config([latent(4, 16, 8, 16, 24, 32, 60), latent(2, 24, 8, 16, 24, 32, None, kv_from=0)], 64, 90, groups=2)
    p = (prompt(cfg, 6) * 6)[:33]
    plain = make(cfg)
    want = plain.generate([p])
    plain.finalize()
    guess = make(cfg, spec_decode_config=spec())
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
    from dodonex_helpers import CONFIGS, prompt, weights
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
    assert sorted(f.name for f in out.iterdir()) == ["0.f32", "2.f32"]
    want = _oracle_logits(cfg, w, toks)
    read = lambda n: torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, cfg["vocab"])).double()
    _close(read(0), want[[69, 3]], torch.float32)
    _close(read(2), want[[1, 70]], torch.float32)
