"""Suborax on the GPU against the plain oracle: every mechanism alone, whole models of several sizes in bf16 and in 32 bits,
prompts against single tokens, portions, mixed batches, pages used again, long decoding, and greedy generation through the
framework's own entry points.  Expected values come from oracle/suborax_ref.py in float64; rows of a bf16 engine are rounded
where it stores them."""
import json

import pytest
import torch

pytestmark = pytest.mark.gpu

F64 = torch.float64


def _session(cfg, w, dtype, max_tokens=512, **kw):
    from mirage.mpk import MirageModelConfig, ServingSession
    return ServingSession.open(model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in w.items()}), dtype=dtype, max_tokens=max_tokens, **kw)


def _oracle_logits(cfg, w, toks):
    from oracle.suborax_ref import SuboraxOracle
    orc = SuboraxOracle(cfg, w)
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
    limit = 0.025 if dtype == torch.bfloat16 else 5e-6
    worst = int(err.argmax())
    assert err.max() < limit, f"{what}: position {worst} is {float(err.max())} off (limit {limit}); first over: {(err > limit).nonzero().flatten()[:8].tolist()}"


# ---------------------------------------------------------------- mechanisms alone
def _graph(rows, slots=None, page=32):
    from helpers import make_meta, make_mpk
    R = slots or rows
    return make_mpk(make_meta(R, 64, rows, R, 2 * R), 64, rows, R, 2 * R, page, mode="onepass")


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("k", [64, 70, 333])
def test_embedding_scale(dtype, k):
    import mirage as mi
    pk, V, ld = _graph(8), 50, -(-k // 4) * 4
    table = torch.randn(V, k, device="cuda").to(dtype)
    ids = pk.meta_tensors["input_tokens"]
    ids[:, 0] = torch.tensor([0, 49, 7, 7, -1, 3, 2, 1])
    r, o = torch.full((8, ld), 9.0, device="cuda"), torch.full((8, ld), 9.0, device="cuda", dtype=dtype)
    pk.embed_scaled_layer(pk.attach_input(ids, "ids"), pk.attach_input(table, "t"), pk.attach_input(r, "r"), pk.attach_input(o, "o"), scale=0.3)
    pk.compile()
    pk.run_once(list(range(8)), [0] * 8)
    want = torch.where(ids >= 0, table[ids[:, 0].clamp(min=0)].float() * torch.tensor(0.3, device="cuda"), 0.0)
    assert torch.equal(r[:, :k], want) and torch.equal(o[:, :k], want.to(dtype)) and bool((r[:, k:] == 9).all())
    pk.finalize()


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("width,ld,alpha,offset,with_y", [(64, 64, 1.0, 0.0, True), (200, 256, 2.3, 1.0, True), (4096, 4096, 0.5, 1.0, True), (130, 192, 1.0, 1.0, False), (6000, 6016, 1.4, 1.0, True)])
def test_residual_norm(dtype, width, ld, alpha, offset, with_y):
    """Several rows and one row; real entries only count, padding stays zero; both outputs."""
    import mirage as mi
    from oracle.suborax_ref import rms_divide
    pk = _graph(8)
    pad = lambda t: torch.nn.functional.pad(t, (0, ld - width))
    x, y = pad(torch.randn(8, width, device="cuda") * 3), pad(torch.randn(8, width, device="cuda")).to(dtype)
    w = pad(torch.randn(width, device="cuda"))
    xo, o = torch.zeros(8, ld, device="cuda"), torch.zeros(8, ld, device="cuda", dtype=dtype)
    a = pk.attach_input
    pk.residual_rmsnorm_layer(a(y, "y") if with_y else None, a(x, "x"), a(w, "w"), a(xo, "xo"), a(o, "o"), width=width, alpha=alpha, eps=1e-3, weight_offset=offset)
    pk.compile()
    for M in (8, 1):
        xo.zero_()
        o.zero_()
        pk.run_once(list(range(M)), [0] * M)
        v = alpha * x.double() + (y.double() if with_y else 0)
        want = torch.zeros(8, ld, dtype=F64, device="cuda")
        want[:M, :width] = rms_divide(v[:M, :width], 1e-3) * (offset + w.double()[:width])
        torch.testing.assert_close(xo.double(), want, rtol=3e-6, atol=3e-6)
        torch.testing.assert_close(o, xo.to(dtype), rtol=0, atol=0)
    pk.finalize()


@pytest.mark.parametrize("width,n", [(192, 80), (1024, 300), (2048, 512), (4096, 700)])
def test_norm_folded_into_a_single_token_linear(width, n):
    """One token: the linear forms the norm itself (every size has its own code path); several tokens: two stages.  Same
    numbers, and the new residual rows and the normalised rows are stored either way."""
    import mirage as mi
    from oracle.suborax_ref import rms_divide
    pk = _graph(16)
    x, y = torch.randn(16, width, device="cuda"), torch.randn(16, width, device="cuda").bfloat16()
    w, W = torch.randn(width, device="cuda") * 0.2, (torch.randn(n, width, device="cuda") / width ** 0.5).bfloat16()
    xo, o, z = torch.zeros(16, width, device="cuda"), torch.zeros(16, width, device="cuda").bfloat16(), torch.zeros(16, n, device="cuda").bfloat16()
    a = pk.attach_input
    oo = a(o, "o")
    pk.residual_rmsnorm_layer(a(y, "y"), a(x, "x"), a(w, "w"), a(xo, "xo"), oo, alpha=1.6, eps=1e-6, weight_offset=1.0)
    pk.linear_layer(oo, a(W, "W"), a(z, "z"), (1, 1, 1), (256, 1, 1))
    pk.compile()
    for M in (1, 2, 5, 16):
        for t in (xo, o, z):
            t.zero_()
        pk.run_once(list(range(M)), [0] * M)
        v = 1.6 * x[:M].double() + y[:M].double()
        want = rms_divide(v, 1e-6) * (1.0 + w.double())
        torch.testing.assert_close(xo[:M].double(), want, rtol=3e-6, atol=3e-6)
        assert torch.equal(o[:M], xo[:M].bfloat16()), M
        torch.testing.assert_close(z[:M].double(), o[:M].double() @ W.double().T, rtol=1e-2, atol=1e-2)
    pk.finalize()


@pytest.mark.parametrize("k,n,silu", [(64, 33, False), (192, 500, False), (448, 130, True), (2048, 64, True)])
def test_32_bit_linear(k, n, silu):
    import mirage as mi
    pk = _graph(64)
    x, wa, wb = torch.randn(64, k, device="cuda"), torch.randn(n, k, device="cuda"), torch.randn(n, k, device="cuda")
    out = torch.zeros(64, n, device="cuda")
    a = pk.attach_input
    if silu:
        mid = pk.new_tensor((64, 2 * n), dtype=mi.float32, name="mid")
        pk.linear_layer(a(x, "x"), pk.shuffle_tensors([a(wa, "wa"), a(wb, "wb")], 0, 1, "w"), mid, (1, 1, 1), (256, 1, 1))
        pk.silu_mul_layer(mid, a(out, "o"), (1, 1, 1), (256, 1, 1))
    else:
        pk.linear_layer(a(x, "x"), a(wa, "wa"), a(out, "o"), (1, 1, 1), (256, 1, 1))
    pk.compile()
    for M in (1, 17, 40, 64):
        out.zero_()
        pk.run_once(list(range(M)), [0] * M)
        want = x[:M].double() @ wa.double().T
        if silu:
            want = torch.nn.functional.silu(want) * (x[:M].double() @ wb.double().T)
        torch.testing.assert_close(out[:M].double(), want, rtol=1e-4, atol=2e-5 * float(want.abs().max()))
        assert not out[M:].any()
    pk.finalize()


def test_32_bit_sampling_takes_the_lowest_of_equal_maxima():
    import mirage as mi
    pk, V = _graph(8), 3001
    x = torch.randn(8, V, device="cuda")
    for r, at in enumerate([0, 3000, 1500, 7, 8, 2047, 2048, 11]):
        x[r, at] = 50.0
        x[r, 2900] = max(float(x[r, 2900]), 50.0 if r % 2 and at < 2900 else -1.0)
    x[4] = 1.0
    out = pk.meta_tensors["output_tokens"]
    pk.argmax_layer(pk.attach_input(x, "x"), pk.attach_input(out, "o"), (1, 1, 1), (256, 1, 1))
    pk.linear_layer(pk.attach_input(torch.zeros(8, 32, device="cuda"), "a"), pk.attach_input(torch.zeros(4, 32, device="cuda"), "b"), pk.new_tensor((8, 4), dtype=mi.float32, name="c"),
                    (1, 1, 1), (256, 1, 1))
    pk.compile()
    pk.run_once(list(range(8)), [0] * 8)
    want = [int((x[r] == x[r].max()).nonzero()[0]) for r in range(8)]
    assert out[:, 0].tolist() == want
    pk.finalize()


RIGS = {  # heads, kv heads, dim, value dim, rotated, softcap, unit norm, sink
    "gqa4": (8, 2, 64, 64, 32, 15.0, True, True),
    "one_kv_head_many_queries": (20, 1, 40, 24, 12, 8.0, True, True),
    "multi_head": (3, 3, 128, 128, 128, 30.0, True, True),
    "value_wider": (6, 2, 72, 136, 2, 0.0, True, True),
    "large_heads": (4, 2, 256, 200, 64, 20.0, True, False),
    "plain": (4, 1, 96, 64, 0, 0.0, False, False),
    "no_norm": (5, 5, 128, 48, 96, 10.0, False, True),
}


def _rig(name, dtype, **kw):
    from suborax_helpers import AttentionRig
    H, G, D, DV, rot, cap, unit, sink = RIGS[name]
    s = (torch.randn(H, generator=torch.Generator().manual_seed(5)) + 2.0) if sink else None
    return AttentionRig(H, G, D, DV, rot, 2.0 / D ** 0.5, cap, unit, s, dtype=dtype, **kw)


def _rows(rig, n, seed):
    H, G, D, DV = rig.dims
    return torch.randn(n, H * D + G * (D + DV), generator=torch.Generator().manual_seed(seed)).to(rig.dtype)


def _tol(dtype):
    return dict(rtol=1.6e-2, atol=1.6e-2) if dtype == torch.bfloat16 else dict(rtol=2e-5, atol=1e-5)


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("name", RIGS)
def test_attention_alone(name, dtype):
    """Portions, single tokens and mixtures of both, four requests on scattered pages; cache garbage never shows."""
    rig = _rig(name, dtype)
    lens = [150, 33, 70, 5]
    perm = torch.randperm(24, generator=torch.Generator().manual_seed(1)).tolist()
    pages = [perm[0:5], perm[5:7], perm[7:10], perm[10:11]]
    data = [_rows(rig, n, 10 + i) for i, n in enumerate(lens)]
    want = [rig.reference(d) for d in data]
    at = [0, 0, 0, 0]
    # (request, rows) lists: portions alone and together, two-token portions, a portion beside single tokens, all single
    plan = [[(0, 64)], [(0, 2), (1, 31), (2, 3)], [(0, 60), (1, 1), (3, 2)], [(1, 1), (2, 30), (0, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 1)], [(2, 33), (0, 2)],
            [(0, 1), (2, 1), (3, 1)], [(0, 1), (2, 1), (3, 1)], [(0, 17)], [(2, 1)]]
    for step in plan:
        got = rig.run([(r, at[r], data[r][at[r]:at[r] + n], pages[r]) for r, n in step])
        for (r, n), g in zip(step, got):
            torch.testing.assert_close(g, want[r][at[r]:at[r] + n], msg=lambda m: f"{name} request {r} rows {at[r]}..{at[r] + n}: {m}", **_tol(dtype))
            at[r] += n
    assert at == [150, 33, 70, 5]
    rig.close()


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_far_keys_and_page_borders(dtype):
    """One key per query that stands out: the query at p is a multiple of the key at j (no rotation), so nearly all weight
    sits on j.  j runs over tile, page and chunk borders, the first positions and the newest ones; single tokens and portions."""
    from suborax_helpers import AttentionRig
    H, G, D, DV, n = 4, 2, 64, 32, 700
    rig = AttentionRig(H, G, D, DV, 0, 0.35, 0.0, True, torch.full((H,), 3.0), dtype=dtype)
    rows = _rows(rig, n, 3).float()
    targets = [0, 1, 2, 15, 16, 17, 31, 32, 33, 63, 64, 65, 127, 128, 255, 256, 300, 511, 512, 513, 600, 639, 640]
    base = 650
    for i, j in enumerate(targets):
        p = base + i
        for h in range(H):
            rows[p, h * D:(h + 1) * D] = 2.0 * rows[j, H * D + (h // 2) * D:H * D + (h // 2 + 1) * D]
    rows = rows.to(dtype)
    want = rig.reference(rows)
    perm = torch.randperm(24, generator=torch.Generator().manual_seed(2)).tolist()
    for p0 in range(0, 640, 64):
        rig.run([(0, p0, rows[p0:p0 + 64], perm)])
    rig.run([(0, 640, rows[640:base], perm)])
    v = rows[:, (H + G) * D:].double().view(n, G, DV)
    for i, j in enumerate(targets):
        p = base + i
        got = rig.run([(0, p, rows[p:p + 1], perm)])[0]
        torch.testing.assert_close(got[0], want[p], msg=lambda m: f"query {p}, key {j}: {m}", **_tol(dtype))
        # the value of the key asked for is what comes out, nearly alone
        assert (got.view(H, DV)[0] - v[j, 0]).norm() < 0.2 * v[j, 0].norm(), (p, j)
    # the same queries once more as portions of two and more (rows rewritten in place)
    for lo, hi in ((650, 652), (652, 660), (660, 673)):
        got = rig.run([(0, lo, rows[lo:hi], perm)])[0]
        torch.testing.assert_close(got, want[lo:hi], **_tol(dtype))
    rig.close()


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_sink_dominates_or_vanishes(dtype):
    from suborax_helpers import AttentionRig
    H, D = 4, 32
    sink = torch.tensor([-60.0, 0.0, 20.0, 90.0])
    rig = AttentionRig(H, 2, D, D, 16, 0.5, 12.0, True, sink, dtype=dtype)
    rows = _rows(rig, 90, 8)
    want = rig.reference(rows)
    got = [rig.run([(0, 0, rows[:50], list(range(3)))])[0], rig.run([(0, 50, rows[50:89], list(range(3)))])[0], rig.run([(0, 89, rows[89:], list(range(3)))])[0]]
    got = torch.cat(got)
    torch.testing.assert_close(got, want, **_tol(dtype))
    assert float(got.view(90, H, D)[:, 3].abs().max()) < 1e-6 and float(got.view(90, H, D)[:, 2].abs().max()) < 0.1
    # the first position sees itself and the sink only
    s0 = want.view(90, H, D)[0, 0]
    torch.testing.assert_close(got.view(90, H, D)[0, 0], s0, **_tol(dtype))
    rig.close()


# ---------------------------------------------------------------- whole models
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
@pytest.mark.parametrize("name", ["even", "odd", "wide_heads", "one_layer"])
def test_prompt_portions_and_decoding_agree_with_the_oracle(name, dtype):
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS[name]
    w, toks = weights(cfg), prompt(cfg, 140)
    want = _oracle_logits(cfg, w, toks)
    s = _session(cfg, w, dtype, max_tokens=192)
    for cuts in ([140], [100] + [1] * 40, [1] * 20 + [120], [2] * 70, [3, 64, 2, 61, 1, 1, 8], [63, 1, 64, 2, 2, 7, 1]):
        _close(_feed(s, "r", toks, cuts), want, dtype, f"{name} cut as {cuts[:6]}")
        s.end("r")
    s.finalize()


def test_token_by_token_kernel():
    """max_num_batched_tokens = 1 has a kernel of its own."""
    from suborax_helpers import CONFIGS, prompt, weights
    for name in ("even", "odd"):
        cfg = CONFIGS[name]
        w, toks = weights(cfg), prompt(cfg, 75)
        s = _session(cfg, w, torch.bfloat16, max_tokens=128, max_rows=1, max_requests=1)
        _close(_feed(s, "r", toks, [75]), _oracle_logits(cfg, w, toks), torch.bfloat16, name)
        s.finalize()


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_mixed_batches_and_pages_used_again(dtype):
    """Unequal requests together, pausing and going on, ending and making room: the logits of every position are those of
    the request alone.  The pool is too small for all requests at once, so pages are used again."""
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    lens = {"a": 200, "b": 65, "c": 1, "d": 130, "e": 90, "f": 64, "g": 37}
    toks = {r: prompt(cfg, n, seed=i) for i, (r, n) in enumerate(lens.items())}
    want = {r: _oracle_logits(cfg, w, t) for r, t in toks.items()}
    s = _session(cfg, w, dtype, max_tokens=384)
    at, got, live = dict.fromkeys(lens, 0), {r: [] for r in lens}, []
    waiting, g, used = list(lens), torch.Generator().manual_seed(4), set()
    pages = lambda r: -(-lens[r] // 64)
    while waiting or live:
        while waiting and len(live) < 4 and sum(map(pages, live)) + pages(waiting[0]) <= 6:
            live.append(waiting.pop(0))
        step = []
        for r in live:
            n = [0, 1, 1, 2, 3, 17, 40, 64][int(torch.randint(0, 8, (1,), generator=g))]
            n = min(n, lens[r] - at[r])
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
            if at[r] == lens[r]:
                s.end(r)
                live.remove(r)
    assert len(s.pool) == 6 and used == set(range(6))
    for r in lens:
        _close(torch.cat(got[r]), want[r], dtype, r)
    s.finalize()


@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_long_decoding(dtype):
    """Hundreds of single tokens across page and chunk borders."""
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["one_layer"]
    w, toks = weights(cfg), prompt(cfg, 620)
    s = _session(cfg, w, dtype, max_tokens=640)
    _close(_feed(s, "r", toks, [3] + [1] * 617), _oracle_logits(cfg, w, toks), dtype)
    s.finalize()


def test_wide_model_takes_the_tuned_linears():
    """A width of 2048 and a feed-forward of 4096: the single-token streaming form, the staged matrix-core form with K
    slices left to the norm and to the attention's row fetch, at 1, 2, 8, 40 and 64 rows."""
    from suborax_helpers import config, layer, prompt, weights
    cfg = config([layer(16, 4, 128, 128, 64, 4096)] * 2, 2048, 1000)
    w, toks = weights(cfg), prompt(cfg, 200)
    want = _oracle_logits(cfg, w, toks)
    s = _session(cfg, w, torch.bfloat16, max_tokens=256)
    for cuts in ([200], [64, 40, 8, 2, 2, 8] + [1] * 76):
        _close(_feed(s, "r", toks, cuts), want, torch.bfloat16, str(cuts[:4]))
        s.end("r")
    # four requests of one token each (rows of different requests, K slices summed in the attention stage)
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
    """32-bit, so that the tokens are the oracle's: the offline engine (on-GPU scheduler, more requests than slots), the
    serving session, and the command line."""
    import generate
    from generate import Generator
    from mirage.mpk import ServingSession
    from oracle.suborax_ref import SuboraxOracle
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["odd"]
    w = weights(cfg)
    path = _checkpoint(tmp_path, cfg, w)
    prompts = [prompt(cfg, n, seed=20 + n) for n in (70, 3, 1, 33, 64)]
    orc = SuboraxOracle(cfg, w)
    want = [orc.generate(p, 20) for p in prompts]
    g = Generator(70 + 20 + 1, model_path=path, batch=2, max_num_batched_tokens=16, max_tokens_per_request=16, page_size=32, total_requests=5, eos_token_id=-1, dtype=torch.float32)
    for _ in range(2):  # the same handle serves again
        assert g.generate(prompts, 20) == want
    g.finalize()
    s = ServingSession.open(model_path=path, dtype=torch.float32, max_tokens=256, max_requests=3)
    assert s.generate(prompts, 20) == want
    assert len(s.pool) == s.pool.num_pages
    stop = want[0][75]
    cut = s.generate([prompts[0]], 20, eos_token_id=stop)[0]
    assert cut == want[0][:70 + want[0][70:].index(stop) + 1]
    s.finalize()
    # (in this process: only one process at a time may launch cooperatively)
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
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["even"]
    w = weights(cfg)
    for rows, batch in ((1, 1), (8, 4)):
        g = Generator(60, model_config=MirageModelConfig(architecture=cfg, state_dict={k: v.cuda() for k, v in w.items()}), batch=batch, max_num_batched_tokens=rows, page_size=32,
                      eos_token_id=-1)
        prompts = [prompt(cfg, 9 + i, seed=i) for i in range(batch)]
        for p, ids in zip(prompts, g.generate(prompts)):
            assert len(ids) == 60 and ids[:len(p)] == p
            lg = _oracle_logits(cfg, w, ids[:-1])
            for t in range(len(p) - 1, 59):
                assert lg[t, ids[t + 1]] > lg[t].max() - 0.15 * lg.std(), t
        g.finalize()


def test_prompt_lookup_speculation_keeps_the_tokens():
    """Speculative decoding over the flex stages: the same tokens as plain greedy decoding."""
    import mirage as mi
    from generate import Generator
    from mirage.mpk import MirageModelConfig
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["odd"]
    w = {k: v.cuda() for k, v in weights(cfg).items()}
    kw = dict(model_config=MirageModelConfig(architecture=cfg, state_dict=w), batch=1, max_num_batched_tokens=8, page_size=32, eos_token_id=-1, dtype=torch.float32)
    p = (prompt(cfg, 6) * 6)[:33]
    plain = Generator(90, **kw)
    want = plain.generate([p])
    plain.finalize()
    spec = Generator(90, spec_decode_config=mi.mpk.spec_decode_class("promptlookup", ngram_size=2, spec_length=4), **kw)
    assert spec.generate([p]) == want
    spec.finalize()


def test_static_launch_and_single_weight_copy():
    """The launch that allocates nothing, and the mode that keeps weights in tile order only, on a flex graph."""
    from generate import Generator
    from mirage.mpk import MirageModelConfig
    from suborax_helpers import config, layer, prompt, weights
    cfg = config([layer(8, 2, 64, 64, 32, 256)] * 2, 256, 300)
    w = {k: v.cuda() for k, v in weights(cfg).items()}
    make = lambda **kw: Generator(50, model_config=MirageModelConfig(architecture=cfg, state_dict=dict(w)), batch=2, max_num_batched_tokens=8, page_size=32, eos_token_id=-1, **kw)
    prompts = [prompt(cfg, 9), prompt(cfg, 17, seed=1)]
    g = make()
    want = g.generate(prompts)
    g.load_prompts(prompts)
    stream = torch.cuda.current_stream().cuda_stream
    g.mpk._g.enqueue_steps(stream, 1 << 20, static=True)
    assert g.mpk._g.wait(stream)
    assert [g.meta["tokens"][i, :50].tolist() for i in range(2)] == want
    g.finalize()
    one = make(single_weight_copy=True)
    lg = _oracle_logits(cfg, {k: v.cpu() for k, v in w.items()}, one.generate(prompts)[0][:-1])
    ids = one.generate(prompts)[0]
    assert one.mpk.stats()["row_major_weight_bytes"] == 0
    assert all(lg[t, ids[t + 1]] > lg[t].max() - 0.15 * lg.std() for t in range(8, 49))
    one.finalize()


def test_trace_replay(tmp_path, monkeypatch, capsys):
    """bin/trace_run on a checkpoint of its own: files, order of the rows, and the `done` lines."""
    import io
    import os
    import sys
    from importlib.machinery import SourceFileLoader

    import numpy as np

    from conftest import ROOT
    from suborax_helpers import CONFIGS, prompt, weights
    cfg = CONFIGS["one_layer"]
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
