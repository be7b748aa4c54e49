"""Dodonex without a GPU: the oracle's mechanisms against closed forms, the product's host side (config reader, operand order,
registry, graph lowering, state-slot bookkeeping), and what each mechanism is worth in the numbers."""
import json
import math

import pytest
import torch

from oracle.dodonex_ref import (DodonexOracle, clamped_glu, decay, delta_scan, delta_step, gelu_tanh, group_rms_norm, latent_attention_core, rms_norm, rotate_half, unit_key)
from dodonex_helpers import CONFIGS, config, delta, latent, prompt, weights

F64 = torch.float64


# ---------------------------------------------------------------- oracle mechanisms
def test_norm_in_parts():
    x = torch.tensor([[3.0, -4.0, 30.0, 40.0]], dtype=F64)
    w = torch.tensor([1.0, 2.0, 1.0, 1.0], dtype=F64)
    y = group_rms_norm(x, w, 0.5, 2)
    assert torch.allclose(y, torch.tensor([[3.0, -8.0, 0.0, 0.0]], dtype=F64) / math.sqrt(13.0) + torch.tensor([[0.0, 0.0, 30.0, 40.0]], dtype=F64) / math.sqrt(1250.5))
    assert torch.allclose(group_rms_norm(x, w, 0.5, 1), rms_norm(x, w, 0.5))


def test_rotation_is_a_complex_product():
    x, pos = torch.randn(4, 3, 10, dtype=F64), torch.tensor([0, 1, 77, 4000])
    f = torch.tensor([55.0 ** (-2 * i / 10) for i in range(5)], dtype=F64)
    z = torch.complex(x[..., :5], x[..., 5:]) * torch.polar(torch.ones(1, dtype=F64), pos[:, None, None].double() * f)
    assert torch.allclose(rotate_half(x, pos, 55.0), torch.cat([z.real, z.imag], -1))


def test_gelu_and_gated_activation():
    z = torch.linspace(-4, 4, 33, dtype=F64)
    assert (gelu_tanh(z) - torch.nn.functional.gelu(z)).abs().max() < 1e-3 and torch.allclose(gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh"))
    g, u = torch.tensor([5.0, -5.0, 0.5], dtype=F64), torch.tensor([-5.0, 5.0, 0.25], dtype=F64)
    s = lambda x: x / (1 + math.exp(-1.702 * x))
    assert torch.allclose(clamped_glu(g, u, 2.0), torch.tensor([s(2.0) * -1.0, s(-5.0) * 3.0, s(0.5) * 1.25], dtype=F64))


def test_latent_attention_in_the_latent_space_is_the_same():
    """Scores and sums formed per head (the oracle) and with the head's matrices moved to the query and the result."""
    g = torch.Generator().manual_seed(0)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=F64)
    T, H, D, P, E, R = 6, 3, 5, 4, 7, 9
    q, qr, c, kr, uk, uv, pos = rnd(T, H, D), rnd(T, H, P), rnd(T, R), rnd(T, P), rnd(H, D, R), rnd(H, E, R), torch.arange(T)
    want = latent_attention_core(q, qr, c, kr, uk, uv, pos, 0.3)
    eye = torch.eye(R, dtype=F64).expand(H, -1, -1)
    lat = latent_attention_core(torch.einsum("thd,hdr->thr", q, uk), qr, c, kr, eye, eye, pos, 0.3)
    assert torch.allclose(torch.einsum("thr,her->the", lat, uv), want)
    c2 = c.clone()
    c2[4:] = 50.0
    assert torch.allclose(latent_attention_core(q, qr, c2, kr, uk, uv, pos, 0.3)[:4], want[:4])  # causal


def test_delta_rule_writes_removes_and_forgets():
    D, E = 4, 3
    k, v, one, zero = torch.tensor([2.0, 0, 0, 0], dtype=F64), torch.tensor([1.0, 2, 3], dtype=F64), torch.ones(D, dtype=F64), torch.zeros(D, dtype=F64)
    S, o = delta_step(torch.zeros(D, E, dtype=F64), k, one, zero, k, v)
    assert torch.allclose(o, 4.0 * v) and torch.allclose(S[0], 2.0 * v)  # a first token is written as it is
    S2, _ = delta_step(S, k, one, one, k, torch.zeros(E, dtype=F64))
    assert S2.abs().max() < 1e-5  # removal along the key empties the row
    S3, _ = delta_step(S, k, 0.5 * one, zero, zero + 1e-9, v)
    assert torch.allclose(S3, 0.5 * S, atol=1e-8)  # decay only
    assert torch.allclose(unit_key(k), k / 2) and decay(torch.tensor(-80.0, dtype=F64)) == 1.0 and decay(torch.tensor(80.0, dtype=F64)) == pytest.approx(math.exp(-math.exp(-0.5)))
    # both terms read the old state: decayed and removed, not removed from what has decayed
    S4, _ = delta_step(S, k, 0.25 * one, one, k, torch.zeros(E, dtype=F64))
    assert torch.allclose(S4[0], (0.25 - 1.0) * S[0], atol=1e-6)


def test_scan_is_the_steps():
    g = torch.Generator().manual_seed(1)
    x = [torch.randn(5, 2, 6, generator=g, dtype=F64) for _ in range(5)]
    r, w, a, k, v = x[0], torch.sigmoid(x[1]), torch.sigmoid(x[2]), x[3], x[4]
    S, o = delta_scan(torch.zeros(2, 6, 6, dtype=F64), r, w, a, k, v)
    s = torch.zeros(6, 6, dtype=F64)
    for t in range(5):
        s, ot = delta_step(s, r[t, 1], w[t, 1], a[t, 1], k[t, 1], v[t, 1])
        assert torch.equal(ot, o[t, 1])
    assert torch.equal(s, S[1])


@pytest.mark.parametrize("name", CONFIGS)
def test_oracle_in_pieces_equals_oracle_at_once(name):
    c = CONFIGS[name]
    orc, toks = DodonexOracle(c, weights(c)), prompt(c, 40)
    whole = orc.forward(toks, orc.new_state(), 0)
    st, at, out = orc.new_state(), 0, []
    for n in (2, 7, 1, 1, 20, 9):
        out.append(orc.forward(toks[at:at + n], st, at))
        at += n
    assert torch.allclose(torch.cat(out), whole, atol=1e-9)


@pytest.mark.parametrize("what", ["groups", "scale", "rotation", "kv_from", "limit", "mult", "logit", "side", "side_slice", "decay", "removal", "far", "state"])
def test_a_mistake_in_one_mechanism_shows_in_the_logits(what):
    """The small models of the GPU tests are sensitive enough: each mechanism done wrong (here, in the oracle) moves the logits by
    more than the tolerances those tests use."""
    c = json.loads(json.dumps(CONFIGS["odd"]))
    if what == "kv_from":  # two layers whose latents have the same form
        c = config([latent(5, 24, 12, 20, 44, 36, 50), latent(5, 24, 12, 20, 44, 36, 50), latent(9, 40, 12, 28, 30, 36, 50, kv_from=0)], 84, 133, groups=3)
    w, toks = weights(c), prompt(c, 100)
    orc = DodonexOracle(c, w)
    good = orc.forward(toks, orc.new_state(), 0)
    b = json.loads(json.dumps(c))
    bw = dict(w)
    latents = [l["mixer"] for l in b["layers"] if l["type"] == "latent_attention"]
    if what == "groups":
        b["norm"]["groups"] = 1
    elif what == "scale":
        for m in latents:
            m["scale"] *= 1.5
    elif what == "rotation":
        for m in latents:
            m["rot"]["base"] = 1e9
    elif what == "kv_from":
        b["layers"][2]["mixer"]["kv_from"] = 1
    elif what == "limit":
        for l in b["layers"]:
            if l["mlp"]:
                l["mlp"]["limit"] = 1e9
    elif what == "mult":
        b["residual_mult"] = 1.0
    elif what == "logit":
        b["logit_scale"] = 1.0
    elif what == "side":
        bw = {n: (torch.zeros_like(t) if n == "side.embed" else t) for n, t in w.items()}
    elif what == "side_slice":
        bw["side.embed"] = torch.roll(w["side.embed"], 1, dims=1)
    elif what == "decay":
        bw = {n: (torch.zeros_like(t) if n.endswith("mix.w2") else t) for n, t in w.items()}
    elif what == "removal":
        bw = {n: (torch.full_like(t, -50.0) if n.endswith("a.b") else t) for n, t in w.items()}
    bad = DodonexOracle(b, bw)
    st = bad.new_state()
    if what in ("far", "state"):  # what the first 32 tokens left is lost between two portions
        a = bad.forward(toks[:64], st, 0)
        for s in st:
            if what == "far" and s.c is not None:
                s.c[:32] = 0
            if what == "state" and s.S is not None:
                s.S = torch.zeros_like(s.S)
        got = torch.cat([a, bad.forward(toks[64:], st, 64)])
    else:
        got = bad.forward(toks, st, 0)
    err = ((got - good)[64:].pow(2).mean(-1).sqrt() / good.std()).median()
    assert err > 0.05, float(err)


# ---------------------------------------------------------------- product, host side
def test_config_reader():
    from mirage.mpk.models.dodonex.builder import DeltaMixer, DodonexConfig, LatentMixer
    c = DodonexConfig.from_dict(CONFIGS["odd"])
    assert (c.vocab, c.width, c.groups, c.residual_mult, c.embedding_scale, c.logit_scale, c.side_dim, c.eps) == (133, 84, 3, 1.3, 1.0, 2.0, 23, 1e-4)
    assert [type(l.mixer) for l in c.layers] == [DeltaMixer, LatentMixer, DeltaMixer, LatentMixer, LatentMixer] and [l.ff for l in c.layers] == [75, None, None, 50, 90]
    s = c.tensor_shapes()
    assert s["l3.mix.uq"] == (9 * 52, 30) and "l3.mix.dkv" not in s and s["l1.mix.dkv"] == (48, 84) and s["l0.mix.w2"] == (60, 12) and "l1.mlp.gate" not in s
    assert s["side.embed"] == (133, 5 * 23) and s["l4.mix.uv"] == (16, 22)
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 0, "mlp", "kind"), "other"), (("layers", 3, "mixer", "kv_from"), 0), (("layers", 3, "mixer", "kv_from"), 4),
                        (("layers", 3, "mixer", "kv_rank"), 40), (("layers", 1, "mixer", "rot", "dims"), 8), (("norm", "groups"), 5)):
        bad = json.loads(json.dumps(CONFIGS["odd"]))
        d = bad
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            DodonexConfig.from_dict(bad)


def test_low_rank_comes_from_the_weights():
    from mirage.mpk.models.dodonex.builder import DodonexConfig
    b = json.loads(json.dumps(CONFIGS["even"]))
    del b["layers"][1]["mixer"]["low_rank"]
    c = DodonexConfig.from_dict(b)
    c.read_low_ranks(weights(CONFIGS["even"]))
    assert c.tensor_shapes() == DodonexConfig.from_dict(CONFIGS["even"]).tensor_shapes()
    with pytest.raises(KeyError, match="l1.mix.w1"):
        DodonexConfig.from_dict(b).read_low_ranks({})


def test_registry_picks_the_builder_by_config():
    from mirage.mpk.model_registry import get_builder, model_name_of
    from mirage.mpk.models.dodonex import DodonexBuilder
    assert get_builder(model_name_of({"architecture": "Dodonex"})) is DodonexBuilder
    assert DodonexBuilder.kernels(torch.float32, 64) == ("MIX_F32",) and DodonexBuilder.kernels(torch.bfloat16, 1) == ("MIX_M1",)


@pytest.mark.parametrize("dtype,kw", [(torch.bfloat16, 32), (torch.float32, 16)])
def test_operand_order(dtype, kw):
    """Lane l of operand row s of row tile t holds W[16 t + l % 16][s kw + (l // 16) (kw / 4) ...]."""
    from mirage.mpk.persistent_kernel import latent_row_dim, operand_tiles
    W = torch.arange(2 * 20 * 70, dtype=torch.float32).view(2, 20, 70).to(dtype)
    t = operand_tiles(W).view(2, 2, -(-70 // kw), 64, kw // 4)
    padded = torch.nn.functional.pad(W, (0, -70 % kw, 0, 12))
    for h, tile, s, lane in ((0, 0, 0, 0), (1, 1, 2, 37), (1, 0, 1, 63), (0, 1, 0, 5)):
        k = s * kw + (lane // 16) * (kw // 4)
        assert torch.equal(t[h, tile, s, lane], padded[h, tile * 16 + lane % 16, k:k + kw // 4])
    assert latent_row_dim(36, 12, dtype) == (96 if kw == 32 else 64) and latent_row_dim(64, 0, dtype) == 64


def _host_mpk(c, dtype=torch.bfloat16, B=64, **kw):
    from mirage.mpk import MPK, MirageModelConfig, MPKMetadata
    m = MPK(MPKMetadata(**{**dict(mode="online_notoken", max_seq_length=256, max_num_batched_requests=min(4, B), max_num_batched_tokens=B, max_num_pages=8, page_size=64, device="cpu",
                                  num_workers=256, dtype=dtype, model_config=MirageModelConfig(architecture=c, state_dict=weights(c))), **kw}))
    m.build()
    return m


def _ops(m):
    return [l.split()[1] for l in m.persistent_kernel.describe_program().splitlines()]


def test_lowering():
    """The stage program of the two kinds of layer: the norm in front folded into the linear of single-token iterations, the output
    linear joining the stream by itself there, one cache for the layers that share it."""
    c = config([latent(4, 16, 8, 16, 24, 32, 48), delta(2, 16, 8, 48), latent(2, 16, 8, 16, 24, 32, None, kv_from=0)], 64, 90)
    join = ["MX_PRENORM[multi-token", "MX_HEAD_LINEAR", "LINEAR"]
    att = ["MX_PRENORM[multi-token", "LINEAR", "MX_LATENT_PREP", "LINEAR", "MX_HEAD_LINEAR", "MX_LATENT_ATTN", "MX_LATENT_MERGE[split", "MX_HEAD_LINEAR", "LINEAR"] + join
    rec = ["MX_PRENORM[multi-token", "LINEAR", "MX_DECAY", "MX_DELTA", "MX_DELTA_OUT[sliced]", "LINEAR"] + join
    m = _host_mpk(c)
    assert _ops(m) == ["FX_EMBED"] + att + rec + att + ["MX_PRENORM[multi-token", "LINEAR", "ARGMAX_PARTIAL", "ARGMAX_REDUCE"]
    assert len(m.model_builder.latent_cache) == 1 and len(m.model_builder.state) == 1
    assert len(json.loads(m.generate_task_graph()["json_file"])["all_tasks"]) > 2
    f32 = _ops(_host_mpk(c, torch.float32))
    assert f32.count("LINEAR_F32") == 12 and "MX_PRENORM[multi-token" not in f32 and f32.count("MX_PRENORM") == 7


def test_builder_refuses_what_does_not_fit():
    from mirage.mpk import MirageModelConfig
    import mirage as mi
    c = CONFIGS["even"]
    for change, match in ((lambda w: w.pop("l1.mix.w0"), "l1.mix.w0"), (lambda w: w.update({"l0.mix.uk": w["l0.mix.uk"][:-1]}), "l0.mix.uk")):
        w = weights(c)
        change(w)
        with pytest.raises((KeyError, ValueError), match=match):
            _host_mpk(c, model_config=MirageModelConfig(architecture=c, state_dict=w))
    with pytest.raises(NotImplementedError, match="recurrent"):
        _host_mpk(c, mode="offline", total_num_requests=1, max_num_pages=16, spec_decode_config=mi.mpk.spec_decode_class("promptlookup", ngram_size=2, spec_length=4))


def test_lowering_refuses_what_does_not_fit():
    m = _host_mpk(CONFIGS["even"], page_size=48, max_num_pages=6)
    with pytest.raises(Exception, match="page_size"):
        m.persistent_kernel.describe_program()
    m = _host_mpk(config([latent(2, 16, 8, 16, 24, 600, 48)], 64, 90))
    with pytest.raises(Exception, match="512"):
        m.persistent_kernel.describe_program()


def test_mix_tasks_check_their_operands():
    import mirage as mi
    from helpers import make_meta, make_mpk
    pk = make_mpk(make_meta(2, 64, 8, 2, 4, device="cpu"), 64, 8, 2, 4, 64, num_workers=256)
    new = lambda name, cols, dt=mi.float32: pk.new_tensor((8, cols), dtype=dt, name=name)
    x, o, w = new("x", 64), new("o", 64, mi.bfloat16), pk.new_tensor((64,), dtype=mi.float32, name="w")
    pk.residual_prenorm_layer(None, x, x, o, weight=w)  # the new rows may not overwrite the old ones
    with pytest.raises(Exception, match="overwrite"):
        pk.describe_program()
    pk = make_mpk(make_meta(2, 64, 8, 2, 4, device="cpu"), 64, 8, 2, 4, 64, num_workers=256)
    new = lambda name, cols, dt=mi.float32: pk.new_tensor((8, cols), dtype=dt, name=name)
    pk.residual_prenorm_layer(None, new("x", 64), new("y", 64), new("o", 64, mi.bfloat16), weight=pk.new_tensor((64,), dtype=mi.float32, name="w"), groups=5)
    with pytest.raises(Exception, match="5 parts"):
        pk.describe_program()


def test_state_slots_of_a_session():
    """A request keeps its slot while it lives, wherever it sits in a pass, and the slot is used again afterwards."""
    from mirage.mpk.serving import PagePool, ServingSession

    class Stub:
        def __call__(self):
            pass

    s, R = ServingSession.__new__(ServingSession), 3
    s.page_size, s.max_rows, s.max_requests, s.rows_per_request, s.max_seq = 4, 8, R, 8, 64
    s.pool, s.slots, s.requests, s.mpk = PagePool(12), PagePool(R, "state slots"), {}, Stub()
    s._block = torch.zeros(4 * R + 2 + 12, dtype=torch.int32)
    s.mpk.input_tokens = torch.zeros(8, 1, dtype=torch.int64)
    slots = lambda n: s._block[3 * R + 2:3 * R + 2 + n].tolist()
    s._pass([("a", [1, 2]), ("b", [3])])
    a, b = slots(2)
    s._pass([("c", [1]), ("b", [4])])
    c, b2 = slots(2)
    assert b2 == b and {a, b, c} == {0, 1, 2}
    s._pass([("b", [5]), ("a", [6]), ("c", [7])])
    assert slots(3) == [b, a, c] and s._block[4 * R + 2:].tolist()[:3] == s.requests["b"].pages + s.requests["a"].pages + s.requests["c"].pages
    with pytest.raises(RuntimeError, match="state slots"):
        s._pass([("d", [1])])
    assert "d" not in s.requests and len(s.slots) == 0
    s.end("b")
    s._pass([("d", [1])])
    assert slots(1) == [b]
