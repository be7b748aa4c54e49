"""Vizonex without a GPU: the oracle's mechanisms against closed forms, the product's host side (config reader, graph lowering, limits),
and what each mechanism is worth in the numbers."""
import json
import math

import pytest
import torch

from oracle.vizonex_ref import (VizonexOracle, causal_conv, chunk_attention_core, chunk_sees, clamped_gate, dual_scan, dual_step, gelu_tanh, rms_norm, rms_norm_parts, route_groups, silu,
                                sink_softmax, softplus)
from vizonex_helpers import CONFIGS, chunked, config, dense, dual, moe, prompt, weights

F64 = torch.float64


# ---------------------------------------------------------------- oracle mechanisms
def test_norms():
    x = torch.tensor([[3.0, -4.0, 1.0, 0.0]], dtype=F64)
    w = torch.tensor([1.0, 2.0, 3.0, 4.0], dtype=F64)
    assert torch.allclose(rms_norm(x, w, 0.5), x * w / math.sqrt(26 / 4 + 0.5))
    assert torch.allclose(rms_norm_parts(x, w, 0.5, 2), x * w / torch.tensor([12.5 + 0.5, 13.0, 1.0, 1.0], dtype=F64).sqrt())


def test_activations():
    z = torch.tensor([-3.0, 0.0, 0.5, 2.0], dtype=F64)
    assert torch.allclose(gelu_tanh(z), torch.nn.functional.gelu(z, approximate="tanh")) and torch.allclose(silu(z), z * torch.sigmoid(z))
    assert torch.allclose(softplus(z), torch.log(1 + torch.exp(z))) and softplus(torch.tensor(800.0, dtype=F64)) == 800.0
    one = lambda v: torch.tensor([v], dtype=F64)
    assert torch.allclose(clamped_gate(one(5.0), one(-9.0), 1.5), one(1.5 / (1 + math.exp(-1.702 * 1.5)) * -0.5))  # both clamped
    assert torch.allclose(clamped_gate(one(-5.0), one(0.25), 1.5), one(-5 / (1 + math.exp(1.702 * 5)) * 1.25))  # the gate has no lower bound


def test_chunk_edges():
    pos = torch.arange(12)
    sees = chunk_sees(pos, pos, 5)
    assert sees[4].nonzero().flatten().tolist() == [0, 1, 2, 3, 4] and sees[5].nonzero().flatten().tolist() == [5] and sees[11].nonzero().flatten().tolist() == [10, 11]
    assert torch.equal(chunk_sees(pos, pos, None), pos[None, :] <= pos[:, None]) and torch.equal(chunk_sees(pos, pos, 1), torch.eye(12, dtype=torch.bool))


def test_sink_has_no_value():
    s, sees = torch.tensor([[0.0, math.log(3.0), 700.0], [-800.0, -900.0, 0.0]], dtype=F64), torch.tensor([[True, True, False], [True, True, False]])
    p = sink_softmax(s, sees, math.log(4.0))
    assert torch.allclose(p[0], torch.tensor([1 / 8, 3 / 8, 0.0], dtype=F64)) and p[1].sum() < 1e-300
    assert sink_softmax(torch.tensor([[-900.0]], dtype=F64), torch.tensor([[True]]), -1000.0).item() > 1 - 1e-12


def test_attention_groups_heads_and_scales_scores():
    g = torch.Generator().manual_seed(2)
    q, k, v = torch.randn(9, 4, 5, generator=g, dtype=F64), torch.randn(9, 2, 5, generator=g, dtype=F64), torch.randn(9, 2, 3, generator=g, dtype=F64)
    pos, temp, sink = torch.arange(9), torch.tensor([0.5, 2.0, 1.0, -1.0], dtype=F64), torch.tensor([0.0, 1.0, -1.0, 2.0], dtype=F64)
    got = chunk_attention_core(q, k, v, pos, 0.7, temp, sink, 4)
    scaled = chunk_attention_core(q * temp[:, None], k.repeat_interleave(2, 1), v.repeat_interleave(2, 1), pos, 0.7, torch.ones(4, dtype=F64), sink, 4)
    assert torch.allclose(got, scaled) and torch.allclose(got[4, 1], v[4, 0] / (1 + torch.exp(1 - 0.7 * 2 * q[4, 1] @ k[4, 0])))
    v2 = v.clone()
    v2[3] = 9.0  # the last position of the first chunk
    other = chunk_attention_core(q, k, v2, pos, 0.7, temp, sink, 4)
    assert torch.equal(other[4:], got[4:]) and torch.equal(other[:3], got[:3]) and not torch.allclose(other[3], got[3])


def test_convolution_over_pieces():
    g = torch.Generator().manual_seed(3)
    x, w, b = torch.randn(10, 3, generator=g, dtype=F64), torch.randn(3, 4, generator=g, dtype=F64), torch.randn(3, generator=g, dtype=F64)
    y, tail = causal_conv(x, torch.zeros(3, 3, dtype=F64), w, b)
    assert torch.allclose(y[0], b + w[:, 3] * x[0]) and torch.allclose(y[5], b + sum(w[:, j] * x[2 + j] for j in range(4))) and torch.equal(tail, x[7:])
    assert torch.allclose(causal_conv(x, torch.zeros(3, 3, dtype=F64), w)[0], y - b)
    t, out = torch.zeros(3, 3, dtype=F64), []
    for lo, hi in ((0, 1), (1, 3), (3, 10)):
        o, t = causal_conv(x[lo:hi], t, w, b)
        out.append(o)
    assert torch.allclose(torch.cat(out), y) and torch.equal(t, tail)


def test_recurrence_remembers_and_forgets():
    B, C, x = torch.tensor([1.0, -1, 2], dtype=F64), torch.tensor([1.0, 1, 1], dtype=F64), torch.tensor([3.0, 4.0], dtype=F64)
    S, y = dual_step(torch.zeros(3, 2, dtype=F64), 0.5, x, torch.tensor(-1.0, dtype=F64), B, C, 2.0)
    assert torch.allclose(S, 0.5 * B[:, None] * x) and torch.allclose(y, x + 2 * x)
    S2, _ = dual_step(S, 1.0, 0 * x, torch.tensor(-2.0, dtype=F64), B, C, 2.0)
    assert torch.allclose(S2, math.exp(-2.0) * S)
    g = torch.Generator().manual_seed(1)
    rnd = lambda *s: torch.rand(*s, generator=g, dtype=F64)
    dt, xs, Bs, Cs, A, D, Z = rnd(5, 4), rnd(5, 4, 2), rnd(5, 2, 3), rnd(5, 2, 3), -rnd(4), rnd(4), torch.zeros(4, 3, 2, dtype=F64)
    a, ya = dual_scan(Z, dt, xs, A, Bs, Cs, D)
    b, y0 = dual_scan(Z, dt[:2], xs[:2], A, Bs[:2], Cs[:2], D)
    b, y1 = dual_scan(b, dt[2:], xs[2:], A, Bs[2:], Cs[2:], D)
    assert torch.allclose(a, b) and torch.allclose(ya, torch.cat([y0, y1])) and not Z.any()
    _, y3 = dual_scan(Z[3:], dt[:, 3:], xs[:, 3:], A[3:], Bs[:, 1:], Cs[:, 1:], D[3:])  # head 3 reads the second of two groups
    assert torch.allclose(ya[:, 3:], y3)


def test_routing():
    s = torch.tensor([0.9, 0.1, 0.6, 0.5, 0.8, 0.2], dtype=F64)
    z, zero = torch.log(s / (1 - s)), torch.zeros(6, dtype=F64)
    idx, w = route_groups(z, zero, 2, 1, 1, 2.5)
    assert idx.tolist() == [0, 4] and torch.allclose(w, torch.tensor([2.25, 2.0], dtype=F64))
    assert route_groups(z, zero, 2, 3, 1, 1.0)[0].tolist() == [2, 3]  # sums 1.0, 1.1, 1.0
    idx, w = route_groups(z, torch.tensor([-2.0, -2, -2, -2, -1.2, -2], dtype=F64), 2, 3, 1, 1.0)  # negative choices; the weights do not see them
    assert idx.tolist() == [4, 5] and torch.allclose(w, s[[4, 5]])
    assert route_groups(z, zero, 2, 6, 2, 1.0)[0].tolist() == [0, 4]  # groups of one expert


@pytest.mark.parametrize("name", list(CONFIGS))
def test_oracle_in_pieces_is_the_oracle_at_once(name):
    c = CONFIGS[name]
    o, toks = VizonexOracle(c, weights(c)), prompt(c, 60)
    whole, st, at, parts = o.forward(toks, o.new_state(), 0), o.new_state(), 0, []
    for n in (2, 31, 1, 1, 20, 5):
        parts.append(o.forward(toks[at:at + n], st, at))
        at += n
    assert torch.allclose(torch.cat(parts), whole, atol=1e-9)


@pytest.mark.parametrize("what", ["chunk", "sink", "temp", "rownorm", "positions", "canon", "factor", "factor2", "state", "tail", "ring", "skip", "gate", "parts", "group", "router", "choice", "scale",
                                  "limit", "shared", "gelu", "order"])
def test_each_mechanism_shows(what, monkeypatch):
    """A mistake in one mechanism of the oracle moves the logits by far more than the GPU tests allow."""
    import oracle.vizonex_ref as ref
    c = config([chunked(4, 2, 16, 24, 20, dense(48)), dual(4, 12, 8, 2, 2, 4, moe(6, 2, 3, 1, 24, 24, limit=0.6, shared_limit=0.5))], 64, 90)
    w, toks = weights(c), prompt(c, 90)
    good = VizonexOracle(c, w).forward(toks, VizonexOracle(c, w).new_state(), 0)
    b, bw = json.loads(json.dumps(c)), dict(w)
    att, ssm, ff = b["layers"][0]["mixer"], b["layers"][1]["mixer"], b["layers"][1]["mlp"]
    if what == "chunk":
        att["mask"]["size"] += 1
    elif what == "parts":
        ssm["norm_groups"] = 1
    elif what == "router":
        ff["router"]["top"] = 1
    elif what == "scale":
        ff["router"]["scale"] = 1.0
    elif what == "limit":
        ff["expert"]["limit"] = 9.0
    elif what == "group":  # all groups stay open
        ff["router"]["groups"]["keep"] = 3
    elif what == "gelu":
        monkeypatch.setattr(ref, "gelu_tanh", ref.silu)
    elif what == "choice":  # the weights see the correction
        route = ref.route_groups
        monkeypatch.setattr(ref, "route_groups", lambda z, corr, *a: (lambda i, s: (i, s + a[3] * corr[i]))(*route(z, corr, *a)))
    elif what == "gate":  # the gate behind the norm
        norm, gates = ref.rms_norm_parts, []
        monkeypatch.setattr(ref, "silu", lambda z: (gates.append(silu(z)), torch.ones_like(z))[1] if z.shape[1] == 48 else silu(z))
        monkeypatch.setattr(ref, "rms_norm_parts", lambda *a: norm(*a) * gates[-1])
    elif what == "order":  # the feed-forward reads what the mixer reads
        ffn = ref.VizonexOracle.feed_forward
        monkeypatch.setattr(ref.VizonexOracle, "feed_forward", lambda self, i, h: ffn(self, i, h + causal_conv(h, torch.zeros(3, h.shape[1], dtype=h.dtype), self.w[f"l{i}.canon1"])[0]))
    else:
        names = {"temp": (".temp",), "rownorm": (".q.norm", ".k.norm"), "positions": ("pos",), "canon": (".canon1",), "factor": (".ls1",), "factor2": (".ls2",), "skip": (".D",),
                 "shared": (".shared.down",), "sink": (".sink",), "state": (), "tail": (), "ring": ()}[what]
        fill = {"sink": -50.0, "temp": 1.0, "rownorm": 1.0, "factor": 1.0, "factor2": 1.0}.get(what, 0.0)
        bw = {n: torch.full_like(t, fill) if names and n.endswith(names) else t for n, t in w.items()}
    bad = VizonexOracle(b, bw)
    st = bad.new_state()
    if what in ("state", "tail", "ring"):  # what the first 64 tokens left is lost between two portions
        a = bad.forward(toks[:64], st, 0)
        for s in st:
            if what == "ring":
                s.canon = torch.zeros_like(s.canon)
            elif s.S is not None:
                s.S, s.tail = (torch.zeros_like(s.S), s.tail) if what == "state" else (s.S, torch.zeros_like(s.tail))
        got, lo, hi = torch.cat([a, bad.forward(toks[64:], st, 64)]), 64, 67
    else:
        got, lo, hi = bad.forward(toks, st, 0), 64, None
    err = ((got - good)[lo:hi].pow(2).mean(-1).sqrt() / good.std()).median()
    assert err > 0.05, float(err)


# ---------------------------------------------------------------- product, host side
def test_config_reader():
    from mirage.mpk.models.vizonex.builder import ChunkMixer, DenseFF, DualMixer, ExpertFF, VizonexConfig
    c = VizonexConfig.from_dict(CONFIGS["odd"])
    assert (c.vocab, c.width, c.eps, c.taps, c.max_positions) == (133, 84, 1e-5, 3, 600)
    assert [type(l.mixer) for l in c.layers] == [DualMixer, ChunkMixer, DualMixer, ChunkMixer, ChunkMixer, DualMixer]
    assert [type(l.ff) for l in c.layers] == [type(None), ExpertFF, DenseFF, type(None), ExpertFF, ExpertFF]
    s = c.tensor_shapes()
    assert s["l0.mix.in"] == (75 + 75 + 22 + 3, 84) and s["l2.mix.conv"] == (84 + 2 * 3 * 37, 6) and s["l1.mix.v"] == (56, 84) and s["l1.mix.k.norm"] == (40,) and s["l1.mix.o"] == (84, 168)
    assert "l0.ls2" not in s and s["l2.ls2"] == (84,) and "l4.mlp.shared.up" not in s and s["l5.mlp.shared.up"] == (20, 84) and s["pos"] == (600, 84) and s["head"] == (133, 84) and s["l0.canon1"] == (84, 3)
    assert (c.layers[1].ff.scale, c.layers[1].ff.limit, c.layers[1].ff.shared_limit, c.layers[4].ff.scale) == (1.7, 2.0, 1.2, 0.8) and c.layers[3].mixer.chunk == 70
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 2, "mlp", "kind"), "other"), (("layers", 1, "mixer", "kv_heads"), 4), (("layers", 2, "mixer", "groups"), 4),
                        (("layers", 0, "mixer", "norm_groups"), 4), (("layers", 1, "mlp", "router", "groups", "count"), 4), (("layers", 1, "mlp", "router", "groups", "keep"), 1),
                        (("layers", 1, "mlp", "router", "groups", "keep"), 4)):
        bad = json.loads(json.dumps(CONFIGS["odd"]))
        d = bad
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            VizonexConfig.from_dict(bad)


def test_registry_picks_the_builder_by_config():
    from mirage.mpk.model_registry import get_builder, model_name_of
    from mirage.mpk.models.vizonex import VizonexBuilder
    assert get_builder(model_name_of({"architecture": "Vizonex"})) is VizonexBuilder
    assert [VizonexBuilder.kernels(*a) for a in ((torch.float32, 64), (torch.bfloat16, 1), (torch.bfloat16, 64))] == [("DUAL_F32",), ("DUAL_M1",), ("DUAL",)]


def _host_mpk(c, dtype=torch.bfloat16, B=64, **kw):
    from mirage.mpk import MPK, MirageModelConfig, MPKMetadata
    m = MPK(MPKMetadata(**{**dict(mode="online_notoken", max_seq_length=256, max_num_batched_requests=min(4, B), max_num_batched_tokens=B, max_num_pages=8, page_size=64, device="cpu",
                                  num_workers=256, dtype=dtype, model_config=MirageModelConfig(architecture=c, state_dict=weights(c))), **kw}))
    m.build()
    return m


def _ops(m):
    return [l.split()[1] for l in m.persistent_kernel.describe_program().splitlines()]


def test_lowering():
    """The stage program of every kind of layer: sum, norm and convolution of single tokens folded into the linear behind, the activation in
    its linear, the routing in the expert stage."""
    c = config([chunked(4, 2, 16, 24, 20, dense(48)), dual(4, 12, 8, 2, 2, 4, moe(6, 2, 3, 2, 24, 24)), chunked(4, 2, 16, 24, 20, None)], 64, 90)
    n, conv = "MX_PRENORM[multi-token", "DU_CONV[portions]"
    att = [n, conv, "LINEAR", "FX_PREP[portions]", "FX_ATTN", "LINEAR"]
    want = (["FX_EMBED"] + att + ["LINEAR+gelu", "LINEAR"] + [n, conv, "LINEAR", "DU_CONV", "DU_SCAN", "MX_PRENORM", "LINEAR", "MX_HEAD_LINEAR", "HY_ROUTE[multi-token", "HY_EXPERTS+route+clamped", "HY_EXPERTS"] +
            att + [n, "LINEAR", "ARGMAX_PARTIAL", "ARGMAX_REDUCE"])
    m = _host_mpk(c)
    assert _ops(m) == want
    b = m.model_builder
    assert (len(b.canon), len(b.state), len(b.tail), len(b.k_cache)) == (3, 1, 1, 2) and b.state_slots is not None
    assert len(json.loads(m.generate_task_graph()["json_file"])["all_tasks"]) > 2
    single = _ops(_host_mpk(c, B=1))
    assert conv not in single and "FX_PREP[portions]" not in single and single.count("DU_CONV") == 1
    f32 = _ops(_host_mpk(c, torch.float32))
    assert n not in f32 and f32.count("MX_PRENORM") == 5 and "LINEAR_F32+gelu" in f32 and "LINEAR" not in f32 and f32.count(conv) == 3


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_every_test_model_lowers(name, dtype):
    assert _ops(_host_mpk(CONFIGS[name], dtype))[-1] == "ARGMAX_REDUCE"


def test_builder_refuses_what_does_not_fit():
    import mirage as mi
    from mirage.mpk import MirageModelConfig
    c = CONFIGS["even"]
    for change, match in ((lambda w: w.pop("l1.mix.A_log"), "l1.mix.A_log"), (lambda w: w.update({"l0.mix.q": w["l0.mix.q"][:-1]}), "l0.mix.q")):
        w = weights(c)
        change(w)
        with pytest.raises((KeyError, ValueError), match=match):
            _host_mpk(c, model_config=MirageModelConfig(architecture=c, state_dict=w))
    offline = dict(mode="offline", total_num_requests=1, max_num_pages=16)
    with pytest.raises(NotImplementedError, match="recurrent"):
        _host_mpk(c, **offline, spec_decode_config=mi.mpk.spec_decode_class("promptlookup", ngram_size=2, spec_length=4))
    short = dict(c, max_positions=100)
    _host_mpk(short, **offline, max_seq_length=101)
    with pytest.raises(ValueError, match="100 positions"):
        _host_mpk(short, **offline, max_seq_length=102)
    assert _host_mpk(short).model_builder.max_positions == 100  # (a session keeps its requests below it)


def test_lowering_refuses_what_does_not_fit():
    for layers, kw, match in (([dual(2, 32, 300, 1, 1, 4, None)], {}, "256"), ([dual(2, 32, 16, 1, 1, 17, None)], {}, "17 taps"), ([chunked(2, 1, 16, 16, 9, None)], {"taps": 17}, "17 taps"),
                              ([chunked(2, 1, 600, 8, 9, None)], {}, "512"), ([chunked(2, 1, 16, 8, 9, moe(300, 2, 1, 1, 16, 16))], {}, "256"), ([chunked(2, 1, 16, 8, 9, moe(30, 20, 1, 1, 16, 16))], {}, "16 of")):
        m = _host_mpk(config(layers, 64, 90, **kw))
        with pytest.raises(Exception, match=match):
            m.persistent_kernel.describe_program()


def test_dual_tasks_check_their_operands():
    import mirage as mi
    from helpers import make_meta, make_mpk
    pk = lambda: make_mpk(make_meta(2, 64, 8, 2, 4, device="cpu"), 64, 8, 2, 4, 64, num_workers=256)
    def new(k, name, *dims, dt=mi.bfloat16):
        return k.new_tensor(dims, dtype=dt, name=name)
    k = pk()
    z, ids, w, c = new(k, "z", 8, 8, dt=mi.float32), new(k, "ids", 8, 4, dt=mi.int32), new(k, "w", 8, 4, dt=mi.float32), new(k, "c", 8, dt=mi.float32)
    k.expert_route_layer(z, ids, w, 8, 4, False, correction=c, groups=4, groups_kept=1)
    with pytest.raises(Exception, match="4 of 8 experts in 4 groups of which 1"):
        k.describe_program()
    k = pk()
    k.ring_conv_layer(new(k, "x", 8, 64), new(k, "w", 4, 64), new(k, "r", 2, 3, 64), new(k, "s", 2, dt=mi.int32), new(k, "o", 8, 64))
    with pytest.raises(Exception, match="4 taps over 64"):
        k.describe_program()
    k = pk()
    k.dual_scan_layer(new(k, "x", 8, 64), new(k, "cv", 8, 80), new(k, "st", 8, 8, dt=mi.float32), new(k, "D", 4, dt=mi.float32), new(k, "S", 2, 4, 16, 12, dt=mi.float32), new(k, "s", 2, dt=mi.int32),
                      new(k, "o", 8, 64, dt=mi.float32), 4, 16, 8, 1, 0, 0, 64, 72, 4)
    with pytest.raises(Exception, match=r"\[>= 2 slots, 4, 16, 8\]"):
        k.describe_program()
    k = pk()
    k.gelu_mul_layer(new(k, "x", 8, 64), new(k, "o", 8, 32))
    with pytest.raises(Exception, match="gelu_mul follows"):
        k.describe_program()
    k = pk()  # latent attention, the delta rule and the selective scan have kernels of their own
    sl = new(k, "s", 2, dt=mi.int32)
    k.ring_conv_layer(new(k, "x", 8, 64), new(k, "w", 4, 64), new(k, "r", 2, 4, 64), sl, new(k, "o", 8, 64))
    k.short_conv_layer(new(k, "x2", 8, 64), new(k, "w2", 4, 64, dt=mi.float32), new(k, "b", 64, dt=mi.float32), new(k, "t", 2, 3, 64), sl, new(k, "o2", 8, 64))
    with pytest.raises(Exception, match="cannot run in one graph"):
        k.describe_program()
