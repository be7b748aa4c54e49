"""Bukatar without a GPU: the oracle's mechanisms against closed forms, the product's host side (config reader, row orders, graph
lowering), and what each mechanism is worth in the numbers."""
import json
import math

import pytest
import torch

from oracle.bukatar_ref import (BukatarOracle, causal_conv, latent_attention_core, relu_squared, rms_norm, rotate_pairs, route, scan_step, selective_scan, silu, sink_softmax, softplus,
                                window_attention_core, window_sees)
from bukatar_helpers import CONFIGS, config, dense, latent, moe, prompt, scan, weights, window

F64 = torch.float64


# ---------------------------------------------------------------- oracle mechanisms
def test_norm_and_activations():
    x = torch.tensor([[3.0, -4.0]], dtype=F64)
    assert torch.allclose(rms_norm(x, torch.tensor([1.0, 2.0], dtype=F64), 0.5), torch.tensor([[3.0, -8.0]], dtype=F64) / math.sqrt(13.0))
    z = torch.tensor([-3.0, 0.0, 2.0], dtype=F64)
    assert relu_squared(z).tolist() == [0.0, 0.0, 4.0]
    assert torch.allclose(silu(z), z * torch.sigmoid(z)) and torch.allclose(softplus(z), torch.log(1 + torch.exp(z))) and softplus(torch.tensor(800.0, dtype=F64)) == 800.0


def test_rotation_is_a_complex_product():
    x, pos = torch.randn(4, 3, 11, dtype=F64), torch.tensor([0, 1, 77, 4000])
    f = torch.tensor([55.0 ** (-2 * i / 6) for i in range(3)], dtype=F64)
    z = torch.complex(x[..., 0:6:2], x[..., 1:6:2]) * torch.polar(torch.ones(1, dtype=F64), pos[:, None, None].double() * f)
    y = rotate_pairs(x, pos, 6, 55.0)
    assert torch.allclose(y[..., 0:6:2], z.real) and torch.allclose(y[..., 1:6:2], z.imag) and torch.equal(y[..., 6:], x[..., 6:])


def test_window_edges():
    pos = torch.arange(12)
    sees = window_sees(pos, pos, 3, 2)
    assert sees[9].nonzero().flatten().tolist() == [0, 1, 7, 8, 9] and sees[1].nonzero().flatten().tolist() == [0, 1]
    assert window_sees(pos, pos, 1, 0).tolist() == torch.eye(12, dtype=torch.bool).tolist()
    assert torch.equal(window_sees(pos, pos, None, 0), pos[None, :] <= pos[:, None])


def test_sink_adds_one_to_the_denominator():
    s = torch.tensor([[0.0, math.log(3.0), 700.0], [-800.0, -900.0, 0.0]], dtype=F64)
    sees = torch.tensor([[True, True, False], [True, True, False]])
    p = sink_softmax(s, sees)
    assert torch.allclose(p[0], torch.tensor([0.2, 0.6, 0.0], dtype=F64)) and p[1].sum() < 1e-300
    assert sink_softmax(torch.tensor([[900.0]], dtype=F64), torch.tensor([[True]])).item() == 1.0


def test_window_attention_groups_heads():
    g = torch.Generator().manual_seed(2)
    q, k, v = (torch.randn(9, n, 5, generator=g, dtype=F64) for n in (4, 2, 2))
    pos = torch.arange(9)
    want = window_attention_core(q, k.repeat_interleave(2, 1), v.repeat_interleave(2, 1), pos, 0.7, 4, 1)
    assert torch.allclose(window_attention_core(q, k, v, pos, 0.7, 4, 1), want)
    k2, v2 = k.clone(), v.clone()
    k2[3], v2[3] = 9.0, 9.0  # position 3 is inside the window up to position 6
    got = window_attention_core(q, k2, v2, pos, 0.7, 4, 1)
    assert torch.equal(got[[0, 1, 2, 7, 8]], window_attention_core(q, k, v, pos, 0.7, 4, 1)[[0, 1, 2, 7, 8]]) and not torch.allclose(got[6], want[6])


def test_latent_attention_in_the_latent_space_is_the_same():
    g = torch.Generator().manual_seed(0)
    rnd = lambda *s: torch.randn(*s, generator=g, dtype=F64)
    T, H, D, P, E, R = 6, 3, 5, 4, 7, 9
    q, qr, c, kr, uk, uv, pos = rnd(T, H, D), rnd(T, H, P), rnd(T, R), rnd(T, P), rnd(H, D, R), rnd(H, E, R), torch.arange(T)
    eye = torch.eye(R, dtype=F64).expand(H, -1, -1)
    lat = latent_attention_core(torch.einsum("thd,hdr->thr", q, uk), qr, c, kr, eye, eye, pos, 0.3)
    assert torch.allclose(torch.einsum("thr,her->the", lat, uv), latent_attention_core(q, qr, c, kr, uk, uv, pos, 0.3))


def test_convolution_over_pieces():
    g = torch.Generator().manual_seed(3)
    x, w, b = torch.randn(10, 3, generator=g, dtype=F64), torch.randn(3, 4, generator=g, dtype=F64), torch.randn(3, generator=g, dtype=F64)
    y, tail = causal_conv(x, torch.zeros(3, 3, dtype=F64), w, b)
    assert torch.allclose(y[0], b + w[:, 3] * x[0]) and torch.allclose(y[5], b + sum(w[:, j] * x[2 + j] for j in range(4))) and torch.equal(tail, x[7:])
    t, out = torch.zeros(3, 3, dtype=F64), []
    for lo, hi in ((0, 1), (1, 3), (3, 10)):
        o, t = causal_conv(x[lo:hi], t, w, b)
        out.append(o)
    assert torch.allclose(torch.cat(out), y) and torch.equal(t, tail)


def test_scan_remembers_and_forgets():
    S, one = torch.zeros(2, 3, dtype=F64), torch.ones(2, dtype=F64)
    A, B, C = -torch.tensor([[1.0, 2, 3], [4, 5, 6]], dtype=F64), torch.tensor([1.0, -1, 2], dtype=F64), torch.tensor([1.0, 1, 1], dtype=F64)
    S, y = scan_step(S, 0.5 * one, torch.tensor([3.0, 4.0], dtype=F64), A, B, C, 2 * one)
    assert torch.allclose(S, 0.5 * torch.tensor([[3.0], [4.0]], dtype=F64) * B) and torch.allclose(y, torch.tensor([1.5 * 2 + 6, 2.0 * 2 + 8], dtype=F64))
    S2, _ = scan_step(S, one, 0 * one, A, B, C, one)
    assert torch.allclose(S2, torch.exp(A) * S)
    g = torch.Generator().manual_seed(1)
    dt, x, Bs, Cs = (torch.rand(5, n, generator=g, dtype=F64) for n in (2, 2, 3, 3))
    a, ya = selective_scan(S, dt, x, A, Bs, Cs, one)
    b, y0 = selective_scan(S, dt[:2], x[:2], A, Bs[:2], Cs[:2], one)
    b, y1 = selective_scan(b, dt[2:], x[2:], A, Bs[2:], Cs[2:], one)
    assert torch.allclose(a, b) and torch.allclose(ya, torch.cat([y0, y1]))


def test_routing():
    idx, w = route(torch.log(torch.tensor([1.0, 4.0, 2.0, 1.0], dtype=F64)), 2)
    assert idx.tolist() == [1, 2] and torch.allclose(w, torch.tensor([2 / 3, 1 / 3], dtype=F64))


@pytest.mark.parametrize("name", ["odd", "even"])
def test_oracle_in_pieces_is_the_oracle_at_once(name):
    c = CONFIGS[name]
    o, toks = BukatarOracle(c, weights(c)), prompt(c, 60)
    whole, st, at, parts = o.forward(toks, o.new_state(), 0), o.new_state(), 0, []
    for n in (2, 31, 1, 1, 20, 5):
        parts.append(o.forward(toks[at:at + n], st, at))
        at += n
    assert torch.allclose(torch.cat(parts), whole, atol=1e-9)


@pytest.mark.parametrize("what", ["window", "keep", "sink", "value", "bias", "latent", "share", "state", "tail", "skip", "gate", "router", "shared", "behind", "pairs"])
def test_each_mechanism_shows(what, monkeypatch):
    """A mistake in one mechanism of the oracle moves the logits by far more than the GPU tests allow."""
    import oracle.bukatar_ref as ref
    c = config([window(4, 2, 16, 8, 20, 6, dense(48)), scan(48, 8, 4, 4, moe(6, 2, 24, 24)), latent(3, 16, 8, 16, 32, dense(48)), latent(3, 16, 8, 16, 32, None, kv_from=2)], 64, 90)
    w, toks = weights(c), prompt(c, 90)
    good = BukatarOracle(c, w).forward(toks, BukatarOracle(c, w).new_state(), 0)
    b, bw = json.loads(json.dumps(c)), dict(w)
    if what == "window":
        b["layers"][0]["mixer"]["mask"]["size"] += 1
    elif what == "keep":
        b["layers"][0]["mixer"]["mask"]["keep_first"] -= 1
    elif what == "share":
        del b["layers"][3]["mixer"]["kv_from"]
        bw.update({"l3.mix.dkv": w["l2.mix.dkv"], "l3.mix.dkv.norm": w["l2.mix.dkv.norm"]})
    elif what == "router":
        b["layers"][1]["mlp"]["router"]["top"] = 1
    elif what == "sink":
        monkeypatch.setattr(ref, "sink_softmax", lambda s, sees: torch.softmax(s.masked_fill(~sees, float("-inf")), -1))
    elif what == "pairs":
        monkeypatch.setattr(ref, "rotate_pairs", lambda x, pos, dims, base: x)
    elif what == "value":  # values taken behind the rotation
        core = ref.window_attention_core
        monkeypatch.setattr(ref, "window_attention_core", lambda q, k, v, *a: core(q, k, k, *a))
    else:
        names = {"bias": (".q.b", ".k.b", ".o.b"), "latent": (".dkv.norm",), "skip": (".D",), "gate": (".shared.sg",), "shared": (".shared.down",), "behind": ("norm1b",),
                 "state": (), "tail": ()}[what]
        bw = {n: (torch.zeros_like(t) if n.endswith(names) and names and what not in ("latent", "behind") else torch.ones_like(t) if names and n.endswith(names) else t) for n, t in w.items()}
    bad = BukatarOracle(b, bw)
    st = bad.new_state()
    if what in ("state", "tail"):  # what the first 64 tokens left is lost between two portions
        a = bad.forward(toks[:64], st, 0)
        for s in st:
            if s.S is not None:
                s.S, s.tail = (torch.zeros_like(s.S), s.tail) if what == "state" else (s.S, torch.zeros_like(s.tail))
        got, lo, hi = torch.cat([a, bad.forward(toks[64:], st, 64)]), 64, 67
    else:
        got, lo, hi = bad.forward(toks, st, 0), 64, None
    err = ((got - good)[lo:hi].pow(2).mean(-1).sqrt() / good.std()).median()
    assert err > 0.04, float(err)


# ---------------------------------------------------------------- product, host side
def test_config_reader():
    from mirage.mpk.models.bukatar.builder import BukatarConfig, DenseFF, ExpertFF, LatentMixer, ScanMixer, WindowMixer
    c = BukatarConfig.from_dict(CONFIGS["odd"])
    assert (c.vocab, c.width, c.eps) == (133, 84, 1e-5)
    assert [type(l.mixer) for l in c.layers] == [ScanMixer, LatentMixer, WindowMixer, WindowMixer, LatentMixer, ScanMixer, WindowMixer]
    assert [type(l.ff) for l in c.layers] == [type(None), ExpertFF, DenseFF, type(None), DenseFF, ExpertFF, ExpertFF]
    s = c.tensor_shapes()
    assert s["l0.mix.x"] == (27, 75) and s["l1.mix.dkv"] == (56, 84) and "l4.mix.dkv" not in s and s["l2.mix.k.b"] == (40,) and "l0.norm2" not in s and s["l5.mlp.e5.down"] == (84, 50)
    assert s["l1.mlp.shared.sg"] == (1, 84) and "l1.mlp.e5.up" not in s and (c.layers[3].mixer.window, c.layers[3].mixer.keep_first) == (70, 0)
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 2, "mlp", "kind"), "other"), (("layers", 4, "mixer", "kv_from"), 0), (("layers", 4, "mixer", "kv_from"), 5),
                        (("layers", 4, "mixer", "kv_rank"), 40), (("layers", 1, "mixer", "rot", "dims"), 8), (("layers", 2, "mixer", "vdim"), 8), (("layers", 2, "mixer", "kv_heads"), 4)):
        bad = json.loads(json.dumps(CONFIGS["odd"]))
        d = bad
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            BukatarConfig.from_dict(bad)


def test_registry_picks_the_builder_by_config():
    from mirage.mpk.model_registry import get_builder, model_name_of
    from mirage.mpk.models.bukatar import BukatarBuilder
    assert get_builder(model_name_of({"architecture": "Bukatar"})) is BukatarBuilder
    assert BukatarBuilder.kernels(torch.float32, 64) == ("HYB_F32",) and BukatarBuilder.kernels(torch.bfloat16, 1) == ("HYB_M1",) and BukatarBuilder.kernels(torch.bfloat16, 64) == ("HYB",)


def test_row_orders():
    from mirage.mpk.persistent_kernel import expert_tiles, gated_rows, operand_tiles, pairs_to_halves
    g = torch.Generator().manual_seed(4)
    x, pos = torch.randn(5, 1, 10, generator=g, dtype=F64), torch.arange(5)
    order, half = pairs_to_halves(10, 6), rotate_pairs(x, pos, 6, 40.0)
    y = x[..., order]
    f = torch.tensor([40.0 ** (-2 * i / 6) for i in range(3)], dtype=F64) * pos[:, None, None]
    lo, hi = y[..., :3], y[..., 3:6]
    assert torch.allclose(torch.cat([lo * f.cos() - hi * f.sin(), hi * f.cos() + lo * f.sin(), y[..., 6:]], -1), half[..., order])
    gate, up = torch.randn(2, 32, 64, generator=g).bfloat16(), torch.randn(2, 32, 64, generator=g).bfloat16()
    w = gated_rows(gate, up)
    assert torch.equal(w[1, :16], gate[1, :16]) and torch.equal(w[1, 16:32], up[1, :16]) and torch.equal(w[0, 48:], up[0, 16:])
    t = expert_tiles(torch.randn(3, 20, 64, generator=g))
    assert t.shape == (3 * 2, 16 * 64) and torch.equal(t[1].view(4, 4, 16, 4)[:, :, 4:].abs().max(), torch.tensor(0.0)) and torch.equal(expert_tiles(w), operand_tiles(w))


def _host_mpk(c, dtype=torch.bfloat16, B=64, **kw):
    from mirage.mpk import MPK, MirageModelConfig, MPKMetadata
    m = MPK(MPKMetadata(**{**dict(mode="online_notoken", max_seq_length=256, max_num_batched_requests=min(4, B), max_num_batched_tokens=B, max_num_pages=8, page_size=64, device="cpu",
                                  num_workers=256, dtype=dtype, model_config=MirageModelConfig(architecture=c, state_dict=weights(c))), **kw}))
    m.build()
    return m


def _ops(m):
    return [l.split()[1] for l in m.persistent_kernel.describe_program().splitlines()]


def test_lowering():
    """The stage program of every kind of layer: the norms in front folded into the linear of single-token iterations, the activation in
    its linear, the routing in the expert stage, one cache for the layers that share it."""
    c = config([window(4, 2, 16, 8, 20, 6, dense(48)), scan(48, 8, 4, 4, moe(6, 2, 24, 24)), latent(3, 16, 8, 16, 32, None), latent(3, 16, 8, 16, 32, dense(40), kv_from=2)], 64, 90)
    n = "MX_PRENORM[multi-token"
    ff = [n, "LINEAR+relu2", "LINEAR"]
    want = (["FX_EMBED", n, "LINEAR", "FX_PREP[portions]", "FX_ATTN", "LINEAR"] + ff + [n, "LINEAR", "HY_CONV", "LINEAR", "HY_STEP", "HY_SCAN", "LINEAR"] +
            ["MX_PRENORM", "MX_HEAD_LINEAR", "HY_ROUTE[multi-token", "HY_EXPERTS+route+silu", "HY_EXPERTS"] +
            [n, "LINEAR", "MX_LATENT_PREP", "MX_HEAD_LINEAR", "MX_LATENT_ATTN", "MX_LATENT_MERGE[split", "MX_HEAD_LINEAR", "LINEAR"] +
            [n, "LINEAR", "MX_HEAD_LINEAR", "MX_LATENT_ATTN", "MX_LATENT_MERGE[split", "MX_HEAD_LINEAR", "LINEAR"] + ff + [n, "LINEAR", "ARGMAX_PARTIAL", "ARGMAX_REDUCE"])
    m = _host_mpk(c)
    assert _ops(m) == want
    b = m.model_builder
    assert (len(b.latent_cache), len(b.state), len(b.tail), len(b.k_cache)) == (1, 1, 1, 1) and b.state_slots is not None
    assert len(json.loads(m.generate_task_graph()["json_file"])["all_tasks"]) > 2
    f32 = _ops(_host_mpk(c, torch.float32))
    assert n not in f32 and f32.count("MX_PRENORM") == 8 and "LINEAR_F32+relu2" in f32 and "LINEAR" not in f32


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", [torch.bfloat16, torch.float32])
def test_every_test_model_lowers(name, dtype):
    assert _ops(_host_mpk(CONFIGS[name], dtype))[-1] == "ARGMAX_REDUCE"


def test_builder_refuses_what_does_not_fit():
    import mirage as mi
    from mirage.mpk import MirageModelConfig
    c = CONFIGS["even"]
    for change, match in ((lambda w: w.pop("l1.mix.A_log"), "l1.mix.A_log"), (lambda w: w.update({"l2.mix.uk": w["l2.mix.uk"][:-1]}), "l2.mix.uk")):
        w = weights(c)
        change(w)
        with pytest.raises((KeyError, ValueError), match=match):
            _host_mpk(c, model_config=MirageModelConfig(architecture=c, state_dict=w))
    with pytest.raises(NotImplementedError, match="recurrent"):
        _host_mpk(c, mode="offline", total_num_requests=1, max_num_pages=16, spec_decode_config=mi.mpk.spec_decode_class("promptlookup", ngram_size=2, spec_length=4))


def test_lowering_refuses_what_does_not_fit():
    for layers, match in (([scan(64, 300, 4, 8, None)], "256"), ([window(2, 1, 16, 8, 9, 1, moe(300, 2, 16, 16))], "256"), ([window(2, 1, 600, 8, 9, 1, None)], "512"),
                          ([window(2, 1, 16, 8, 9, 1, moe(30, 20, 16, 16))], "16 of")):
        m = _host_mpk(config(layers, 64, 90))
        with pytest.raises(Exception, match=match):
            m.persistent_kernel.describe_program()


def test_hybrid_tasks_check_their_operands():
    import mirage as mi
    from helpers import make_meta, make_mpk
    pk = lambda: make_mpk(make_meta(2, 64, 8, 2, 4, device="cpu"), 64, 8, 2, 4, 64, num_workers=256)
    def new(k, name, cols, dt=mi.bfloat16, rows=8):
        return k.new_tensor((rows, cols), dtype=dt, name=name)
    k = pk()
    z, ids, w = new(k, "z", 8, mi.float32), new(k, "ids", 2, mi.int32), new(k, "w", 4, mi.float32)
    k.expert_route_layer(z, ids, w, 8, 2, False)
    with pytest.raises(Exception, match="followed by the expert_linear"):
        k.describe_program()
    k = pk()
    k.expert_linear_layer(new(k, "x", 64), new(k, "wt", 16 * 64, rows=3 * 2), new(k, "ids", 2, mi.int32), new(k, "o", 64), 4, 2, 32, 64, 32)
    with pytest.raises(Exception, match="4 experts of 32 x 64"):
        k.describe_program()
    k = pk()
    slots = k.new_tensor((2,), dtype=mi.int32, name="slots")
    k.short_conv_layer(new(k, "x", 64), new(k, "w", 64, mi.float32, 4), k.new_tensor((64,), dtype=mi.float32, name="b"), k.new_tensor((2, 2, 64), dtype=mi.bfloat16, name="t"), slots, new(k, "o", 64))
    with pytest.raises(Exception, match="4 taps over 64"):
        k.describe_program()
    k = pk()
    k.relu_squared_layer(new(k, "x", 64), new(k, "o", 64))
    with pytest.raises(Exception):
        k.describe_program()
