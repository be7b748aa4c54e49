"""Suborax without a GPU: the oracle's mechanisms against closed forms, the product's host side (frequencies, config reader,
registry, graph lowering, page bookkeeping) against the oracle or by hand, and what each mechanism is worth in the numbers."""
import json
import math

import pytest
import torch

from oracle.suborax_ref import (SuboraxOracle, attention_core, cap_scores, rms_norm_offset, rotary_frequencies, rotate, softmax_with_sink, swiglu)
from suborax_helpers import CONFIGS, SCALING, config, layer, prompt, weights

F64 = torch.float64


# ---------------------------------------------------------------- oracle mechanisms
def test_norm_weight_is_stored_around_zero():
    x = torch.tensor([[3.0, -4.0]], dtype=F64)
    y = rms_norm_offset(x, torch.tensor([0.0, 1.0], dtype=F64), 0.5)
    assert torch.allclose(y, torch.tensor([[3.0, -8.0]], dtype=F64) / math.sqrt(13.0))


def test_frequency_scaling_keeps_stretches_and_blends():
    rot = {"dims": 32, "base": 1e4, "scaling": {"factor": 8.0, "low": 1.0, "high": 4.0, "original": 512}}
    plain, scaled = rotary_frequencies({"dims": 32, "base": 1e4}), rotary_frequencies(rot)
    seen = set()
    for f, g in zip(plain.tolist(), scaled.tolist()):
        wave = 2 * math.pi / f
        if wave < 128:
            seen.add("keep")
            assert g == f
        elif wave > 512:
            seen.add("stretch")
            assert g == pytest.approx(f / 8)
        else:
            seen.add("blend")
            s = (512 / wave - 1) / 3
            assert g == pytest.approx(s * f + (1 - s) * f / 8) and f / 8 <= g <= f
    assert seen == {"keep", "stretch", "blend"}


@pytest.mark.parametrize("dims", [2, 8, 24])
def test_rotation_is_a_complex_product_on_the_first_dims(dims):
    rot = {"dims": dims, "base": 77.0, "scaling": SCALING}
    x, pos = torch.randn(5, 2, 24, dtype=F64), torch.tensor([0, 1, 9, 300, 5000])
    y = rotate(x, pos, rot)
    z = torch.complex(x[..., :dims // 2], x[..., dims // 2:dims]) * torch.polar(torch.ones(1, dtype=F64), pos[:, None, None].double() * rotary_frequencies(rot))
    assert torch.allclose(y[..., :dims], torch.cat([z.real, z.imag], -1)) and torch.equal(y[..., dims:], x[..., dims:])


def test_sink_takes_its_share_once():
    s = torch.tensor([[1.0, 2.0, float("-inf")]], dtype=F64)
    p = softmax_with_sink(s, torch.tensor([0.5], dtype=F64))
    den = math.exp(1) + math.exp(2) + math.exp(0.5)
    assert torch.allclose(p, torch.tensor([[math.exp(1), math.exp(2), 0.0]], dtype=F64) / den)
    assert torch.allclose(softmax_with_sink(s, torch.tensor([-1e9], dtype=F64)), s.softmax(-1))


def test_cap_bounds_the_scores_and_zero_means_none():
    s = torch.linspace(-100, 100, 9, dtype=F64)
    c = cap_scores(s, 5.0)
    assert c.abs().max() <= 5.0 and torch.allclose(cap_scores(s * 1e-4, 5.0), s * 1e-4, rtol=1e-5) and torch.equal(cap_scores(s, 0), s)


def test_attention_is_causal_and_shares_key_heads():
    g = torch.Generator().manual_seed(0)
    q, k, v = (torch.randn(6, n, 8, generator=g, dtype=F64) for n in (4, 2, 2))
    pos, sink = torch.arange(6), torch.zeros(4, dtype=F64)
    a = attention_core(q, k, v, pos, sink, 0.3, 10.0)
    k2, v2 = k.clone(), v.clone()
    k2[4:], v2[4:, 1] = 9.0, -9.0
    b = attention_core(q, k2, v2, pos, sink, 0.3, 10.0)
    assert torch.equal(a[:4], b[:4]) and not torch.allclose(a[4:], b[4:])
    c = attention_core(q, torch.stack([k[:, 0], k2[:, 1]], 1), torch.stack([v[:, 0], v2[:, 1]], 1), pos, sink, 0.3, 10.0)
    assert torch.equal(a[:, :2], c[:, :2])  # query heads 0, 1 use key head 0


def test_swiglu():
    h = torch.randn(3, 4, dtype=F64)
    w = [torch.randn(5, 4, dtype=F64), torch.randn(5, 4, dtype=F64), torch.randn(4, 5, dtype=F64)]
    assert torch.allclose(swiglu(h, *w), (torch.nn.functional.silu(h @ w[0].T) * (h @ w[1].T)) @ w[2].T)


@pytest.mark.parametrize("name", CONFIGS)
def test_oracle_in_pieces_equals_oracle_at_once(name):
    c = CONFIGS[name]
    orc, toks = SuboraxOracle(c, weights(c)), prompt(c, 40)
    whole = orc.forward(toks, orc.new_state(), 0)
    st, at, out = orc.new_state(), 0, []
    for n in (2, 7, 1, 1, 20, 9):
        out.append(orc.forward(toks[at:at + n], st, at))
        at += n
    assert torch.allclose(torch.cat(out), whole, atol=1e-10)


@pytest.mark.parametrize("what", ["sink", "cap", "scaling", "offset", "alpha", "causal_far"])
def test_a_mistake_in_one_mechanism_shows_in_the_logits(what):
    """The small models of the GPU tests are sensitive enough: each mechanism done wrong (here, in the oracle) moves the
    logits by far more than the tolerances those tests use."""
    c = json.loads(json.dumps(CONFIGS["even"]))
    w, toks = weights(c), prompt(c, 100)
    good = SuboraxOracle(c, w).forward(toks, SuboraxOracle(c, w).new_state(), 0)
    bad = SuboraxOracle(c, w)
    if what == "sink":
        for n in w:
            if n.endswith("sink"):
                bad.w[n] = torch.full_like(bad.w[n], -1e9)
    elif what == "cap":
        for l in c["layers"]:
            l["mixer"]["softcap"] = 0.0
    elif what == "scaling":
        for l in c["layers"]:
            del l["mixer"]["rot"]["scaling"]
    elif what == "offset":
        bad.w = {n: (t - 1.0 if "norm" in n else t) for n, t in bad.w.items()}
    elif what == "alpha":
        c["postln_alpha"] = 1.0
    st = bad.new_state()
    if what == "causal_far":  # the first 32 keys are lost between two portions
        a = bad.forward(toks[:64], st, 0)
        for s in st:
            s.v[:32] = 0
        b = bad.forward(toks[64:], st, 64)
        got = torch.cat([a, b])
    else:
        bad.c = c
        got = bad.forward(toks, st, 0)
    err = ((got - good)[70:].pow(2).mean(-1).sqrt() / good.std()).median()
    assert err > 0.03, float(err)


# ---------------------------------------------------------------- product, host side
@pytest.mark.parametrize("scaling", [None, SCALING, {"factor": 32.0, "low": 1.0, "high": 4.0, "original": 8192}])
def test_rotary_tables_match_the_oracle_frequencies(scaling):
    from mirage.mpk.models.checkpoint import rotary_frequencies as product, rotary_tables_f32
    rot = {"dims": 48, "base": 5e5, **({"scaling": scaling} if scaling else {})}
    assert torch.allclose(product(48, 5e5, scaling), rotary_frequencies(rot), rtol=1e-14)
    cos, sin = rotary_tables_f32(48, 5e5, scaling, 3000, device="cpu")
    ang = 2999.0 * rotary_frequencies(rot)
    assert cos.dtype == torch.float32 and torch.allclose(cos[2999].double(), ang.cos(), atol=1e-7) and torch.allclose(sin[2999].double(), ang.sin(), atol=1e-7)


def test_config_reader():
    from mirage.mpk.models.suborax.builder import SuboraxConfig
    c = SuboraxConfig.from_dict(CONFIGS["odd"])
    assert (c.vocab, c.width, c.alpha, c.embedding_scale, c.eps) == (133, 84, 0.9, 3.0, 1e-5)
    assert [l.ff for l in c.layers] == [75, None, 33] and c.layers[1].softcap == 4.0 and c.layers[0].rot_scaling is None
    shapes = c.tensor_shapes()
    assert shapes["l2.mix.q"] == (320, 84) and shapes["l1.mix.o"] == (84, 6 * 88) and "l1.norm2" not in shapes and shapes["l0.mlp.down"] == (84, 75)
    for path, value in ((("layers", 0, "type"), "other"), (("layers", 0, "mlp", "kind"), "other"), (("layers", 1, "mixer", "kv_heads"), 4)):
        bad = json.loads(json.dumps(CONFIGS["odd"]))
        d = bad
        for k in path[:-1]:
            d = d[k]
        d[path[-1]] = value
        with pytest.raises(ValueError):
            SuboraxConfig.from_dict(bad)


def test_registry_picks_the_builder_by_config():
    from mirage.mpk.model_registry import get_builder, model_name_of
    from mirage.mpk.models.qwen3 import Qwen3Builder
    from mirage.mpk.models.suborax import SuboraxBuilder
    assert get_builder(model_name_of({"architecture": "Suborax"})) is SuboraxBuilder
    assert get_builder(model_name_of({"architectures": ["Qwen3ForCausalLM"]})) is Qwen3Builder
    with pytest.raises(ValueError):
        model_name_of({"architecture": "Nobody"})


def _host_mpk(c, dtype=torch.bfloat16, B=64, **kw):
    from mirage.mpk import MPK, MirageModelConfig, MPKMetadata
    m = MPK(MPKMetadata(mode="online_notoken", max_seq_length=256, max_num_batched_requests=min(4, B), max_num_batched_tokens=B, max_num_pages=8, page_size=64, device="cpu",
                        num_workers=256, dtype=dtype, model_config=MirageModelConfig(architecture=c, state_dict=weights(c)), **kw))
    m.build()
    return m


def _ops(c, *args, **kw):
    m = _host_mpk(c, *args, **kw)
    return [l.split()[1] for l in m.persistent_kernel.describe_program().splitlines()]


def test_lowering_of_one_layer():
    """The stage program of a layer, in the bf16 build (norms folded into the linears of single-token iterations, SwiGLU in
    the gate/up linear, no separate activation stage) and in the 32-bit one."""
    c = config([layer(4, 2, 64, 32, 32, 96)], 128, 100)
    assert _ops(c) == ["FX_EMBED", "LINEAR", "FX_PREP[portions]", "FX_ATTN", "LINEAR", "FX_ADDNORM[multi-token", "LINEAR+silu", "LINEAR", "FX_ADDNORM", "FX_ADDNORM[multi-token",
                       "LINEAR", "ARGMAX_PARTIAL", "ARGMAX_REDUCE"]
    assert "FX_PREP[portions]" not in _ops(c, B=1)
    f32 = _ops(c, torch.float32)
    assert f32.count("LINEAR_F32") == 4 and f32.count("LINEAR_F32+silu") == 1 and f32.count("FX_ADDNORM") == 3
    m = _host_mpk(c)
    assert len(json.loads(m.generate_task_graph()["json_file"])["all_tasks"]) > 2


def test_builder_refuses_what_does_not_fit():
    from mirage.mpk import MPK, MirageModelConfig, MPKMetadata
    c = CONFIGS["even"]
    w = weights(c)
    del w["l1.mix.k"]
    meta = dict(mode="online_notoken", max_seq_length=64, max_num_batched_requests=1, max_num_batched_tokens=8, max_num_pages=1, page_size=64, device="cpu", num_workers=256)
    with pytest.raises(KeyError, match="l1.mix.k"):
        MPK(MPKMetadata(model_config=MirageModelConfig(architecture=c, state_dict=w), **meta)).build()
    w = weights(c)
    w["l0.mix.v"] = w["l0.mix.v"][:-1]
    with pytest.raises(ValueError, match="l0.mix.v"):
        MPK(MPKMetadata(model_config=MirageModelConfig(architecture=c, state_dict=w), **meta)).build()
    w["l0.mix.v"] = weights(c)["l0.mix.v"]
    with pytest.raises(Exception, match="page_size"):
        m = MPK(MPKMetadata(model_config=MirageModelConfig(architecture=c, state_dict=w), **{**meta, "page_size": 40, "max_num_pages": 2}))
        m.build()
        m.persistent_kernel.describe_program()


def test_qwen3_builder_refuses_32_bit():
    from mirage.mpk.models.qwen3 import Qwen3Builder
    b = Qwen3Builder.__new__(Qwen3Builder)
    with pytest.raises(NotImplementedError):
        Qwen3Builder.set_dtype(b, torch.float32)


def test_flex_tasks_check_their_operands():
    import mirage as mi
    from helpers import make_meta, make_mpk
    pk = make_mpk(make_meta(2, 64, 8, 2, 4, device="cpu"), 64, 8, 2, 4, 32, num_workers=256)
    new = lambda name, cols, dt=mi.float32: pk.new_tensor((8, cols), dtype=dt, name=name)
    x, xo, o, wt = new("x", 64), new("xo", 64), new("o", 64, mi.bfloat16), pk.new_tensor((64,), dtype=mi.float32, name="w")
    pk.residual_rmsnorm_layer(None, x, wt, x, o)  # the new rows may not overwrite the old ones
    with pytest.raises(Exception, match="overwrite"):
        pk.describe_program()


def test_page_pool_and_step_packing():
    """ServingSession's bookkeeping with the launch replaced by a recorder: passes are packed single tokens first, pages
    grow with the request, are given back, and used again."""
    from mirage.mpk.serving import PagePool, ServingSession

    class Stub:
        pass

    s = ServingSession.__new__(ServingSession)
    s.page_size, s.max_rows, s.max_requests, s.rows_per_request, s.max_seq = 4, 8, 3, 8, 64
    s.pool, s.requests, passes = PagePool(6), {}, []
    s.mpk = Stub()
    s.mpk.output_tokens = torch.arange(8)
    s.logits = lambda: torch.arange(8.0)[:, None]

    def run(batch):
        for rid, toks in batch:
            r = s.requests.setdefault(rid, type("R", (), {"pages": [], "length": 0})())
            r.length += len(toks)
            r.pages += s.pool.take(-(-r.length // 4) - len(r.pages))
        passes.append([(rid, len(t)) for rid, t in batch])

    s._pass = run
    lg, greedy = s.step([("a", list(range(11))), ("b", [1])], [[0, 10, 10], [0]])
    assert passes == [[("b", 1), ("a", 7)], [("a", 4)]]
    assert lg.flatten().tolist() == [1.0, 3.0, 3.0, 0.0] and greedy == [3, 0]
    assert len(s.pool) == 2 and len(s.requests["a"].pages) == 3
    mine = list(s.requests["a"].pages)
    s.end("a")
    s.step([("c", [1] * 5)])
    assert s.requests["c"].pages == mine[:2] and len(s.pool) == 3
    with pytest.raises(ValueError):
        s.step([("b", [1]), ("b", [2])])
    with pytest.raises(ValueError):
        s.step([("b", [1] * 64)])
    with pytest.raises(RuntimeError):
        s.pool.take(4)
