"""Bukatar graph builder: a decoder with a norm before and behind each sub-layer whose layers mix three kinds of token mixer (windowed
attention, latent attention, selective scan) with dense and expert feed-forwards.

A layer keeps a 32-bit residual stream x (N: RMS norm):

    x <- x + N1b(mixer(N1(x)));   x <- x + N2b(ff(N2(x)))          (the second only where the layer has a feed-forward)

What a layer records (every sum and norm between two sub-layers is ONE residual_prenorm, which also adds the output projection's
bias or forms the weighted sum of a token's experts):

    attention:        linear (q, k) -> flex_attention (biases, window, kept first positions, unit sink, values from keys) -> linear
    latent attention: linear (queries, latent, rotated part) -> latent_prep -> head_linear (into the latent space)
                      -> latent_attention -> head_linear (out of it) -> linear
    selective scan:   linear (x, z) -> short_conv -> linear (step, B, C) -> scan_step -> selective_scan -> linear
    dense:            linear + relu_squared -> linear
    experts:          head_linear (router and shared gate, 32-bit sums) -> expert_route -> expert_linear (gated) -> expert_linear

Latent layers with `kv_from` read the rows another layer has cached.  Rotations of neighbouring dimensions become the kernels'
rotation of halves by an order of the projection's rows.  Sizes need no alignment: sections of fused matrices, heads and channels are
padded with zero rows or columns.  Checkpoint names: `embed` (also the output matrix), `l<i>.{norm1,norm1b,norm2,norm2b}`,
`l<i>.mix.{q,q.b,k,k.b,o,o.b}`, `l<i>.mix.{q,dkv,dkv.norm,uk,uv,o}` or `l<i>.mix.{in,conv,conv.b,x,dt,dt.b,A_log,D,o}`,
`l<i>.mlp.{up,down}` or `l<i>.mlp.{router,e<j>.{gate,up,down},shared.{gate,up,down,sg}}`, `final.norm`; linear weights are [out, in].

Runs in bfloat16 (the served form) and float32 (everything in true 32-bit).
"""
import math
from dataclasses import dataclass
from typing import List, Optional

import torch

from ...model_registry import register_model_builder
from ...persistent_kernel import PersistentKernel, flex_cache_dims, latent_row_dim, operand_row, operand_tiles, pairs_to_halves
from ....kernel import float32, int32
from ..graph_builder import MirageModelConfig
from ..layer_list import LayerListBuilder, up_to as _up


def _rot(m: dict):
    rot = m.get("rot") or {"dims": 0, "base": 1.0}
    if rot["dims"] % 2:
        raise ValueError(f"a rotation over {rot['dims']} dimensions")
    return rot["dims"], float(rot["base"])


@dataclass
class WindowMixer:
    heads: int
    kv_heads: int
    dim: int
    rot_dims: int
    rot_base: float
    scale: float
    window: int  # 0: every earlier position is seen
    keep_first: int

    def tensor_shapes(self, W):
        q, k = self.heads * self.dim, self.kv_heads * self.dim
        return {"q": (q, W), "q.b": (q,), "k": (k, W), "k.b": (k,), "o": (W, q), "o.b": (W,)}


@dataclass
class LatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    kv_rank: int
    rot_base: float
    scale: float
    kv_from: Optional[int]

    def tensor_shapes(self, W):
        H = self.heads
        out = {"q": (H * (self.dim + self.rot_dim), W)}
        if self.kv_from is None:
            out.update({"dkv": (self.kv_rank + self.rot_dim, W), "dkv.norm": (self.kv_rank,)})
        out.update({"uk": (H * self.dim, self.kv_rank), "uv": (H * self.vdim, self.kv_rank), "o": (W, H * self.vdim)})
        return out


@dataclass
class ScanMixer:
    inner: int
    state: int
    conv: int
    dt_rank: int

    @property
    def channels(self):
        return _up(self.inner, 64)

    @property
    def padded_state(self):
        return _up(self.state, 4)

    def tensor_shapes(self, W):
        n = self.inner
        return {"in": (2 * n, W), "conv": (n, self.conv), "conv.b": (n,), "x": (self.dt_rank + 2 * self.state, n), "dt": (n, self.dt_rank), "dt.b": (n,),
                "A_log": (n, self.state), "D": (n,), "o": (W, n)}


@dataclass
class DenseFF:
    ff: int

    def tensor_shapes(self, W):
        return {"up": (self.ff, W), "down": (W, self.ff)}


@dataclass
class ExpertFF:
    experts: int
    top: int
    ff: int
    shared_ff: Optional[int]

    def tensor_shapes(self, W):
        out = {"router": (self.experts, W)}
        units = [(f"e{j}", self.ff) for j in range(self.experts)] + ([] if self.shared_ff is None else [("shared", self.shared_ff)])
        for name, ff in units:
            out.update({f"{name}.gate": (ff, W), f"{name}.up": (ff, W), f"{name}.down": (W, ff)})
        if self.shared_ff is not None:
            out["shared.sg"] = (1, W)
        return out


@dataclass
class BukatarLayer:
    mixer: object
    ff: object  # None: the layer has no feed-forward


@dataclass
class BukatarConfig:
    vocab: int
    width: int
    eps: float
    layers: List[BukatarLayer]

    @staticmethod
    def from_dict(c: dict) -> "BukatarConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            m, mlp, kind = e["mixer"], e.get("mlp"), e["type"]
            if kind == "attention":
                mask, (dims, base) = m.get("mask") or {}, _rot(m)
                if m["heads"] % m["kv_heads"] or m.get("vdim", m["dim"]) != m["dim"] or dims > m["dim"]:
                    raise ValueError(f"layer {i}: {m['heads']} query heads over {m['kv_heads']} key heads of {m['dim']} that are values of {m.get('vdim')}, {dims} rotated")
                mixer = WindowMixer(m["heads"], m["kv_heads"], m["dim"], dims, base, m["scale"], mask.get("size") or 0, mask.get("keep_first") or 0)
            elif kind == "latent_attention":
                dims, base = _rot(m)
                if dims != m["rot_dim"]:
                    raise ValueError(f"layer {i}: rotation over {dims} of a rotated part of {m['rot_dim']}")
                mixer = LatentMixer(m["heads"], m["dim"], dims, m["vdim"], m["kv_rank"], base, m["scale"], m.get("kv_from"))
                if mixer.kv_from is not None:
                    src = layers[mixer.kv_from].mixer if 0 <= mixer.kv_from < i else None
                    if not isinstance(src, LatentMixer) or src.kv_from is not None or (src.kv_rank, src.rot_dim, src.rot_base) != (mixer.kv_rank, dims, base):
                        raise ValueError(f"layer {i}: kv_from={mixer.kv_from} names no earlier layer with a latent of the same form")
            elif kind == "mamba1":
                mixer = ScanMixer(m["inner"], m["state"], m["conv"], m["dt_rank"])
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            if mlp is None:
                ff = None
            elif mlp.get("kind", "dense") == "dense":
                ff = DenseFF(mlp["ff"])
            elif mlp["kind"] == "moe":
                ff = ExpertFF(mlp["router"]["experts"], mlp["router"]["top"], mlp["expert"]["ff"], mlp["shared"]["ff"] if mlp.get("shared") else None)
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layers.append(BukatarLayer(mixer, ff))
        return BukatarConfig(c["vocab"], c["width"], c["norm"]["eps"], layers)

    def tensor_shapes(self) -> dict:
        """Checkpoint name -> shape."""
        W, out = self.width, {"embed": (self.vocab, self.width)}
        for i, l in enumerate(self.layers):
            p = f"l{i}."
            out.update({p + "norm1": (W,), p + "norm1b": (W,)})
            out.update({p + "mix." + k: s for k, s in l.mixer.tensor_shapes(W).items()})
            if l.ff is not None:
                out.update({p + "norm2": (W,), p + "norm2b": (W,)})
                out.update({p + "mlp." + k: s for k, s in l.ff.tensor_shapes(W).items()})
        out["final.norm"] = (W,)
        return out

    def weight_bytes_per_token(self, elem=2):
        """Weight bytes one single-token step streams (output matrix included; of the experts those one token visits)."""
        total = 0
        for name, s in self.tensor_shapes().items():
            if len(s) != 2 or name.endswith((".conv", ".A_log")):
                continue
            share = 1.0
            if ".mlp.e" in name:
                ff = self.layers[int(name[1:name.index(".")])].ff
                share = ff.top / ff.experts
            total += s[0] * s[1] * share
        return int(elem * total)

    def kv_bytes_per_position(self, elem=2):
        out = 0
        for l in self.layers:
            m = l.mixer
            if isinstance(m, LatentMixer):
                out += m.kv_rank + m.rot_dim
            elif isinstance(m, WindowMixer) and not m.window:
                out += 2 * m.kv_heads * m.dim
        return elem * out

    def state_bytes(self):
        """Recurrent state of one request (read and written by every step)."""
        return 4 * sum(l.mixer.inner * l.mixer.state for l in self.layers if isinstance(l.mixer, ScanMixer))


def random_state_dict(cfg: BukatarConfig, seed: int = 0, device="cuda", std: float = 0.02) -> dict:
    """Random-init weights: matrices ~ N(0, std), norm weights and D 1, biases 0, step offsets -3, A from 1 to the number of states."""
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        if name.endswith(".A_log"):
            t = torch.arange(1, shape[1] + 1, dtype=torch.float32, device=device).log().expand(shape)
        elif len(shape) == 2:
            t = torch.empty(shape, dtype=torch.bfloat16, device=device).normal_(0.0, std, generator=g)
        else:
            t = torch.full(shape, -3.0 if name.endswith(".dt.b") else 0.0 if name.endswith(".b") else 1.0, device=device)
        out[name] = t.to(torch.bfloat16).contiguous()
    return out


@register_model_builder("Bukatar")
class BukatarBuilder(LayerListBuilder):

    def __init__(self, mpk: PersistentKernel, weights: Optional[dict] = None):
        super().__init__(mpk, weights)
        self.k_cache, self.v_cache, self.latent_cache, self.state, self.tail, self.state_slots = {}, {}, {}, {}, {}, None
        self._tables, self._attached = {}, {}

    @classmethod
    def kernels(cls, dtype, max_num_batched_tokens):
        if dtype == torch.float32:
            return ("HYB_F32",)
        return ("HYB_M1",) if max_num_batched_tokens == 1 else ("HYB",)

    # ------------------------------------------------------------------ entry points
    def build_from_config(self, model_config: MirageModelConfig):
        """`model_config.architecture` is the parsed config.json; caches and states are allocated here."""
        self.config = BukatarConfig.from_dict(model_config.architecture)
        self.build_from_dict(model_config.state_dict, model_config.with_lm_head)

    def build_from_model(self, model_name: str = None, model_path: str = None):
        from .. import checkpoint
        if model_path is None:
            raise ValueError(f"model '{model_name}': a local model_path is required (no hub access); it must hold config.json and *.safetensors")
        cfg, state_dict = checkpoint.load_checkpoint(model_path, device=self.mpk.device, dtype=None, required=("embed", "final.norm"))
        self.config = BukatarConfig.from_dict(cfg)
        self.tokenizer = checkpoint.load_tokenizer(model_path)
        self.build_from_dict(state_dict, True)

    # ------------------------------------------------------------------ tensors
    def _rotary(self, dims: int, base: float):
        from .. import checkpoint
        if dims == 0:
            return None, None
        if (dims, base) not in self._tables:
            cos, sin = checkpoint.rotary_tables_f32(dims, base, None, self.mpk.max_seq_length, self.mpk.device)
            n = len(self._tables)
            self._tables[dims, base] = (self._attach(cos, f"cos_{n}"), self._attach(sin, f"sin_{n}"))
        return self._tables[dims, base]

    def _latents(self, i: int):
        """The latent rows layer `i` owns, attached once for every layer that reads them."""
        if i not in self._attached:
            self._attached[i] = self._attach(self.latent_cache[i], f"l{i}.latent_cache")
        return self._attached[i]

    def allocate_caches(self):
        """Keys and values or latent rows in pages; scan states [slots, channels, states] and convolution tails in slots."""
        mpk = self.mpk
        zeros = lambda *shape, dtype=self.dtype: torch.zeros(*shape, dtype=dtype, device=mpk.device)
        for i, l in enumerate(self.config.layers):
            m = l.mixer
            if isinstance(m, ScanMixer):
                self.state[i] = zeros(mpk.max_num_batched_requests, m.channels, m.padded_state, dtype=torch.float32)
                self.tail[i] = zeros(mpk.max_num_batched_requests, max(m.conv - 1, 1), m.channels)
            elif isinstance(m, WindowMixer):
                dk, dv = flex_cache_dims(m.dim, m.dim, self.dtype)
                self.k_cache[i] = zeros(mpk.max_num_pages, mpk.page_size, m.kv_heads, dk)
                self.v_cache[i] = zeros(mpk.max_num_pages, mpk.page_size, m.kv_heads, dv)
            elif m.kv_from is None:
                self.latent_cache[i] = zeros(mpk.max_num_pages, mpk.page_size, latent_row_dim(m.kv_rank, m.rot_dim, self.dtype))
        if self.state:
            self.state_slots = self._new_state_slots()

    # ------------------------------------------------------------------ sub-layers: each returns what the next residual sum takes
    def _window(self, i: int, p: str, m: WindowMixer, h):
        mpk, E, H, G, D = self.mpk, self._E, m.heads, m.kv_heads, m.dim
        order = pairs_to_halves(D, m.rot_dims).to(self._w(p + "q").device)
        by_head = lambda w: w.view(-1, D, *w.shape[1:])[:, order].reshape(w.shape)
        nq, nk = H * D, G * D
        w_in, _, cols = self._sections([("q", by_head(self._w(p + "q")), nq), ("k", by_head(self._w(p + "k")), _up(nq + nk, 16) - nq)])
        qk = self._linear(h, w_in, p + "qk", self._rows("sublayers_in", cols, E))
        bias = torch.nn.functional.pad(torch.cat([by_head(self._w(p + "q.b")), by_head(self._w(p + "k.b"))]).to(torch.float32), (0, cols - nq - nk))
        cos, sin = self._rotary(m.rot_dims, m.rot_base)
        dk, _ = flex_cache_dims(D, D, self.dtype)
        A = _up(nq, 64)
        out = self._rows(f"attn_out_{nq}", A, E)
        mpk.flex_attention_layer(input=qk, k_cache=self._attach(self.k_cache[i], p + "k_cache"), v_cache=self._attach(self.v_cache[i], p + "v_cache"), cos=cos, sin=sin,
                                 sink=self._attach(torch.zeros(H, dtype=torch.float32, device=w_in.device), p + "sink"), q_workspace=self._rows("q_ws", H * dk, E), output=out,
                                 num_q_heads=H, num_kv_heads=G, head_dim=D, v_dim=D, rot_dims=m.rot_dims, scale=m.scale, window=m.window, keep_first=m.keep_first,
                                 values_from_keys=True, input_bias=self._attach(bias, p + "qk.b"))
        w_o = by_head(self._matrix(p + "o").T).T  # (a head's outputs come in the order of its keys)
        return dict(input=self._linear(out, self._pad(w_o, cols=A), p + "o", self._y), input_bias=self._vector(p + "o.b", self._W))

    def _latent(self, i: int, p: str, m: LatentMixer, h):
        mpk, E, KW, H, P = self.mpk, self._E, operand_row(self.dtype), m.heads, m.rot_dim
        dev = self._w(p + "q").device
        order = pairs_to_halves(P, P).to(dev)
        dp, rp, Rp = _up(m.dim, KW), _up(P, 16), _up(m.kv_rank, KW)
        hs = dp + rp  # a head's query columns: unrotated part, rotated part, each padded
        w = self._w(p + "q").view(H, m.dim + P, -1)
        q_w = torch.zeros(H, hs, w.shape[2], dtype=w.dtype, device=dev)
        q_w[:, :m.dim] = w[:, :m.dim]
        q_w[:, dp:dp + P] = w[:, m.dim:][:, order]
        parts = [("q", q_w.view(H * hs, -1), H * hs)]
        if m.kv_from is None:
            dkv = self._w(p + "dkv")
            parts += [("c", dkv[:m.kv_rank], _up(m.kv_rank, 16)), ("rot", dkv[m.kv_rank:][order], rp)]
        w_in, col, cols = self._sections(parts)
        rows = self._linear(h, w_in, p + "in", self._rows("sublayers_in", cols, E))
        cos, sin = self._rotary(P, m.rot_base)
        cache = self._latents(i if m.kv_from is None else m.kv_from)
        if m.kv_from is None:
            mpk.latent_prep_layer(input=rows, eps=self.config.eps, cache=cache, latent_weight=self._vector(p + "dkv.norm", _up(m.kv_rank, 4)), cos=cos, sin=sin,
                                  latent_column=col["c"], latent_rank=m.kv_rank, rot_column=col["rot"], rot_dims=P)
        uk = self._pad(self._w(p + "uk").to(self.dtype).view(H, m.dim, m.kv_rank).transpose(1, 2), Rp, dp)
        ql, ol = self._rows("queries_in_latent", H * Rp, E), self._rows("latent_sums", H * Rp, E)
        mpk.head_linear_layer(input=rows, weight=self._attach(operand_tiles(uk), p + "uk"), output=ql, heads=H, n=Rp, k=dp, in_stride=hs, out_stride=Rp)
        mpk.latent_attention_layer(input=rows, q_latent=ql, cache=cache, cos=cos, sin=sin, output=ol, num_heads=H, latent_rank=m.kv_rank, rot_dims=P, head_stride=hs,
                                   rot_column=dp, scale=m.scale)
        A = _up(H * m.vdim, 64)
        out = self._rows(f"latent_out_{H * m.vdim}", A, E)
        uv = operand_tiles(self._w(p + "uv").to(self.dtype).view(H, m.vdim, m.kv_rank))
        mpk.head_linear_layer(input=ol, weight=self._attach(uv, p + "uv"), output=out, heads=H, n=m.vdim, k=Rp, in_stride=Rp, out_stride=m.vdim)
        return dict(input=self._linear(out, self._matrix(p + "o", cols=A), p + "o", self._y))

    def _scan(self, i: int, p: str, m: ScanMixer, h):
        mpk, E, I, N, Np, K = self.mpk, self._E, m.channels, m.state, m.padded_state, _up(m.dt_rank, operand_row(self.dtype))
        w = self._w(p + "in")
        w_in, col, cols = self._sections([("x", w[:m.inner], I), ("z", w[m.inner:], I)])
        xz = self._linear(h, w_in, p + "in", self._rows("sublayers_in", cols, E))
        slots, tail = self._slots, self._attach(self.tail[i], p + "tail")
        taps = torch.zeros(m.conv, I, dtype=torch.float32, device=w_in.device)
        taps[:, :m.inner] = self._w(p + "conv").T
        x = self._rows("convolved", I, E)
        mpk.short_conv_layer(input=xz, weight=self._attach(taps, p + "conv"), bias=self._vector(p + "conv.b", I), tail=tail, state_slots=slots, output=x, column=col["x"])
        w = self._w(p + "x").to(self.dtype)
        r, s = m.dt_rank, _up(N, 16)
        w_x = torch.zeros(_up(K, 16) + 2 * s, I, dtype=self.dtype, device=w.device)
        for at, lo, hi in ((0, 0, r), (_up(K, 16), r, r + N), (_up(K, 16) + s, r + N, r + 2 * N)):
            w_x[at:at + hi - lo, :m.inner] = w[lo:hi]
        dbc = self._linear(x, w_x, p + "x", self._rows("step_b_c", w_x.shape[0], E))
        step = self._rows("steps", I, float32)
        mpk.scan_step_layer(input=dbc, weight=self._attach(operand_tiles(self._matrix(p + "dt", I, K)[None]), p + "dt"), offset=self._vector(p + "dt.b", I), output=step, n=I, k=K)
        A = (-torch.exp(self._w(p + "A_log").to(torch.float64)) / math.log(2.0)).to(torch.float32)
        out = self._rows(f"scan_out_{m.inner}", I, E)
        mpk.selective_scan_layer(input=xz, conv=x, step=step, bc=dbc, A=self._attach(self._pad(A, I, Np), p + "A"), D=self._vector(p + "D", I),
                                 state=self._attach(self.state[i], p + "state"), tail=tail, state_slots=slots, output=out, states=N, taps=m.conv, x_column=col["x"],
                                 z_column=col["z"], b_column=_up(K, 16), c_column=_up(K, 16) + s)
        return dict(input=self._linear(out, self._matrix(p + "o", cols=I), p + "o", self._y))

    def _dense(self, i: int, p: str, f: DenseFF, h):
        F = _up(f.ff, 64)
        up = self._linear(h, self._matrix(p + "up", F, self._W), p + "up", self._rows("ff_up", F, self._E))  # never written: the activation is the linear's epilogue
        act = self._rows("ff_act", F, self._E)
        self.mpk.relu_squared_layer(input=up, output=act)
        return dict(input=self._linear(act, self._matrix(p + "down", cols=F), p + "down", self._y))

    def _experts(self, i: int, p: str, f: ExpertFF, h):
        mpk, W = self.mpk, self._W
        shared, top = f.shared_ff is not None, f.top
        router = self._matrix(p + "router", cols=W)
        if shared:
            router = torch.cat([router, self._matrix(p + "shared.sg", cols=W)])
        n = router.shape[0]
        z = self._rows("router_logits", _up(n, 4), float32)
        mpk.head_linear_layer(input=h, weight=self._attach(operand_tiles(router[None]), p + "router"), output=z, heads=1, n=n, k=W, in_stride=0, out_stride=0)
        ids, shares = self._rows(f"expert_ids_{i}", top, int32), self._rows(f"expert_shares_{i}", _up(top + 1, 4), float32)
        mpk.expert_route_layer(z, ids, shares, f.experts, top, shared)

        y, places = self._expert_linears(p, h, ids, f.experts, top, f.ff, f.shared_ff)
        return dict(input=y, slot_weights=shares, slots=places, slot_columns=W)

    # ------------------------------------------------------------------ graph
    def build_from_dict(self, state_dict: dict, with_lm_head: bool = True):
        mpk, c = self.mpk, self.config
        self._begin(c, state_dict, with_lm_head)
        if mpk.spec_decode_config is not None and any(isinstance(l.mixer, ScanMixer) for l in c.layers):
            raise NotImplementedError("speculative decoding: rows of rejected guesses cannot be taken back out of a recurrent state")
        f32, E, W = self.dtype == torch.float32, self._E, self._W
        self.allocate_caches()
        self._slots = self._attach(self.state_slots, "state_slots") if self.state else None
        # the residual rows alternate between two buffers: a single-token iteration forms the new rows in every workgroup of
        # the linear that reads them, from the old ones
        streams = [self._rows("residual_a", W, float32), self._rows("residual_b", W, float32)]
        which = 0
        h, x16 = self._rows("normed", W, E), self._rows("stream", W, E)
        self._y = self._rows("sublayer_out", W, E)

        def join(norm_behind, weight, **summand):
            nonlocal which
            old, which = streams[which], 1 - which
            mpk.residual_prenorm_layer(**{"input": None, **summand}, input_weight=norm_behind, residual=old, weight=weight, new_residual=streams[which], output=h, width=c.width,
                                       eps=c.eps, input_eps=c.eps)

        ids, spec, spec_tokens = self._token_ids(with_lm_head)
        embed = self._attach(self._matrix("embed", cols=W), "embed")
        mpk.embed_scaled_layer(input=ids, weight=embed, residual=streams[which], output=streams[which] if f32 else x16)
        summand, behind = {}, None
        mixers = {WindowMixer: self._window, LatentMixer: self._latent, ScanMixer: self._scan}
        for i, l in enumerate(c.layers):
            p = f"l{i}."
            join(behind, self._vector(p + "norm1", W), **summand)
            summand, behind = mixers[type(l.mixer)](i, p + "mix.", l.mixer, h), self._vector(p + "norm1b", W)
            if l.ff is not None:
                join(behind, self._vector(p + "norm2", W), **summand)
                ff = self._dense if isinstance(l.ff, DenseFF) else self._experts
                summand, behind = ff(i, p + "mlp.", l.ff, h), self._vector(p + "norm2b", W)
        join(behind, self._vector("final.norm", W), **summand)
        self.hidden = h
        if not with_lm_head:
            self._state = None
            return
        self._head_and_sampling(h, embed, c.vocab, spec, spec_tokens)
        self._state = None
