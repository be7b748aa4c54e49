"""Vizonex graph builder: a decoder whose two sub-layers work side by side on one norm of the residual stream.

A layer keeps a 32-bit residual stream x (N: RMS norm, conv: short causal convolution over time, per channel):

    h = N(x);   x <- x + s1 * mixer(h + conv(h)) + s2 * ff(h)          (s1, s2: vectors; the last term only where there is a feed-forward)

What a layer records (the sum of two sub-layers, the norm behind it and the convolution of single tokens are ONE residual_prenorm):

    norm:        residual_prenorm (both summands with their factors, weighted sum of a token's experts) -> ring_conv (prompt portions)
    attention:   linear (q, k, v) -> flex_attention (chunks, norms over all heads of a row, score factors, sink) -> linear
    recurrence:  linear (gate z, x, B, C, step) -> ring_conv (silu, step sizes and decays) -> dual_scan -> residual_prenorm (norm in parts) -> linear
    dense:       linear + gelu_mul -> linear
    experts:     head_linear (router, 32-bit sums) -> expert_route (groups) -> expert_linear (clamped) -> expert_linear

Positions enter as a learned vector added to the embedding, so a sequence is no longer than the table.  Sizes need no alignment.
Checkpoint names: `embed`, `pos`, `head`, `final.norm`, `l<i>.{norm1,canon1,ls1,ls2}`, `l<i>.mix.{q,k,v,q.norm,k.norm,temp,sink,o}` or
`l<i>.mix.{in,conv,conv.b,dt_bias,A_log,D,norm,o}`, `l<i>.mlp.{gate,up,down}` or `l<i>.mlp.{router,correction,{e<j>,shared}.{gate,up,down}}`;
linear weights are [out, in].

Runs in bfloat16 (the served form) and float32 (everything in true 32-bit).
"""
import math
from dataclasses import dataclass
from typing import List, Optional

import torch

from ...model_registry import register_model_builder
from ...persistent_kernel import PersistentKernel, flex_cache_dims, operand_tiles
from ....kernel import float32, int32
from ..graph_builder import MirageModelConfig
from ..layer_list import LayerListBuilder, up_to

GLU_BETA, GLU_BIAS = 1.702, 1.0  # of the experts' activation: g sigmoid(beta g) (u + bias)


@dataclass
class ChunkMixer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    chunk: int  # 0: every earlier position is seen

    def tensor_shapes(self, W):
        q, k, v = self.heads * self.dim, self.kv_heads * self.dim, self.kv_heads * self.vdim
        return {"q": (q, W), "k": (k, W), "v": (v, W), "q.norm": (q,), "k.norm": (k,), "temp": (self.heads,), "sink": (self.heads,), "o": (W, self.heads * self.vdim)}


@dataclass
class DualMixer:
    heads: int
    vdim: int
    state: int
    groups: int
    norm_groups: int
    conv: int

    @property
    def inner(self):
        return self.heads * self.vdim

    @property
    def padded_state(self):
        return up_to(self.state, 4)

    def tensor_shapes(self, W):
        I, H = self.inner, self.heads
        n = I + 2 * self.groups * self.state
        return {"in": (I + n + H, W), "conv": (n, self.conv), "conv.b": (n,), "dt_bias": (H,), "A_log": (H,), "D": (H,), "norm": (I,), "o": (W, I)}


@dataclass
class DenseFF:
    ff: int

    def tensor_shapes(self, W):
        return {"gate": (self.ff, W), "up": (self.ff, W), "down": (W, self.ff)}


@dataclass
class ExpertFF:
    experts: int
    top: int
    groups: int
    keep: int
    scale: float
    ff: int
    limit: float
    shared_ff: Optional[int]
    shared_limit: float

    def tensor_shapes(self, W):
        out = {"router": (self.experts, W), "correction": (self.experts,)}
        units = [(f"e{j}", self.ff) for j in range(self.experts)] + ([] if self.shared_ff is None else [("shared", self.shared_ff)])
        for name, ff in units:
            out.update({f"{name}.gate": (ff, W), f"{name}.up": (ff, W), f"{name}.down": (W, ff)})
        return out


@dataclass
class VizonexLayer:
    mixer: object
    ff: object  # None: the layer has no feed-forward


@dataclass
class VizonexConfig:
    vocab: int
    width: int
    eps: float
    taps: int  # of the convolution in front of every mixer
    max_positions: int
    layers: List[VizonexLayer]

    @staticmethod
    def from_dict(c: dict) -> "VizonexConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            m, mlp, kind = e["mixer"], e.get("mlp"), e["type"]
            if kind == "attention":
                if m["heads"] % m["kv_heads"]:
                    raise ValueError(f"layer {i}: {m['heads']} query heads over {m['kv_heads']} key heads")
                mixer = ChunkMixer(m["heads"], m["kv_heads"], m["dim"], m["vdim"], m["scale"], (m.get("mask") or {}).get("size") or 0)
            elif kind == "mamba2":
                mixer = DualMixer(m["heads"], m["vdim"], m["state"], m["groups"], m["norm_groups"], m["conv"])
                if mixer.heads % mixer.groups or mixer.inner % mixer.norm_groups:
                    raise ValueError(f"layer {i}: {mixer.heads} heads of {mixer.vdim} in {mixer.groups} groups, normalised in {mixer.norm_groups} parts")
            else:
                raise ValueError(f"layer {i}: unknown mixer type {kind!r}")
            if mlp is None:
                ff = None
            elif mlp.get("kind", "dense") == "dense":
                ff = DenseFF(mlp["ff"])
            elif mlp["kind"] == "moe":
                r, s = mlp["router"], mlp.get("shared")
                g = r.get("groups") or {"count": 1, "keep": 1}
                ff = ExpertFF(r["experts"], r["top"], g["count"], g["keep"], r["scale"], mlp["expert"]["ff"], mlp["expert"]["limit"], s["ff"] if s else None, s["limit"] if s else 0.0)
                if ff.experts % ff.groups or not 0 < ff.keep <= ff.groups or ff.top > ff.keep * (ff.experts // ff.groups):
                    raise ValueError(f"layer {i}: {ff.top} of {ff.experts} experts in {ff.groups} groups of which {ff.keep} stay open")
            else:
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layers.append(VizonexLayer(mixer, ff))
        return VizonexConfig(c["vocab"], c["width"], c["norm"]["eps"], c["canon"]["taps"], c["max_positions"], layers)

    def tensor_shapes(self) -> dict:
        """Checkpoint name -> shape."""
        W, out = self.width, {"embed": (self.vocab, self.width), "pos": (self.max_positions, self.width)}
        for i, l in enumerate(self.layers):
            p = f"l{i}."
            out.update({p + "norm1": (W,), p + "canon1": (W, self.taps), p + "ls1": (W,)})
            out.update({p + "mix." + k: s for k, s in l.mixer.tensor_shapes(W).items()})
            if l.ff is not None:
                out[p + "ls2"] = (W,)
                out.update({p + "mlp." + k: s for k, s in l.ff.tensor_shapes(W).items()})
        out.update({"final.norm": (W,), "head": (self.vocab, W)})
        return out

    def weight_bytes_per_token(self, elem=2):
        """Weight bytes one single-token step streams (output matrix included; of the experts those one token visits)."""
        total = 0
        for name, s in self.tensor_shapes().items():
            if len(s) != 2 or name in ("embed", "pos") or name.endswith((".conv", ".canon1")):
                continue
            share = 1.0
            if ".mlp.e" in name:
                ff = self.layers[int(name[1:name.index(".")])].ff
                share = ff.top / ff.experts
            total += s[0] * s[1] * share
        return int(elem * total)

    def kv_bytes_per_position(self, elem=2):
        """Of the layers that see every position (a chunk bounds what the others read)."""
        return elem * sum(l.mixer.kv_heads * (l.mixer.dim + l.mixer.vdim) for l in self.layers if isinstance(l.mixer, ChunkMixer) and not l.mixer.chunk)

    def state_bytes(self):
        """Recurrent state of one request (read and written by every step)."""
        return 4 * sum(l.mixer.inner * l.mixer.state for l in self.layers if isinstance(l.mixer, DualMixer))


def random_state_dict(cfg: VizonexConfig, seed: int = 0, device="cuda", std: float = 0.02) -> dict:
    """Random-init weights: matrices ~ N(0, std), norm weights, layer scales, score factors and D 1, biases, sinks and corrections 0, step
    offsets -3, A 1."""
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        if len(shape) == 2:
            t = torch.empty(shape, dtype=torch.bfloat16, device=device).normal_(0.0, std, generator=g)
        else:
            t = torch.full(shape, -3.0 if name.endswith(".dt_bias") else 0.0 if name.endswith((".conv.b", ".A_log", ".sink", ".correction")) else 1.0, device=device)
        out[name] = t.to(torch.bfloat16).contiguous()
    return out


@register_model_builder("Vizonex")
class VizonexBuilder(LayerListBuilder):
    def __init__(self, mpk: PersistentKernel, weights: Optional[dict] = None):
        super().__init__(mpk, weights)
        self.k_cache, self.v_cache, self.state, self.tail, self.canon, self.state_slots = {}, {}, {}, {}, {}, None

    @classmethod
    def kernels(cls, dtype, max_num_batched_tokens):
        if dtype == torch.float32:
            return ("DUAL_F32",)
        return ("DUAL_M1",) if max_num_batched_tokens == 1 else ("DUAL",)

    @property
    def max_positions(self):
        """Positions a sequence may take."""
        return self.config.max_positions

    # ------------------------------------------------------------------ entry points
    def build_from_config(self, model_config: MirageModelConfig):
        """`model_config.architecture` is the parsed config.json; caches and states are allocated here."""
        self.config = VizonexConfig.from_dict(model_config.architecture)
        self.build_from_dict(model_config.state_dict, model_config.with_lm_head)

    def build_from_model(self, model_name: str = None, model_path: str = None):
        from .. import checkpoint
        if model_path is None:
            raise ValueError(f"model '{model_name}': a local model_path is required (no hub access); it must hold config.json and *.safetensors")
        cfg, state_dict = checkpoint.load_checkpoint(model_path, device=self.mpk.device, dtype=None, required=("embed", "final.norm"))
        self.config = VizonexConfig.from_dict(cfg)
        self.tokenizer = checkpoint.load_tokenizer(model_path)
        self.build_from_dict(state_dict, True)

    def allocate_caches(self):
        """Keys and values in pages; in state slots the recurrence's state [slots, heads, values, states] and the rings of both
        convolutions (position p in row p % taps)."""
        mpk, R = self.mpk, self.mpk.max_num_batched_requests
        zeros = lambda *shape, dtype=self.dtype: torch.zeros(*shape, dtype=dtype, device=mpk.device)
        for i, l in enumerate(self.config.layers):
            m = l.mixer
            self.canon[i] = zeros(R, self.config.taps, self._W)
            if isinstance(m, DualMixer):
                self.state[i] = zeros(R, m.heads, m.vdim, m.padded_state, dtype=torch.float32)
                self.tail[i] = zeros(R, m.conv, up_to(m.inner, 4) + 2 * m.groups * m.padded_state)
            else:
                dk, dv = flex_cache_dims(m.dim, m.vdim, self.dtype)
                self.k_cache[i] = zeros(mpk.max_num_pages, mpk.page_size, m.kv_heads, dk)
                self.v_cache[i] = zeros(mpk.max_num_pages, mpk.page_size, m.kv_heads, dv)
        self.state_slots = self._new_state_slots()

    # ------------------------------------------------------------------ sub-layers: each returns what the next residual sum takes
    def _attention(self, i: int, p: str, m: ChunkMixer, h):
        mpk, E, H, G = self.mpk, self._E, m.heads, m.kv_heads
        nq, nk, nv = H * m.dim, G * m.dim, G * m.vdim
        w_in, _, cols = self._sections([("q", self._w(p + "q"), nq), ("k", self._w(p + "k"), nk), ("v", self._w(p + "v"), up_to(nq + nk + nv, 16) - nq - nk)])
        qkv = self._linear(h, w_in, p + "qkv", self._rows("mixer_in", cols, E))
        dk, _ = flex_cache_dims(m.dim, m.vdim, self.dtype)
        A = up_to(H * m.vdim, 64)
        out = self._rows(f"attn_out_{H * m.vdim}", A, E)
        mpk.flex_attention_layer(input=qkv, k_cache=self._attach(self.k_cache[i], p + "k_cache"), v_cache=self._attach(self.v_cache[i], p + "v_cache"), cos=None, sin=None,
                                 sink=self._vector(p + "sink", H), q_workspace=self._rows("q_ws", H * dk, E), output=out, num_q_heads=H, num_kv_heads=G, head_dim=m.dim, v_dim=m.vdim,
                                 rot_dims=0, scale=m.scale, eps=self.config.eps, chunk=m.chunk, q_row_weight=self._vector(p + "q.norm", nq), k_row_weight=self._vector(p + "k.norm", nk),
                                 score_factors=self._vector(p + "temp", H))
        return self._linear(out, self._matrix(p + "o", cols=A), p + "o", self._y)

    def _recurrence(self, i: int, p: str, m: DualMixer, h):
        mpk, E, I, H, G, N, Np = self.mpk, self._E, m.inner, m.heads, m.groups, m.state, m.padded_state
        Ip, GN = up_to(I, 4), G * Np
        by_group = lambda w: torch.nn.functional.pad(w.reshape(G, N, -1), (0, 0, 0, Np - N)).reshape(GN, -1)  # a group's rows padded to whole quads
        w = self._w(p + "in")
        z, x, B, C, dt = w.split([I, I, G * N, G * N, H])
        at = 2 * Ip + 2 * GN
        w_in, col, cols = self._sections([("z", z, Ip), ("x", x, Ip), ("B", by_group(B), GN), ("C", by_group(C), GN), ("dt", dt, up_to(at + H, 16) - at)])
        rows = self._linear(h, w_in, p + "in", self._rows("mixer_in", cols, E))
        n, c = Ip + 2 * GN, torch.cat([self._w(p + "conv"), self._w(p + "conv.b")[:, None]], dim=1)  # (the bias travels as one more tap)
        taps = torch.zeros(m.conv + 1, n, dtype=c.dtype, device=c.device)
        for lo, part in ((0, c[:I]), (Ip, by_group(c[I:I + G * N])), (Ip + GN, by_group(c[I + G * N:]))):
            taps[:, lo:lo + len(part)] = part.T
        conv, steps = self._rows(f"convolved_{I}_{G}x{N}", n, E), self._rows(f"steps_{H}", 2 * up_to(H, 4), float32)
        rates = (-torch.exp(self._w(p + "A_log").to(torch.float64)) / math.log(2.0)).to(torch.float32)
        mpk.ring_conv_layer(rows, self._attach(taps[:-1].to(self.dtype), p + "conv"), self._attach(self.tail[i], p + "tail"), self._slots, conv, bias=self._attach(taps[-1].to(torch.float32), p + "conv.b"),
                            column=col["x"], silu=True, heads=H, step_column=col["dt"], decay_column=up_to(H, 4), step_bias=self._vector(p + "dt_bias", H), rates=self._attach(rates, p + "A"),
                            steps=steps)
        A = up_to(I, 64)
        gated, out = self._rows(f"scan_out_{I}", A, float32), self._rows(f"scan_normed_{I}", A, E)
        mpk.dual_scan_layer(rows, conv, steps, self._vector(p + "D", H), self._attach(self.state[i], p + "state"), self._slots, gated, H, m.vdim, N, G, z_column=col["z"], x_column=0, b_column=Ip,
                            c_column=Ip + GN, decay_column=up_to(H, 4))
        mpk.residual_prenorm_layer(input=None, residual=gated, new_residual=None, output=out, weight=self._vector(p + "norm", A), width=I, groups=m.norm_groups, eps=self.config.eps)
        return self._linear(out, self._matrix(p + "o", cols=A), p + "o", self._y)

    def _dense(self, i: int, p: str, f: DenseFF, h):
        F, W = up_to(f.ff, 64), self._W
        w_gu = self.mpk.shuffle_tensors(inputs=[self._attach(self._matrix(p + n, F, W), p + n) for n in ("gate", "up")], shuffled_dim=0, num_groups=1, name=p + "gate_up")
        gate_up, act = self._rows("gate_up", 2 * F, self._E), self._rows("ff_act", F, self._E)  # (gate_up is never written: the activation is the linear's epilogue)
        self.mpk.linear_layer(input=h, weight=w_gu, output=gate_up, grid_dim=(1, 1, 1), block_dim=(256, 1, 1))
        self.mpk.gelu_mul_layer(input=gate_up, output=act)
        return dict(input2=self._linear(act, self._matrix(p + "down", cols=F), p + "down", self._y2))

    def _experts(self, i: int, p: str, f: ExpertFF, h):
        mpk, W = self.mpk, self._W
        z = self._rows("router_logits", up_to(f.experts, 4), float32)
        mpk.head_linear_layer(input=h, weight=self._attach(operand_tiles(self._matrix(p + "router", cols=W)[None]), p + "router"), output=z, heads=1, n=f.experts, k=W, in_stride=0, out_stride=0)
        ids, shares = self._rows(f"expert_ids_{i}", f.top, int32), self._rows(f"expert_shares_{i}", up_to(f.top + 1, 4), float32)
        mpk.expert_route_layer(z, ids, shares, f.experts, f.top, f.shared_ff is not None, correction=self._vector(p + "correction", f.experts), groups=f.groups, groups_kept=f.keep, scale=f.scale)
        y, places = self._expert_linears(p, h, ids, f.experts, f.top, f.ff, f.shared_ff, clamp=(f.limit, GLU_BETA, GLU_BIAS, f.shared_limit))
        return dict(input2=y, slot_weights=shares, slots=places, slot_columns=W)

    # ------------------------------------------------------------------ graph
    def build_from_dict(self, state_dict: dict, with_lm_head: bool = True):
        mpk, c = self.mpk, self.config
        self._begin(c, state_dict, with_lm_head)
        if mpk.spec_decode_config is not None:
            raise NotImplementedError("speculative decoding: rows of rejected guesses cannot be taken back out of a recurrent state")
        if mpk.mode != "online_notoken" and mpk.max_seq_length - 1 > c.max_positions:  # (a host that describes its batches keeps to max_positions itself)
            raise ValueError(f"max_seq_length={mpk.max_seq_length}: the model has vectors for {c.max_positions} positions")
        f32, E, W = self.dtype == torch.float32, self._E, self._W
        self.allocate_caches()
        self._slots = self._attach(self.state_slots, "state_slots")
        # the residual rows alternate between two buffers: a single-token iteration forms the new rows in every workgroup of
        # the linear that reads them, from the old ones
        streams = [self._rows("residual_a", W, float32), self._rows("residual_b", W, float32)]
        which = 0
        h, x16 = self._rows("normed", W, E), self._rows("stream", W, E)
        mixed = self._rows("normed_convolved", W, E)
        self._y, self._y2 = self._rows("mixer_out", W, E), self._rows("ff_out", W, E)

        def join(weight, **summands):
            nonlocal which
            old, which = streams[which], 1 - which
            mpk.residual_prenorm_layer(**{"input": None, **summands}, residual=old, weight=weight, new_residual=streams[which], output=h, width=c.width, eps=c.eps)

        ids, _, _ = self._token_ids(with_lm_head)
        mpk.embed_scaled_layer(input=ids, weight=self._attach(self._matrix("embed", cols=W), "embed"), residual=streams[which], output=streams[which] if f32 else x16,
                               positions=self._attach(self._matrix("pos", cols=W), "pos"))
        summands = {}
        for i, l in enumerate(c.layers):
            p = f"l{i}."
            join(self._vector(p + "norm1", W), **summands)
            taps = self._pad(self._matrix(p + "canon1").T, cols=W)
            mpk.ring_conv_layer(h, self._attach(taps, p + "canon1"), self._attach(self.canon[i], p + "canon"), self._slots, mixed, identity=True)
            mixer = self._attention if isinstance(l.mixer, ChunkMixer) else self._recurrence
            summands = dict(input=mixer(i, p + "mix.", l.mixer, mixed), factor=self._vector(p + "ls1", W))
            if l.ff is not None:
                ff = self._dense if isinstance(l.ff, DenseFF) else self._experts
                summands.update(ff(i, p + "mlp.", l.ff, h), factor2=self._vector(p + "ls2", W))
        join(self._vector("final.norm", W), **summands)
        self.hidden = h
        if with_lm_head:
            self._head_and_sampling(h, self._attach(self._matrix("head", cols=W), "head"), c.vocab)
        self._state = None
