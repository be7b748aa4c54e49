"""Dodonex graph builder: a parallel-sublayer decoder whose mixers are latent attention or a generalised delta rule.

A layer keeps a 32-bit residual stream x, normalises it once (RMS norm in equal parts) and feeds both sub-layers from that;
afterwards a per-token vector of the layer's own enters through a gate:

    h = N(x);  x <- x + m (mixer(h) + glu(h));   g = gelu(A x) * e_layer[token];  x <- x + m rms_norm(B g)

What a layer records:

    residual_prenorm (the previous layer's B g, normalised, joins the stream) -> linear: everything that reads h, one matrix
    latent attention: latent_prep (+ the gated activation) -> linear (queries) -> head_linear (into the latent space)
                      -> latent_attention -> head_linear (out of it)
    delta rule:       general_delta (+ the gated activation)
    -> linear: mixer output and feed-forward output, one matrix over both inputs side by side
    -> residual_prenorm (sum only) -> head_linear (A, gelu, e) -> linear (B)

Layers with `kv_from` read the latent rows another layer has cached.  Sizes need no alignment: sections of fused matrices and
heads are padded with zero rows or columns.  Checkpoint names: `embed` (also the output matrix), `side.embed`, `l<i>.norm1`,
`l<i>.mix.{dq,dq.norm,uq,dkv,dkv.norm,uk,uv,o}` or `l<i>.mix.{r,k,v,g,a,a.b,w1,w2,w0,norm,o}`, `l<i>.mlp.{gate,up,down}`,
`l<i>.side.{gate,proj,norm}`, `final.norm`; linear weights are [out, in].

Runs in bfloat16 (the served form) and float32 (everything in true 32-bit).
"""
from dataclasses import dataclass
from typing import List, Optional

import torch

from ...model_registry import register_model_builder
from ...persistent_kernel import PersistentKernel, latent_row_dim, operand_row, operand_tiles
from ....kernel import bfloat16, float32, int64
from ..graph_builder import GraphBuilder, MirageModelConfig

def _up(n: int, m: int) -> int:
    return -(-n // m) * m


GLU_BETA, GLU_BIAS = 1.702, 1.0  # feed-forward: g sigmoid(1.702 g) (u + 1)


@dataclass
class LatentMixer:
    heads: int
    dim: int
    rot_dim: int
    vdim: int
    q_rank: int
    kv_rank: int
    rot_base: float
    scale: float
    kv_from: Optional[int]

    @property
    def out_cols(self):
        return self.heads * self.vdim

    def tensor_shapes(self, W):
        H = self.heads
        out = {"dq": (self.q_rank, W), "dq.norm": (self.q_rank,), "uq": (H * (self.dim + self.rot_dim), self.q_rank)}
        if self.kv_from is None:
            out.update({"dkv": (self.kv_rank + self.rot_dim, W), "dkv.norm": (self.kv_rank,)})
        out.update({"uk": (H * self.dim, self.kv_rank), "uv": (H * self.vdim, self.kv_rank), "o": (W, H * self.vdim)})
        return out


@dataclass
class DeltaMixer:
    heads: int
    dim: int
    low_rank: Optional[int]  # None until the weights are seen: the shape of w1 gives it

    @property
    def padded_dim(self):
        return _up(self.dim, 16)

    @property
    def out_cols(self):
        return self.heads * self.padded_dim

    def tensor_shapes(self, W):
        n = self.heads * self.dim
        out = {x: (n, W) for x in "rkvga"}
        out.update({"a.b": (n,), "w1": (self.low_rank, W), "w2": (n, self.low_rank), "w0": (n,), "norm": (n,), "o": (W, n)})
        return out


@dataclass
class DodonexLayer:
    mixer: object
    ff: Optional[int]  # None: the layer has no feed-forward
    limit: float


@dataclass
class DodonexConfig:
    vocab: int
    width: int
    eps: float
    groups: int
    residual_mult: float
    embedding_scale: float
    logit_scale: float
    side_dim: int
    layers: List[DodonexLayer]

    @staticmethod
    def from_dict(c: dict) -> "DodonexConfig":
        """The rank of a decay projection is the shape of its weights; `low_rank` in a mixer gives it where there are none yet."""
        layers = []
        for i, e in enumerate(c["layers"]):
            m, mlp = e["mixer"], e.get("mlp")
            if e["type"] == "latent_attention":
                if m["rot"]["dims"] != m["rot_dim"]:
                    raise ValueError(f"layer {i}: rotation over {m['rot']['dims']} of a rotated part of {m['rot_dim']}")
                mixer = LatentMixer(m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["q_rank"], m["kv_rank"], m["rot"]["base"], m["scale"], m.get("kv_from"))
                if mixer.kv_from is not None:
                    src = layers[mixer.kv_from].mixer if 0 <= mixer.kv_from < i else None
                    if not isinstance(src, LatentMixer) or src.kv_from is not None or (src.kv_rank, src.rot_dim, src.rot_base) != (mixer.kv_rank, mixer.rot_dim, mixer.rot_base):
                        raise ValueError(f"layer {i}: kv_from={mixer.kv_from} names no earlier layer with a latent of the same form")
            elif e["type"] == "general_delta":
                mixer = DeltaMixer(m["heads"], m["dim"], m.get("low_rank"))
            else:
                raise ValueError(f"layer {i}: unknown mixer type {e['type']!r}")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            layers.append(DodonexLayer(mixer, None if mlp is None else mlp["ff"], 0.0 if mlp is None else mlp["limit"]))
        if c["width"] % c["norm"]["groups"]:
            raise ValueError(f"width {c['width']} is not divided by {c['norm']['groups']} norm groups")
        return DodonexConfig(c["vocab"], c["width"], c["norm"]["eps"], c["norm"]["groups"], c["residual_mult"], c["embedding"]["scale"], c["logit_scale"],
                             c["token_side"]["dim"], layers)

    def read_low_ranks(self, state_dict: dict):
        for i, l in enumerate(self.layers):
            if isinstance(l.mixer, DeltaMixer) and l.mixer.low_rank is None:
                name = f"l{i}.mix.w1"
                if name not in state_dict:
                    raise KeyError(f"the state dict lacks ['{name}']")
                l.mixer.low_rank = state_dict[name].shape[0]

    def tensor_shapes(self) -> dict:
        """Checkpoint name -> shape."""
        W, n = self.width, self.side_dim
        out = {"embed": (self.vocab, W), "side.embed": (self.vocab, len(self.layers) * n)}
        for i, l in enumerate(self.layers):
            p = f"l{i}."
            out[p + "norm1"] = (W,)
            out.update({p + "mix." + k: s for k, s in l.mixer.tensor_shapes(W).items()})
            if l.ff is not None:
                out.update({p + "mlp.gate": (l.ff, W), p + "mlp.up": (l.ff, W), p + "mlp.down": (W, l.ff)})
            out.update({p + "side.gate": (n, W), p + "side.proj": (W, n), p + "side.norm": (W,)})
        out["final.norm"] = (W,)
        return out

    def weight_bytes_per_token(self, elem=2):
        """Weight bytes one decode step streams (output matrix included)."""
        return elem * sum(s[0] * s[1] for name, s in self.tensor_shapes().items() if len(s) == 2 and name != "side.embed")

    def kv_bytes_per_position(self, elem=2):
        return elem * sum(l.mixer.kv_rank + l.mixer.rot_dim for l in self.layers if isinstance(l.mixer, LatentMixer))

    def state_bytes(self):
        """Recurrent state of one request (read and written by every step)."""
        return 4 * sum(l.mixer.heads * l.mixer.dim ** 2 for l in self.layers if isinstance(l.mixer, DeltaMixer))


def random_state_dict(cfg: DodonexConfig, seed: int = 0, device="cuda", std: float = 0.02) -> dict:
    """Random-init weights: matrices ~ N(0, std), norm weights 1, offsets 0."""
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        if len(shape) == 2:
            out[name] = torch.empty(shape, dtype=torch.bfloat16, device=device).normal_(0.0, std, generator=g)
        else:
            out[name] = torch.full(shape, 0.0 if name.endswith((".w0", ".a.b")) else 1.0, dtype=torch.bfloat16, device=device)
    return out


@register_model_builder("Dodonex")
class DodonexBuilder(GraphBuilder):
    owns_kv_cache = True
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, mpk: PersistentKernel, weights: Optional[dict] = None):
        super().__init__(mpk, weights)
        self.tokenizer = None
        self.returned_hidden_state = None
        self.logits = None
        self.latent_cache, self.state, self.state_slots = {}, {}, None
        self._keep, self._tables, self._attached = {}, {}, {}

    @classmethod
    def kernels(cls, dtype, max_num_batched_tokens):
        if dtype == torch.float32:
            return ("MIX_F32",)
        return ("MIX_M1",) if max_num_batched_tokens == 1 else ("MIX",)

    # ------------------------------------------------------------------ entry points
    def build_from_config(self, model_config: MirageModelConfig):
        """`model_config.architecture` is the parsed config.json; caches and states are allocated here."""
        self.config = DodonexConfig.from_dict(model_config.architecture)
        self.build_from_dict(model_config.state_dict, model_config.with_lm_head)

    def build_from_model(self, model_name: str = None, model_path: str = None):
        from .. import checkpoint
        if model_path is None:
            raise ValueError(f"model '{model_name}': a local model_path is required (no hub access); it must hold config.json and *.safetensors")
        cfg, state_dict = checkpoint.load_checkpoint(model_path, device=self.mpk.device, dtype=None, required=("embed", "side.embed", "final.norm"))
        self.config = DodonexConfig.from_dict(cfg)
        self.tokenizer = checkpoint.load_tokenizer(model_path)
        self.build_from_dict(state_dict, True)

    # ------------------------------------------------------------------ tensors
    def _attach(self, t: torch.Tensor, name: str):
        t = t.contiguous()
        self._keep[name] = t
        return self.mpk.attach_input(torch_tensor=t, name=name)

    def release_weights(self, names):
        return sum(self._keep.pop(n, None) is not None for n in names)

    def _w(self, name: str) -> torch.Tensor:
        w = self._state[name]
        if tuple(w.shape) != self._shapes[name]:
            raise ValueError(f"{name} has shape {tuple(w.shape)}, expected {self._shapes[name]}")
        return w

    def _matrix(self, name: str, rows: int = None, cols: int = None):
        w = self._w(name).to(self.dtype)
        rows, cols = rows or w.shape[0], cols or w.shape[1]
        if (rows, cols) != tuple(w.shape):
            w = torch.nn.functional.pad(w, (0, cols - w.shape[1], 0, rows - w.shape[0]))
        return w

    def _head_vector(self, name: str, m: DeltaMixer):
        """Attach a per-channel vector in fp32, every head zero-padded to a multiple of 16."""
        v = self._w(name).to(torch.float32).view(m.heads, m.dim)
        return self._attach(torch.nn.functional.pad(v, (0, m.padded_dim - m.dim)).reshape(-1), name)

    def _vector(self, name: str, size: int = None, factor: float = 1.0):
        """Attach a norm weight or an offset in fp32, zero-padded to `size`."""
        v = self._w(name).to(torch.float32) * factor
        return self._attach(torch.nn.functional.pad(v, (0, (size or len(v)) - len(v))), name)

    def _rows(self, name: str, cols: int, dt):
        """Activation rows of one iteration (library-owned, zero-filled), one tensor per name and size."""
        key = f"{name}_{cols}"
        if key not in self._acts:
            self._acts[key] = self.mpk.new_tensor(dims=(self.mpk.max_num_batched_tokens, cols), dtype=dt, name=key, io_category="cuda_tensor")
        return self._acts[key]

    def _rotary(self, m: LatentMixer):
        from .. import checkpoint
        if m.rot_dim == 0:
            return None, None
        key = (m.rot_dim, m.rot_base)
        if key not in self._tables:
            cos, sin = checkpoint.rotary_tables_f32(m.rot_dim, m.rot_base, None, self.mpk.max_seq_length, self.mpk.device)
            n = len(self._tables)
            self._tables[key] = (self._attach(cos, f"cos_{n}"), self._attach(sin, f"sin_{n}"))
        return self._tables[key]

    def _cache(self, i: int):
        """The latent rows layer `i` owns, attached once for every layer that reads them."""
        if i not in self._attached:
            self._attached[i] = self._attach(self.latent_cache[i], f"l{i}.latent_cache")
        return self._attached[i]

    def allocate_caches(self):
        """Latent rows [pages, page_size, row] of the layers that own some, states [slots, heads, dim, dim] (both rounded up)."""
        mpk = self.mpk
        for i, l in enumerate(self.config.layers):
            m = l.mixer
            if isinstance(m, DeltaMixer):
                d = m.padded_dim
                self.state[i] = torch.zeros(mpk.max_num_batched_requests, m.heads, d, d, dtype=torch.float32, device=mpk.device)
            elif m.kv_from is None:
                self.latent_cache[i] = torch.zeros(mpk.max_num_pages, mpk.page_size, latent_row_dim(m.kv_rank, m.rot_dim, self.dtype), dtype=self.dtype, device=mpk.device)
        if self.state:
            self.state_slots = mpk.meta_tensors.get("state_slots_buffer")
            if self.state_slots is None:
                self.state_slots = torch.arange(mpk.max_num_batched_requests, dtype=torch.int32, device=mpk.device)

    # ------------------------------------------------------------------ graph
    def build_from_dict(self, state_dict: dict, with_lm_head: bool = True):
        mpk, c = self.mpk, self.config
        c.read_low_ranks(state_dict)
        self._shapes = c.tensor_shapes()
        missing = sorted(set(self._shapes) - set(state_dict))
        if missing:
            raise KeyError(f"the state dict lacks {missing}")
        if mpk.spec_decode_config is not None and any(isinstance(l.mixer, DeltaMixer) for l in c.layers):
            raise NotImplementedError("speculative decoding: rows of rejected guesses cannot be taken back out of a recurrent state")
        self._state, self._acts, self.with_lm_head = state_dict, {}, with_lm_head
        f32 = self.dtype == torch.float32
        E, KW = float32 if f32 else bfloat16, operand_row(self.dtype)
        self.allocate_caches()
        slots = self._attach(self.state_slots, "state_slots") if self.state else None
        W = _up(c.width, 64)
        one = dict(grid_dim=(1, 1, 1), block_dim=(256, 1, 1))
        # the residual rows alternate between two buffers: a single-token iteration forms the new rows in every workgroup of
        # the linear that reads them, from the old ones
        streams = [self._rows("residual_a", W, float32), self._rows("residual_b", W, float32)]
        which = 0
        h, x16, y = self._rows("normed", W, E), self._rows("stream", W, E), self._rows("sublayers_out", W, E)

        def join(inp, inp_weight, weight, out):
            nonlocal which
            old, which = streams[which], 1 - which
            mpk.residual_prenorm_layer(input=inp, input_weight=inp_weight, residual=old, weight=weight, new_residual=streams[which], output=out or streams[which],
                                       width=c.width, groups=c.groups, alpha=c.residual_mult, eps=c.eps, input_eps=c.eps)

        ids = self._attach(mpk.meta_tensors["input_tokens"], "input_token")
        spec, spec_tokens = mpk.spec_decode_config, None
        if spec is not None:
            all_tokens = self._attach(mpk.meta_tensors["tokens"], "all_tokens")
            spec_tokens = mpk.draft_forward_layer_dispatcher(spec_decode_config=spec, tokens=all_tokens, grid_dim=(96, 1, 1), block_dim=(128, 1, 1))
            ids = spec_tokens
        embed = self._attach(self._matrix("embed", cols=W), "embed")
        side_table = self._attach(self._matrix("side.embed"), "side.embed")
        mpk.embed_scaled_layer(input=ids, weight=embed, residual=streams[which], output=streams[which] if f32 else x16, scale=c.embedding_scale)
        side_in, side_norm = None, None
        for i, l in enumerate(c.layers):
            p, m = f"l{i}.", l.mixer
            latent = isinstance(m, LatentMixer)
            join(side_in, side_norm, self._vector(p + "norm1", W), h)
            # ---- everything that reads h: sections of one matrix
            F = 0 if l.ff is None else _up(l.ff, 64)
            sections = []
            if latent:
                sections.append(("dq", self._w(p + "mix.dq"), _up(m.q_rank, 16)))
                if m.kv_from is None:
                    dkv = self._w(p + "mix.dkv")
                    sections += [("c", dkv[:m.kv_rank], _up(m.kv_rank, 16)), ("rot", dkv[m.kv_rank:], _up(m.rot_dim, 16))]
            else:
                by_head = lambda w: torch.nn.functional.pad(w.view(m.heads, m.dim, -1), (0, 0, 0, m.padded_dim - m.dim)).reshape(m.out_cols, -1)
                sections += [(n, by_head(self._w(p + "mix." + n)), m.out_cols) for n in "rkvga"]
                sections.append(("w1", self._w(p + "mix.w1"), _up(m.low_rank, KW)))
            if F:
                sections += [(n, self._w(p + "mlp." + n), F) for n in ("gate", "up")]
            col, at = {}, 0
            for n, _, size in sections:
                col[n], at = at, at + size
            w_in = torch.zeros(at, W, dtype=self.dtype, device=self._w(p + "norm1").device)
            for n, w, _ in sections:
                w_in[col[n]:col[n] + w.shape[0], :c.width] = w.to(self.dtype)
            rows = self._rows("sublayers_in", at, E)
            mpk.linear_layer(input=h, weight=self._attach(w_in, p + "in"), output=rows, **one)
            # ---- mixer, with the feed-forward's activation beside it; both outputs side by side
            A = _up(m.out_cols, 64)
            both = self._rows(f"both_{m.out_cols}_{l.ff}", A + F, E)
            glu = None if not F else (both, A, F, col["gate"], col["up"], l.limit, GLU_BETA, GLU_BIAS)
            if latent:
                cq_cols, dp, rp, Rp = _up(m.q_rank, 64), _up(m.dim, KW), _up(m.rot_dim, 16), _up(m.kv_rank, KW)
                cq = self._rows(f"q_latent_{m.q_rank}", cq_cols, E)
                cos, sin = self._rotary(m)
                own = {}
                if m.kv_from is None:
                    own = dict(cache=self._cache(i), latent_weight=self._vector(p + "mix.dkv.norm", _up(m.kv_rank, 4)), cos=cos, sin=sin, latent_column=col["c"],
                               latent_rank=m.kv_rank, rot_column=col["rot"], rot_dims=m.rot_dim)
                mpk.latent_prep_layer(input=rows, q_weight=self._vector(p + "mix.dq.norm", _up(m.q_rank, 4)), output=cq, q_column=col["dq"], q_rank=m.q_rank, eps=c.eps,
                                      glu=glu, **own)
                hs = dp + rp  # a head's query columns: unrotated part, rotated part, each padded
                uq = torch.zeros(m.heads, hs, cq_cols, dtype=self.dtype, device=w_in.device)
                w = self._w(p + "mix.uq").to(self.dtype).view(m.heads, m.dim + m.rot_dim, m.q_rank)
                uq[:, :m.dim, :m.q_rank] = w[:, :m.dim]
                uq[:, dp:dp + m.rot_dim, :m.q_rank] = w[:, m.dim:]
                q = self._rows("queries", m.heads * hs, E)
                mpk.linear_layer(input=cq, weight=self._attach(uq.view(m.heads * hs, cq_cols), p + "mix.uq"), output=q, **one)
                uk = torch.zeros(m.heads, Rp, dp, dtype=self.dtype, device=w_in.device)
                uk[:, :m.kv_rank, :m.dim] = self._w(p + "mix.uk").to(self.dtype).view(m.heads, m.dim, m.kv_rank).transpose(1, 2)
                ql, ol = self._rows("queries_in_latent", m.heads * Rp, E), self._rows("latent_sums", m.heads * Rp, E)
                mpk.head_linear_layer(input=q, weight=self._attach(operand_tiles(uk), p + "mix.uk"), output=ql, heads=m.heads, n=Rp, k=dp, in_stride=hs, out_stride=Rp)
                mpk.latent_attention_layer(input=q, q_latent=ql, cache=self._cache(i if m.kv_from is None else m.kv_from), cos=cos, sin=sin, output=ol, num_heads=m.heads,
                                           latent_rank=m.kv_rank, rot_dims=m.rot_dim, head_stride=hs, rot_column=dp, scale=m.scale)
                uv = operand_tiles(self._w(p + "mix.uv").to(self.dtype).view(m.heads, m.vdim, m.kv_rank))
                mpk.head_linear_layer(input=ol, weight=self._attach(uv, p + "mix.uv"), output=both, heads=m.heads, n=m.vdim, k=Rp, in_stride=Rp, out_stride=m.vdim)
            else:
                w2 = operand_tiles(by_head(self._w(p + "mix.w2").to(self.dtype))[None])
                mpk.general_delta_layer(input=rows, decay_weight=self._attach(w2, p + "mix.w2"), decay_offset=self._head_vector(p + "mix.w0", m),
                                        removal_offset=self._head_vector(p + "mix.a.b", m), norm_weight=self._head_vector(p + "mix.norm", m),
                                        state=self._attach(self.state[i], p + "state"), state_slots=slots, workspace=self._rows("delta_work", 2 * m.out_cols, float32),
                                        output=both, heads=m.heads, dim=m.dim, low_rank=_up(m.low_rank, KW),
                                        columns=tuple(col[n] for n in ("r", "k", "v", "g", "a", "w1")), eps=c.eps, glu=glu)
            w_out = self._matrix(p + "mix.o")
            if not latent:
                w_out = by_head(w_out.T).T
            w_out = torch.nn.functional.pad(w_out, (0, A - w_out.shape[1]))
            if F:
                w_out = torch.cat([w_out, self._matrix(p + "mlp.down", cols=F)], dim=1)
            mpk.linear_layer(input=both, weight=self._attach(w_out, p + "out"), output=y, **one)
            # ---- the token's own vector
            join(y, None, None, None if f32 else x16)
            n = c.side_dim
            side = self._rows(f"side_{n}", _up(n, 64), E)
            gate = operand_tiles(self._matrix(p + "side.gate", cols=W)[None])
            mpk.head_linear_layer(input=streams[which] if f32 else x16, weight=self._attach(gate, p + "side.gate"), output=side, heads=1, n=n, k=W, in_stride=0,
                                  out_stride=0, ids=ids, table=side_table, table_column=i * n)
            side_in, side_norm = self._rows("side_out", W, E), self._vector(p + "side.norm", W)
            mpk.linear_layer(input=side, weight=self._attach(self._matrix(p + "side.proj", cols=_up(n, 64)), p + "side.proj"), output=side_in, **one)
        # (the logit scale rides on the last norm's weight)
        join(side_in, side_norm, self._vector("final.norm", W, factor=c.logit_scale), h)
        self.hidden = h
        if not with_lm_head:
            if spec_tokens is not None:
                raise ValueError("speculative decoding needs the LM head and the sampling stages in the graph (with_lm_head)")
            self._state = None
            return
        self.logits = self._rows("logits", c.vocab, E)
        mpk.linear_layer(input=h, weight=embed, output=self.logits, **one)
        out = self._attach(mpk.meta_tensors["output_tokens"], "output_token")
        part = (self._rows("argmax_value", mpk.num_workers, E), self._rows("argmax_index", mpk.num_workers, int64))
        mpk.argmax_partial_layer(input=self.logits, output=part, grid_dim=(mpk.num_workers, 1, 1), block_dim=(128, 1, 1))
        mpk.argmax_reduce_layer(input=part, output=out, grid_dim=(1, 1, 1), block_dim=(128, 1, 1))
        if spec_tokens is not None:
            self.verify_out = mpk.verify_layer_dispatcher(spec_decode_config=spec, spec_tokens=spec_tokens, target_output=out)
        self._state = None

    def decode(self, ids: torch.Tensor):
        return self.tokenizer.decode(ids, skip_special_tokens=True)
