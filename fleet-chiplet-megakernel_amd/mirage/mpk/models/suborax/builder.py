"""Suborax graph builder: a post-norm decoder with partly rotated, unit-norm, softcapped attention and per-head sinks.

A layer keeps a 32-bit residual stream x and normalises BEHIND each sum (N = RMS norm with weight 1 + w):

    x <- N1(alpha x + attention(x));   x <- N2(alpha x + swiglu(x))          (the second only where the layer has an mlp)

so one recorded layer is: linear (q, k, v) -> flex_attention -> linear (o) -> residual_rmsnorm -> linear + silu_mul
(gate / up) -> linear (down) -> residual_rmsnorm.  Single-token iterations fold each residual_rmsnorm into the linear that
reads it.  Everything is described by the parsed config.json: every layer has its own head counts, head sizes, rotation,
scale, cap and feed-forward width.

Sizes need no alignment: the builder pads rows to 64 entries (zero columns in the weights, zero entries in the activation
rows), which is what the matrix-core linears want.  Checkpoint names: `embed`, `l<i>.norm1`, `l<i>.norm2`, `l<i>.mix.{q,k,v,o,
sink}`, `l<i>.mlp.{gate,up,down}`, `final.norm`, `head`; linear weights are [out, in].

Runs in bfloat16 (the served form) and float32 (everything in true 32-bit).
"""
from dataclasses import dataclass
from typing import List, Optional

import torch

from ...model_registry import register_model_builder
from ...persistent_kernel import PersistentKernel, flex_cache_dims
from ....kernel import bfloat16, float32, int64
from ..graph_builder import GraphBuilder, MirageModelConfig


@dataclass
class SuboraxLayer:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    rot_dims: int
    rot_base: float
    rot_scaling: Optional[dict]
    scale: float
    softcap: float
    ff: Optional[int]  # None: the layer has no feed-forward

    @property
    def qkv_cols(self):
        return self.heads * self.dim + self.kv_heads * (self.dim + self.vdim)


@dataclass
class SuboraxConfig:
    vocab: int
    width: int
    eps: float
    alpha: float
    embedding_scale: float
    layers: List[SuboraxLayer]

    @staticmethod
    def from_dict(c: dict) -> "SuboraxConfig":
        layers = []
        for i, e in enumerate(c["layers"]):
            if e["type"] != "attention":
                raise ValueError(f"layer {i}: unknown mixer type {e['type']!r}")
            m, mlp = e["mixer"], e.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"layer {i}: unknown feed-forward kind {mlp['kind']!r}")
            rot = m.get("rot") or {"dims": 0, "base": 1.0}
            if m["heads"] % m["kv_heads"]:
                raise ValueError(f"layer {i}: {m['heads']} query heads over {m['kv_heads']} key/value heads")
            layers.append(SuboraxLayer(m["heads"], m["kv_heads"], m["dim"], m["vdim"], rot["dims"], rot["base"], rot.get("scaling"), m["scale"],
                                       m.get("softcap") or 0.0, None if mlp is None else mlp["ff"]))
        return SuboraxConfig(c["vocab"], c["width"], c["norm"]["eps"], c["postln_alpha"], c.get("embedding", {}).get("scale", 1.0), layers)

    def tensor_shapes(self) -> dict:
        """Checkpoint name -> shape."""
        W, out = self.width, {"embed": (self.vocab, self.width)}
        for i, l in enumerate(self.layers):
            out.update({f"l{i}.norm1": (W,), f"l{i}.mix.q": (l.heads * l.dim, W), f"l{i}.mix.k": (l.kv_heads * l.dim, W), f"l{i}.mix.v": (l.kv_heads * l.vdim, W),
                        f"l{i}.mix.sink": (l.heads,), f"l{i}.mix.o": (W, l.heads * l.vdim)})
            if l.ff is not None:
                out.update({f"l{i}.norm2": (W,), f"l{i}.mlp.gate": (l.ff, W), f"l{i}.mlp.up": (l.ff, W), f"l{i}.mlp.down": (W, l.ff)})
        out.update({"final.norm": (W,), "head": (self.vocab, W)})
        return out

    def weight_bytes_per_token(self, elem=2):
        """Linear weight bytes one decode step streams (LM head included)."""
        shapes = self.tensor_shapes()
        return elem * sum(s[0] * s[1] for n, s in shapes.items() if len(s) == 2 and n != "embed")

    def kv_bytes_per_position(self, elem=2):
        return elem * sum(l.kv_heads * (l.dim + l.vdim) for l in self.layers)


def random_state_dict(cfg: SuboraxConfig, seed: int = 0, device="cuda", std: float = 0.02) -> dict:
    """Random-init weights: linears and embedding ~ N(0, std), norm weights 0 (a factor of one), sinks 0."""
    g = torch.Generator(device=device).manual_seed(seed)
    out = {}
    for name, shape in cfg.tensor_shapes().items():
        if len(shape) == 2:
            out[name] = torch.empty(shape, dtype=torch.bfloat16, device=device).normal_(0.0, std, generator=g)
        else:
            out[name] = torch.zeros(shape, dtype=torch.bfloat16, device=device)
    return out


def _pad64(n: int) -> int:
    return -(-n // 64) * 64


@register_model_builder("Suborax")
class SuboraxBuilder(GraphBuilder):
    owns_kv_cache = True
    dtypes = (torch.bfloat16, torch.float32)

    def __init__(self, mpk: PersistentKernel, weights: Optional[dict] = None):
        super().__init__(mpk, weights)
        self.tokenizer = None
        self.returned_hidden_state = None
        self.logits = None
        self._keep = {}   # name -> torch tensor the graph points at
        self._tables = {}

    @classmethod
    def kernels(cls, dtype, max_num_batched_tokens):
        if dtype == torch.float32:
            return ("FLEX_F32",)
        return ("FLEX_M1",) if max_num_batched_tokens == 1 else ("FLEX",)

    # ------------------------------------------------------------------ entry points
    def build_from_config(self, model_config: MirageModelConfig):
        """`model_config.architecture` is the parsed config.json; caches are the caller's when given, else allocated here."""
        self.config = SuboraxConfig.from_dict(model_config.architecture)
        self.k_cache, self.v_cache = model_config.k_cache, model_config.v_cache
        self.build_from_dict(model_config.state_dict, model_config.with_lm_head)

    def build_from_model(self, model_name: str = None, model_path: str = None):
        from .. import checkpoint
        if model_path is None:
            raise ValueError(f"model '{model_name}': a local model_path is required (no hub access); it must hold config.json and *.safetensors")
        cfg, state_dict = checkpoint.load_checkpoint(model_path, device=self.mpk.device, dtype=None, required=("embed", "final.norm", "head"))
        self.config = SuboraxConfig.from_dict(cfg)
        self.k_cache = self.v_cache = None
        self.tokenizer = checkpoint.load_tokenizer(model_path)
        self.build_from_dict(state_dict, True)

    # ------------------------------------------------------------------ tensors
    def _attach(self, t: torch.Tensor, name: str):
        t = t.contiguous()
        self._keep[name] = t
        return self.mpk.attach_input(torch_tensor=t, name=name)

    def release_weights(self, names):
        return sum(self._keep.pop(n, None) is not None for n in names)

    def _linear_weight(self, name: str, rows: int = None, cols: int = None):
        """Attach a [out, in] weight in the build's type, zero-padded to `rows` x `cols`."""
        w = self._state[name]
        want = self.config.tensor_shapes()[name]
        if tuple(w.shape) != want:
            raise ValueError(f"{name} has shape {tuple(w.shape)}, expected {want}")
        w = w.to(self.dtype)
        rows, cols = rows or w.shape[0], cols or w.shape[1]
        if (rows, cols) != tuple(w.shape):
            w = torch.nn.functional.pad(w, (0, cols - w.shape[1], 0, rows - w.shape[0]))
        return self._attach(w, name)

    def _vector(self, name: str, size: int = None):
        """Attach a norm weight or a sink in fp32, zero-padded to `size`."""
        v = self._state[name].to(torch.float32)
        if tuple(v.shape) != self.config.tensor_shapes()[name]:
            raise ValueError(f"{name} has shape {tuple(v.shape)}, expected {self.config.tensor_shapes()[name]}")
        return self._attach(torch.nn.functional.pad(v, (0, (size or len(v)) - len(v))), name)

    def _rows(self, name: str, cols: int, dt):
        """Activation rows of one iteration (library-owned, zero-filled), one tensor per name and size."""
        key = f"{name}_{cols}"
        if key not in self._acts:
            self._acts[key] = self.mpk.new_tensor(dims=(self.mpk.max_num_batched_tokens, cols), dtype=dt, name=key, io_category="cuda_tensor")
        return self._acts[key]

    def _rotary(self, layer: SuboraxLayer):
        from .. import checkpoint
        if layer.rot_dims == 0:
            return None, None
        key = (layer.rot_dims, layer.rot_base, tuple(sorted((layer.rot_scaling or {}).items())))
        if key not in self._tables:
            cos, sin = checkpoint.rotary_tables_f32(layer.rot_dims, layer.rot_base, layer.rot_scaling, self.mpk.max_seq_length, self.mpk.device)
            n = len(self._tables)
            self._tables[key] = (self._attach(cos, f"cos_{n}"), self._attach(sin, f"sin_{n}"))
        return self._tables[key]

    def allocate_kv_cache(self):
        """Per layer [pages, page_size, kv heads, padded head size]; zero-filled."""
        mpk = self.mpk
        self.k_cache, self.v_cache = [], []
        for l in self.config.layers:
            dk, dv = flex_cache_dims(l.dim, l.vdim, self.dtype)
            self.k_cache.append(torch.zeros(mpk.max_num_pages, mpk.page_size, l.kv_heads, dk, dtype=self.dtype, device=mpk.device))
            self.v_cache.append(torch.zeros(mpk.max_num_pages, mpk.page_size, l.kv_heads, dv, dtype=self.dtype, device=mpk.device))

    # ------------------------------------------------------------------ graph
    def build_from_dict(self, state_dict: dict, with_lm_head: bool = True):
        mpk, c = self.mpk, self.config
        missing = sorted(set(c.tensor_shapes()) - set(state_dict))
        if missing:
            raise KeyError(f"the state dict lacks {missing}")
        self._state, self._acts = state_dict, {}
        self.with_lm_head = with_lm_head
        f32 = self.dtype == torch.float32
        E = float32 if f32 else bfloat16
        if self.k_cache is None:
            self.allocate_kv_cache()
        W = _pad64(c.width)
        one = dict(grid_dim=(1, 1, 1), block_dim=(256, 1, 1))
        # the residual rows alternate between two buffers: a single-token iteration forms the new rows in every workgroup of
        # the linear that reads them, from the old ones
        streams = [self._rows("residual_a", W, float32), self._rows("residual_b", W, float32)]
        which = 0
        x16 = self._rows("stream", W, E)
        y = self._rows("mixer_out", W, E)
        rows = lambda: streams[which] if f32 else x16  # what the next linear reads

        def norm(inp, name, alpha):
            nonlocal which
            old, which = streams[which], 1 - which
            mpk.residual_rmsnorm_layer(input=inp, residual=old, weight=self._vector(name, W), new_residual=streams[which], output=rows(), width=c.width,
                                       alpha=alpha, eps=c.eps, weight_offset=1.0)

        ids = self._attach(mpk.meta_tensors["input_tokens"], "input_token")
        spec, spec_tokens = mpk.spec_decode_config, None
        if spec is not None:
            all_tokens = self._attach(mpk.meta_tensors["tokens"], "all_tokens")
            spec_tokens = mpk.draft_forward_layer_dispatcher(spec_decode_config=spec, tokens=all_tokens, grid_dim=(96, 1, 1), block_dim=(128, 1, 1))
            ids = spec_tokens
        mpk.embed_scaled_layer(input=ids, weight=self._linear_weight("embed"), residual=streams[which], output=rows(), scale=c.embedding_scale)
        for i, l in enumerate(c.layers):
            p = f"l{i}."
            qkv = self._rows("qkv", l.qkv_cols, E)
            w_qkv = mpk.shuffle_tensors(inputs=[self._linear_weight(p + "mix." + n, cols=W) for n in "qkv"], shuffled_dim=0, num_groups=1, name=p + "mix.qkv")
            mpk.linear_layer(input=rows(), weight=w_qkv, output=qkv, **one)
            dk, _ = flex_cache_dims(l.dim, l.vdim, self.dtype)
            attn_cols = _pad64(l.heads * l.vdim)
            attn = self._rows(f"attn_out_{l.heads * l.vdim}", attn_cols, E)
            cos, sin = self._rotary(l)
            mpk.flex_attention_layer(input=qkv, k_cache=self._attach(self.k_cache[i], p + "k_cache"), v_cache=self._attach(self.v_cache[i], p + "v_cache"),
                                     cos=cos, sin=sin, sink=self._vector(p + "mix.sink"), q_workspace=self._rows("q_ws", l.heads * dk, E), output=attn,
                                     num_q_heads=l.heads, num_kv_heads=l.kv_heads, head_dim=l.dim, v_dim=l.vdim, rot_dims=l.rot_dims, scale=l.scale,
                                     softcap=l.softcap, unit_norm=True, eps=c.eps)
            mpk.linear_layer(input=attn, weight=self._linear_weight(p + "mix.o", cols=attn_cols), output=y, **one)
            norm(y, p + "norm1", c.alpha)
            if l.ff is None:
                continue
            F = _pad64(l.ff)
            act = self._rows(f"act_{l.ff}", F, E)
            w_gu = mpk.shuffle_tensors(inputs=[self._linear_weight(p + "mlp." + n, rows=F, cols=W) for n in ("gate", "up")], shuffled_dim=0, num_groups=1,
                                       name=p + "mlp.gate_up")
            gate_up = self._rows("gate_up", 2 * F, E)  # never written: the activation is the linear's epilogue
            mpk.linear_layer(input=rows(), weight=w_gu, output=gate_up, **one)
            mpk.silu_mul_layer(input=gate_up, output=act, **one)
            mpk.linear_layer(input=act, weight=self._linear_weight(p + "mlp.down", cols=F), output=y, **one)
            norm(y, p + "norm2", c.alpha)
        norm(None, "final.norm", 1.0)
        self.hidden = rows()
        if not with_lm_head:
            if spec_tokens is not None:
                raise ValueError("speculative decoding needs the LM head and the sampling stages in the graph (with_lm_head)")
            self._state = None
            return
        self.logits = self._rows("logits", c.vocab, E)
        mpk.linear_layer(input=rows(), weight=self._linear_weight("head", cols=W), output=self.logits, **one)
        out = self._attach(mpk.meta_tensors["output_tokens"], "output_token")
        part = (self._rows("argmax_value", mpk.num_workers, E), self._rows("argmax_index", mpk.num_workers, int64))
        mpk.argmax_partial_layer(input=self.logits, output=part, grid_dim=(mpk.num_workers, 1, 1), block_dim=(128, 1, 1))
        mpk.argmax_reduce_layer(input=part, output=out, grid_dim=(1, 1, 1), block_dim=(128, 1, 1))
        if spec_tokens is not None:
            self.verify_out = mpk.verify_layer_dispatcher(spec_decode_config=spec, spec_tokens=spec_tokens, target_output=out)
        self._state = None

    def decode(self, ids: torch.Tensor):
        return self.tokenizer.decode(ids, skip_special_tokens=True)
