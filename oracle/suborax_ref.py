"""Plain, slow restatement of the Suborax decoder, one function per mechanism (the oracle of tests/test_suborax*.py).

Nothing here is shared with the product path: no page tables, no batching, no cache unless the caller keeps one.  All
functions compute in the dtype of their inputs (the tests use float64 for the truth and float32 where they want rounding
of the same size as the kernel's).

A layer holds one residual stream x [tokens, width] and updates it with the norm BEHIND each sum:

    x <- N1(alpha x + attention(x)),    x <- N2(alpha x + swiglu(x)),    N(y) = y / sqrt(mean(y^2) + eps) * (1 + w)

The attention rotates the first `rot.dims` dimensions of every query and key head (rotate-half pairing, Llama-3.1 frequency
scaling), divides the rotated heads by their root mean square, caps the scores with tanh, and lets a learned per-head
logit (the sink) take part in the softmax's denominator without a key or a value.
"""
import math
from dataclasses import dataclass
from typing import Optional

import torch


def rms_divide(x, eps):
    """x / sqrt(mean(x^2) + eps) over the last dimension."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def rms_norm_offset(x, w, eps):
    """RMS norm whose stored weight is the distance from one."""
    return rms_divide(x, eps) * (1.0 + w)


def rotary_frequencies(rot: dict):
    """f_i, i < dims/2, float64: base^(-2i/dims), then the Llama-3.1 scaling by wavelength when `rot` has one."""
    dims = rot["dims"]
    out = []
    sc = rot.get("scaling")
    for i in range(dims // 2):
        f = float(rot["base"]) ** (-2.0 * i / dims)
        if sc:
            wavelength = 2.0 * math.pi / f
            if wavelength < sc["original"] / sc["high"]:
                pass
            elif wavelength > sc["original"] / sc["low"]:
                f = f / sc["factor"]
            else:
                s = (sc["original"] / wavelength - sc["low"]) / (sc["high"] - sc["low"])
                f = (1.0 - s) * f / sc["factor"] + s * f
        out.append(f)
    return torch.tensor(out, dtype=torch.float64)


def rotate(x, positions, rot: dict):
    """x [tokens, heads, dim]; dimension i < dims/2 pairs with i + dims/2, the rest passes."""
    dims = rot["dims"]
    ang = positions.to(torch.float64)[:, None] * rotary_frequencies(rot)[None, :]
    c, s = ang.cos().to(x.dtype)[:, None, :], ang.sin().to(x.dtype)[:, None, :]
    u, v, rest = x[..., :dims // 2], x[..., dims // 2:dims], x[..., dims:]
    return torch.cat([u * c - v * s, v * c + u * s, rest], dim=-1)


def cap_scores(s, cap):
    return s if not cap else cap * torch.tanh(s / cap)


def softmax_with_sink(s, sink):
    """s [..., keys] with -inf where masked; sink broadcastable to s[..., 0].  Rows sum to less than one."""
    m = torch.maximum(s.amax(dim=-1), sink)
    e = torch.exp(s - m[..., None])
    return e / (e.sum(dim=-1) + torch.exp(sink - m))[..., None]


def attention_core(q, k, v, q_pos, sink, scale, cap):
    """q [Tq, H, dim], k [Tk, G, dim], v [Tk, G, vdim]; key j sits at position j.  Returns [Tq, H, vdim]."""
    H, G = q.shape[1], k.shape[1]
    out = torch.empty(q.shape[0], H, v.shape[2], dtype=q.dtype)
    j = torch.arange(k.shape[0])
    for h in range(H):
        g = h // (H // G)
        s = cap_scores((q[:, h] @ k[:, g].T) * scale, cap)
        s = s.masked_fill(j[None, :] > q_pos[:, None], float("-inf"))
        p = softmax_with_sink(s, sink[h].to(s.dtype).expand(s.shape[0]))
        out[:, h] = p @ v[:, g]
    return out


def swiglu(h, gate, up, down):
    a = h @ gate.T
    return (a * torch.sigmoid(a) * (h @ up.T)) @ down.T


@dataclass
class Cache:
    """Rotated, normalised keys and the values of one layer, in position order."""
    k: Optional[torch.Tensor] = None
    v: Optional[torch.Tensor] = None

    def extend(self, k, v):
        self.k = k if self.k is None else torch.cat([self.k, k])
        self.v = v if self.v is None else torch.cat([self.v, v])


class SuboraxOracle:
    """config: the parsed config.json; weights: name -> tensor.  `round16` (optional) is applied where a 16-bit engine
    stores a value: linear inputs and outputs, cached keys and values."""

    def __init__(self, config: dict, weights: dict, dtype=torch.float64, round16=False):
        self.c, self.dtype = config, dtype
        self.w = {n: t.to(dtype) for n, t in weights.items()}
        self.r = (lambda t: t.to(torch.bfloat16).to(dtype)) if round16 else (lambda t: t)

    def new_state(self):
        return [Cache() for _ in self.c["layers"]]

    def attention(self, i, h, pos, cache: Cache):
        m, w, r = self.c["layers"][i]["mixer"], self.w, self.r
        H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
        T = h.shape[0]
        q = r(h @ w[f"l{i}.mix.q"].T).view(T, H, D)
        k = r(h @ w[f"l{i}.mix.k"].T).view(T, G, D)
        v = r(h @ w[f"l{i}.mix.v"].T).view(T, G, E)
        eps = self.c["norm"]["eps"]
        q = r(rms_divide(rotate(q, pos, m["rot"]), eps))
        k = r(rms_divide(rotate(k, pos, m["rot"]), eps))
        cache.extend(k, v)
        o = attention_core(q, cache.k, cache.v, pos, w[f"l{i}.mix.sink"], m["scale"], m["softcap"])
        return r(r(o).reshape(T, H * E) @ w[f"l{i}.mix.o"].T)

    def layer(self, i, x, pos, cache):
        c, w, r = self.c, self.w, self.r
        eps, alpha = c["norm"]["eps"], c["postln_alpha"]
        x = rms_norm_offset(alpha * x + self.attention(i, r(x), pos, cache), w[f"l{i}.norm1"], eps)
        if c["layers"][i]["mlp"] is not None:
            h = r(x)
            a, u = h @ w[f"l{i}.mlp.gate"].T, h @ w[f"l{i}.mlp.up"].T
            f = r(r(a * torch.sigmoid(a) * u) @ w[f"l{i}.mlp.down"].T)
            x = rms_norm_offset(alpha * x + f, w[f"l{i}.norm2"], eps)
        return x

    def forward(self, tokens, state, start, streams=None):
        """Logits of `tokens`, which follow `start` earlier ones whose keys and values are in `state`."""
        pos = torch.arange(start, start + len(tokens))
        x = self.w["embed"][torch.as_tensor(tokens, dtype=torch.long)] * self.c["embedding"]["scale"]
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x, pos, state[i])
            if streams is not None:
                streams.append(x)
        h = self.r(rms_norm_offset(x, self.w["final.norm"], self.c["norm"]["eps"]))
        return h @ self.w["head"].T

    def generate(self, prompt, n):
        """Greedy continuation: n tokens after the prompt."""
        state, toks = self.new_state(), list(prompt)
        logits = self.forward(toks, state, 0)[-1]
        for _ in range(n):
            toks.append(int(logits.argmax()))
            logits = self.forward(toks[-1:], state, len(toks) - 1)[-1]
        return toks
