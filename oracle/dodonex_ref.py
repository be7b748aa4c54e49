"""Plain, slow restatement of the Dodonex decoder, one function per mechanism (the oracle of tests/test_dodonex*.py).

Nothing here is shared with the product path: no page tables, no batching, keys and values are formed per head and the
recurrence is run token by token.  All functions compute in the dtype of their inputs (the tests use float64 for the truth).

A layer reads its residual stream x once, feeds the same normalised rows to both sub-layers, and then lets a per-token
vector of its own into the stream:

    h = N(x);  x <- x + m (mixer(h) + glu(h));   g = gelu(A x) * e[token];  x <- x + m rms_norm(B g)

with N an RMS norm over equal consecutive parts of the row.  The mixer is an attention whose keys and values are linear
images of one small latent per position, or a matrix-valued recurrence with decay and removal along key channels.
"""
import math
from dataclasses import dataclass
from typing import Optional

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def group_rms_norm(x, w, eps, groups):
    """Every one of `groups` consecutive parts is divided by a root mean square of its own."""
    parts = x.reshape(*x.shape[:-1], groups, x.shape[-1] // groups)
    return (parts / torch.sqrt((parts * parts).mean(dim=-1, keepdim=True) + eps)).reshape(x.shape) * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def clamped_glu(gate, up, limit):
    g, u = torch.clamp(gate, max=limit), torch.clamp(up, min=-limit, max=limit)
    return g * torch.sigmoid(1.702 * g) * (u + 1.0)


def rotate_half(x, positions, base):
    """x [tokens, ..., dims]: dimension i < dims/2 pairs with i + dims/2, angle position * base^(-2i/dims)."""
    dims = x.shape[-1]
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = (positions.to(torch.float64)[:, None] * f[None, :]).reshape(len(positions), *([1] * (x.dim() - 2)), dims // 2)
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    u, v = x[..., :dims // 2], x[..., dims // 2:]
    return torch.cat([u * c - v * s, v * c + u * s], dim=-1)


def latent_attention_core(q_plain, q_rot, c, k_rot, w_uk, w_uv, q_pos, scale):
    """q_plain [T, H, D], q_rot [T, H, P], latents c [S, R] and shared rotated keys k_rot [S, P] at positions 0..S-1,
    w_uk [H, D, R], w_uv [H, E, R].  Returns [T, H, E]."""
    T, H = q_plain.shape[:2]
    out = torch.empty(T, H, w_uv.shape[1], dtype=q_plain.dtype)
    hidden = torch.arange(c.shape[0])[None, :] > q_pos[:, None]
    for h in range(H):
        k, v = c @ w_uk[h].T, c @ w_uv[h].T
        s = (q_plain[:, h] @ k.T + q_rot[:, h] @ k_rot.T) * scale
        p = torch.softmax(s.masked_fill(hidden, float("-inf")), dim=-1)
        out[:, h] = p @ v
    return out


def unit_key(k):
    """k / sqrt(sum(k^2) + 1e-6) over the last dimension."""
    return k / torch.sqrt((k * k).sum(dim=-1, keepdim=True) + 1e-6)


def decay(z):
    """Per-channel decay exp(-exp(-1/2) sigmoid(z))."""
    return torch.exp(-math.exp(-0.5) * torch.sigmoid(z))


def delta_step(S, r, w, a, k, v):
    """One token of one head.  S [D, E] -> (S', o): S' = diag(w) S - (a u)(u^T S) + k v^T with u the unit key, o = S'^T r."""
    u = unit_key(k)
    S = w[:, None] * S - (a * u)[:, None] * (u @ S)[None, :] + k[:, None] * v[None, :]
    return S, S.T @ r


def delta_scan(S, r, w, a, k, v):
    """r, w, a, k [T, H, D], v [T, H, E], S [H, D, E].  Returns (S after the last token, o [T, H, E])."""
    S, out = S.clone(), torch.empty_like(v)
    for t in range(r.shape[0]):
        for h in range(r.shape[1]):
            S[h], out[t, h] = delta_step(S[h], r[t, h], w[t, h], a[t, h], k[t, h], v[t, h])
    return S, out


@dataclass
class LayerState:
    c: Optional[torch.Tensor] = None      # latents, in position order
    k_rot: Optional[torch.Tensor] = None  # rotated shared keys
    S: Optional[torch.Tensor] = None      # recurrent state [heads, dim, dim]

    def extend(self, c, k_rot):
        self.c = c if self.c is None else torch.cat([self.c, c])
        self.k_rot = k_rot if self.k_rot is None else torch.cat([self.k_rot, k_rot])


class DodonexOracle:
    """config: the parsed config.json; weights: name -> tensor.  `round16` applies a rounding to 16 bits where a 16-bit engine
    stores a value: linear inputs and outputs and the cached rows."""

    def __init__(self, config: dict, weights: dict, dtype=torch.float64, round16=False):
        self.c, self.dtype = config, dtype
        self.w = {n: t.to(dtype) for n, t in weights.items() if t.is_floating_point()}
        self.r = (lambda t: t.to(torch.bfloat16).to(dtype)) if round16 else (lambda t: t)
        self.eps = config["norm"]["eps"]

    def new_state(self):
        return [LayerState() for _ in self.c["layers"]]

    def lin(self, x, name):
        return self.r(x @ self.w[name].T)

    def latent_attention(self, i, h, pos, state):
        m, p, w = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w
        H, D, P, E, R = m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        T, base = len(h), m["rot"]["base"]
        cq = self.r(rms_norm(self.lin(h, p + "dq"), w[p + "dq.norm"], self.eps))
        q = self.lin(cq, p + "uq").view(T, H, D + P)
        owner = m.get("kv_from")
        if owner is None:
            ckr = self.lin(h, p + "dkv")
            state[i].extend(self.r(rms_norm(ckr[:, :R], w[p + "dkv.norm"], self.eps)), self.r(rotate_half(ckr[:, R:], pos, base)))
            owner = i
        o = latent_attention_core(q[..., :D], self.r(rotate_half(q[..., D:], pos, base)), state[owner].c, state[owner].k_rot, w[p + "uk"].view(H, D, R),
                                  w[p + "uv"].view(H, E, R), pos, m["scale"])
        return self.r(o).reshape(T, H * E)

    def general_delta(self, i, h, pos, state):
        m, p, w = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w
        H, D, T = m["heads"], m["dim"], len(h)
        heads = lambda t: t.view(T, H, D)
        r, k, v = (heads(self.lin(h, p + n)) for n in "rkv")
        dec = decay(heads(torch.tanh(self.lin(h, p + "w1")) @ w[p + "w2"].T + w[p + "w0"]))
        a = torch.sigmoid(heads(self.lin(h, p + "a") + w[p + "a.b"]))
        S = state[i].S if state[i].S is not None else torch.zeros(H, D, D, dtype=self.dtype)
        state[i].S, o = delta_scan(S, r, dec, a, k, v)
        o = rms_norm(o, torch.ones(D, dtype=self.dtype), self.eps).reshape(T, H * D) * w[p + "norm"]
        return self.r(o * torch.sigmoid(self.lin(h, p + "g")))

    def layer(self, i, x, tokens, pos, state):
        c, w, r, e = self.c, self.w, self.r, self.c["layers"][i]
        p, m = f"l{i}.", self.c["residual_mult"]
        h = r(group_rms_norm(x, w[p + "norm1"], self.eps, c["norm"]["groups"]))
        y = getattr(self, e["type"])(i, h, pos, state) @ w[p + "mix.o"].T
        if e.get("mlp") is not None:
            g = clamped_glu(self.lin(h, p + "mlp.gate"), self.lin(h, p + "mlp.up"), e["mlp"]["limit"])
            y = y + r(g) @ w[p + "mlp.down"].T
        x = x + m * r(y)
        n = c["token_side"]["dim"]
        extra = w["side.embed"][tokens][:, i * n:(i + 1) * n]
        y = self.lin(r(gelu_tanh(r(x) @ w[p + "side.gate"].T) * extra), p + "side.proj")
        return x + m * rms_norm(y, w[p + "side.norm"], self.eps)

    def forward(self, tokens, state, start, streams=None):
        """Logits of `tokens`, which follow `start` earlier ones that `state` has seen."""
        tokens = torch.as_tensor(tokens, dtype=torch.long)
        pos = torch.arange(start, start + len(tokens))
        x = self.w["embed"][tokens] * self.c["embedding"]["scale"]
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x, tokens, pos, state)
            if streams is not None:
                streams.append(x)
        h = self.r(group_rms_norm(x, self.w["final.norm"], self.eps, self.c["norm"]["groups"]))
        return h @ self.w["embed"].T * self.c["logit_scale"]

    def generate(self, prompt, n):
        """Greedy continuation: n tokens after the prompt."""
        state, toks = self.new_state(), list(prompt)
        logits = self.forward(toks, state, 0)[-1]
        for _ in range(n):
            toks.append(int(logits.argmax()))
            logits = self.forward(toks[-1:], state, len(toks) - 1)[-1]
        return toks
