"""Plain, slow restatement of the Bukatar decoder, one function per mechanism (the oracle of tests/test_bukatar*.py).

Nothing here is shared with the product path: no page tables, no batching, every head, expert and token is formed on its own.
All functions compute in the dtype of their inputs (the tests use float64 for the truth).

A layer reads its residual stream x twice, with an RMS norm N in front of and behind each sub-layer:

    x <- x + N1b(mixer(N1(x)));   x <- x + N2b(ff(N2(x)))          (the second only where the layer has a feed-forward)

The mixer is a windowed attention whose values are its keys before rotation, an attention over one cached latent per position, or
a selective scan behind a short convolution; the feed-forward is dense (square of relu) or a mixture of experts with a gated
shared expert.
"""
from dataclasses import dataclass
from typing import Optional

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def relu_squared(z):
    return torch.where(z > 0, z * z, torch.zeros_like(z))


def softplus(z):
    """log(1 + e^z)"""
    return torch.logaddexp(z, torch.zeros_like(z))


def rotate_pairs(x, positions, dims, base):
    """x [tokens, ..., D]: of the first `dims` dimensions, 2i and 2i + 1 turn together by position * base^(-2i/dims)."""
    if dims == 0:
        return x
    f = torch.tensor([float(base) ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    a = (positions.to(torch.float64)[:, None] * f[None, :]).reshape(len(positions), *([1] * (x.dim() - 2)), dims // 2)
    c, s = a.cos().to(x.dtype), a.sin().to(x.dtype)
    out = x.clone()
    u, v = x[..., 0:dims:2], x[..., 1:dims:2]
    out[..., 0:dims:2] = u * c - v * s
    out[..., 1:dims:2] = v * c + u * s
    return out


def window_sees(q_pos, k_pos, size, keep_first):
    """[Q, K] bool: nothing ahead, the `size` newest positions (its own included) and the `keep_first` first ones."""
    i, j = q_pos[:, None], k_pos[None, :]
    sees = j <= i
    if size is not None:
        sees = sees & ((i - j < size) | (j < keep_first))
    return sees


def sink_softmax(s, sees):
    """exp(s_j) / (1 + sum exp(s_j)) over the visible keys."""
    m = torch.clamp(s.masked_fill(~sees, float("-inf")).max(dim=-1, keepdim=True).values, min=0.0)
    e = torch.where(sees, torch.exp(s - m), torch.zeros_like(s))
    return e / (torch.exp(-m) + e.sum(dim=-1, keepdim=True))


def window_attention_core(q, k, v, q_pos, scale, size, keep_first):
    """q [T, H, D], k [S, G, D], v [S, G, E] at positions 0..S-1; query head h reads key/value head h // (H / G)."""
    T, H = q.shape[:2]
    per = H // k.shape[1]
    sees = window_sees(q_pos, torch.arange(k.shape[0]), size, keep_first)
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        out[:, h] = sink_softmax((q[:, h] @ k[:, h // per].T) * scale, sees) @ v[:, h // per]
    return out


def latent_attention_core(q_plain, q_rot, c, k_rot, w_uk, w_uv, q_pos, scale):
    """q_plain [T, H, D], q_rot [T, H, P], latents c [S, R], shared rotated keys k_rot [S, P], w_uk [H, D, R], w_uv [H, E, R]."""
    T, H = q_plain.shape[:2]
    out = torch.empty(T, H, w_uv.shape[1], dtype=q_plain.dtype)
    hidden = torch.arange(c.shape[0])[None, :] > q_pos[:, None]
    for h in range(H):
        s = (q_plain[:, h] @ (c @ w_uk[h].T).T + q_rot[:, h] @ k_rot.T) * scale
        out[:, h] = torch.softmax(s.masked_fill(hidden, float("-inf")), dim=-1) @ (c @ w_uv[h].T)
    return out


def causal_conv(x, tail, w, b):
    """x [T, C], tail [taps - 1, C] the inputs before them (zeros where a sequence begins), w [C, taps] (last column: the current
    token's), b [C].  Returns (convolved [T, C], new tail)."""
    taps = w.shape[1]
    rows = torch.cat([tail, x])
    y = b.expand(len(x), -1).clone()
    for j in range(taps):
        y = y + rows[j:j + len(x)] * w[:, j]
    return y, rows[len(rows) - (taps - 1):]


def scan_step(S, dt, x, A, B, C, D):
    """One token.  S [channels, states]: S' = exp(dt A) S + dt x B, y = S' C + D x."""
    S = torch.exp(dt[:, None] * A) * S + (dt * x)[:, None] * B[None, :]
    return S, S @ C + D * x


def selective_scan(S, dt, x, A, B, C, D):
    """dt, x [T, channels], A [channels, states], B, C [T, states], D [channels].  Returns (S after the last token, y)."""
    y = torch.empty_like(x)
    for t in range(len(x)):
        S, y[t] = scan_step(S, dt[t], x[t], A, B[t], C[t], D)
    return S, y


def route(z, top):
    """z [experts] -> (chosen experts, weights): softmax over all, the largest `top`, divided by their sum."""
    s = torch.softmax(z, dim=-1)
    idx = torch.argsort(s, descending=True, stable=True)[:top]
    return idx, s[idx] / (s[idx].sum() + 1e-20)


@dataclass
class LayerState:
    k: Optional[torch.Tensor] = None     # window attention: rotated keys, unrotated keys as values; latent attention: k_rot, latents
    v: Optional[torch.Tensor] = None
    S: Optional[torch.Tensor] = None     # scan state [channels, states]
    tail: Optional[torch.Tensor] = None  # last inputs of the convolution

    def extend(self, k, v):
        self.k = k if self.k is None else torch.cat([self.k, k])
        self.v = v if self.v is None else torch.cat([self.v, v])


class BukatarOracle:
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
        y = x @ self.w[name].T
        return self.r(y + self.w[name + ".b"] if name + ".b" in self.w else y)

    def attention(self, i, h, pos, state):
        m, p = self.c["layers"][i]["mixer"], f"l{i}.mix."
        T, H, G, D = len(h), m["heads"], m["kv_heads"], m["dim"]
        mask, rot = m.get("mask") or {}, m.get("rot") or {"dims": 0, "base": 1.0}
        turn = lambda t: self.r(rotate_pairs(t, pos, rot["dims"], rot["base"]))
        q, k = self.lin(h, p + "q").view(T, H, D), self.lin(h, p + "k").view(T, G, D)
        state[i].extend(turn(k), k)
        return self.r(window_attention_core(turn(q), state[i].k, state[i].v, pos, m["scale"], mask.get("size"), mask.get("keep_first", 0))).reshape(T, H * D)

    def latent_attention(self, i, h, pos, state):
        m, p, w = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w
        T, H, D, P, E, R = len(h), m["heads"], m["dim"], m["rot_dim"], m["vdim"], m["kv_rank"]
        turn = lambda t: self.r(rotate_pairs(t, pos, P, m["rot"]["base"]))
        q = self.lin(h, p + "q").view(T, H, D + P)
        owner = m.get("kv_from")
        if owner is None:
            ckr = self.lin(h, p + "dkv")
            state[i].extend(turn(ckr[:, R:]), self.r(rms_norm(ckr[:, :R], w[p + "dkv.norm"], self.eps)))
            owner = i
        o = latent_attention_core(q[..., :D], turn(q[..., D:]), state[owner].v, state[owner].k, w[p + "uk"].view(H, D, R), w[p + "uv"].view(H, E, R), pos, m["scale"])
        return self.r(o).reshape(T, H * E)

    def mamba1(self, i, h, pos, state):
        m, p, w, st = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w, state[i]
        I, N, K, R = m["inner"], m["state"], m["conv"], m["dt_rank"]
        xz = self.lin(h, p + "in")
        if st.S is None:
            st.S, st.tail = torch.zeros(I, N, dtype=self.dtype), torch.zeros(K - 1, I, dtype=self.dtype)
        x, st.tail = causal_conv(xz[:, :I], st.tail, w[p + "conv"], w[p + "conv.b"])
        x = self.r(silu(x))
        dbc = self.lin(x, p + "x")
        dt = softplus(dbc[:, :R] @ w[p + "dt"].T + w[p + "dt.b"])
        st.S, y = selective_scan(st.S, dt, x, -torch.exp(w[p + "A_log"]), dbc[:, R:R + N], dbc[:, R + N:], w[p + "D"])
        return self.r(y * silu(xz[:, I:]))

    def expert(self, h, p):
        return self.lin(self.r(silu(h @ self.w[p + ".gate"].T) * (h @ self.w[p + ".up"].T)), p + ".down")

    def feed_forward(self, i, h):
        mlp, p = self.c["layers"][i]["mlp"], f"l{i}.mlp"
        if mlp.get("kind", "dense") == "dense":
            return self.lin(self.r(relu_squared(h @ self.w[p + ".up"].T)), p + ".down")
        z, y = h @ self.w[p + ".router"].T, torch.zeros_like(h)
        for t in range(len(h)):
            for e, g in zip(*route(z[t], mlp["router"]["top"])):
                y[t] += g * self.expert(h[t:t + 1], f"{p}.e{int(e)}")[0]
        if mlp.get("shared"):
            y = y + torch.sigmoid(h @ self.w[p + ".shared.sg"].T) * self.expert(h, p + ".shared")
        return y

    def layer(self, i, x, pos, state):
        w, r, e, p = self.w, self.r, self.c["layers"][i], f"l{i}."
        y = self.lin(getattr(self, e["type"])(i, r(rms_norm(x, w[p + "norm1"], self.eps)), pos, state), p + "mix.o")
        x = x + rms_norm(y, w[p + "norm1b"], self.eps)
        if e.get("mlp") is not None:
            x = x + rms_norm(self.feed_forward(i, r(rms_norm(x, w[p + "norm2"], self.eps))), w[p + "norm2b"], self.eps)
        return x

    def forward(self, tokens, state, start, streams=None):
        """Logits of `tokens`, which follow `start` earlier ones that `state` has seen."""
        tokens = torch.as_tensor(tokens, dtype=torch.long)
        pos = torch.arange(start, start + len(tokens))
        x = self.w["embed"][tokens]
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x, pos, state)
            if streams is not None:
                streams.append(x)
        return self.r(rms_norm(x, self.w["final.norm"], self.eps)) @ self.w["embed"].T

    def generate(self, prompt, n):
        """Greedy continuation: n tokens after the prompt."""
        state, toks = self.new_state(), list(prompt)
        logits = self.forward(toks, state, 0)[-1]
        for _ in range(n):
            toks.append(int(logits.argmax()))
            logits = self.forward(toks[-1:], state, len(toks) - 1)[-1]
        return toks
