"""Plain, slow restatement of the Vizonex decoder, one function per mechanism (the oracle of tests/test_vizonex*.py).

Nothing here is shared with the product path: no page tables, no batching, every head, expert and token is formed on its own.
All functions compute in the dtype of their inputs (the tests use float64 for the truth).

A layer reads its residual stream x once; both sub-layers work on the same norm N and join the stream together, each scaled by a
vector of its own:

    h = N(x);   x <- x + s1 * mixer(h + conv(h)) + s2 * ff(h)          (s2 * ff(h) only where the layer has a feed-forward)

The mixer is an attention inside chunks of the sequence or a state-space recurrence with one decay per head; the feed-forward is
dense (tanh gelu, gated) or a mixture of experts chosen group by group.
"""
import math
from dataclasses import dataclass
from typing import Optional

import torch


def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def rms_norm_parts(x, w, eps, parts):
    """The row in `parts` equal parts, each divided by its own root mean square."""
    T, n = x.shape
    y = x.reshape(T, parts, n // parts)
    return (y / torch.sqrt((y * y).mean(dim=-1, keepdim=True) + eps)).reshape(T, n) * w


def silu(z):
    return z / (1.0 + torch.exp(-z))


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def clamped_gate(a, b, limit):
    """g sigmoid(1.702 g) (u + 1) with g = min(a, limit) and u = b clamped to [-limit, limit]."""
    g, u = torch.clamp(a, max=limit), torch.clamp(b, min=-limit, max=limit)
    return g / (1.0 + torch.exp(-1.702 * g)) * (u + 1.0)


def softplus(z):
    """log(1 + e^z)"""
    return torch.logaddexp(z, torch.zeros_like(z))


def causal_conv(x, tail, w, b=None):
    """x [T, C], tail [taps - 1, C] the inputs before them (zeros where a sequence begins), w [C, taps] (last column: the current
    token's), b [C] or None.  Returns (convolved [T, C], new tail)."""
    taps = w.shape[1]
    rows = torch.cat([tail, x])
    y = torch.zeros_like(x) if b is None else b.expand(len(x), -1).clone()
    for j in range(taps):
        y = y + rows[j:j + len(x)] * w[:, j]
    return y, rows[len(rows) - (taps - 1):]


def chunk_sees(q_pos, k_pos, size):
    """[Q, K] bool: nothing ahead, and only positions of the query's own chunk of `size` positions, counted from position 0."""
    i, j = q_pos[:, None], k_pos[None, :]
    sees = j <= i
    if size:
        sees = sees & (torch.div(i, size, rounding_mode="floor") == torch.div(j, size, rounding_mode="floor"))
    return sees


def sink_softmax(s, sees, sink):
    """exp(s_j) / (exp(sink) + sum exp(s_j)) over the visible keys."""
    sink = torch.as_tensor(sink, dtype=s.dtype)
    m = torch.maximum(s.masked_fill(~sees, float("-inf")).max(dim=-1, keepdim=True).values, sink)
    e = torch.where(sees, torch.exp(s - m), torch.zeros_like(s))
    return e / (torch.exp(sink - m) + e.sum(dim=-1, keepdim=True))


def chunk_attention_core(q, k, v, q_pos, scale, temp, sink, size):
    """q [T, H, D], k [S, G, D], v [S, G, E] at positions 0..S-1, temp and sink [H]; query head h reads key/value head h // (H / G)."""
    T, H = q.shape[:2]
    per = H // k.shape[1]
    sees = chunk_sees(q_pos, torch.arange(k.shape[0]), size)
    out = torch.empty(T, H, v.shape[2], dtype=q.dtype)
    for h in range(H):
        out[:, h] = sink_softmax((q[:, h] @ k[:, h // per].T) * scale * temp[h], sees, sink[h]) @ v[:, h // per]
    return out


def dual_step(S, dt, x, A, B, C, D):
    """One token of one head.  S [states, values], x [values], B and C [states], the rest numbers: S' = exp(dt A) S + dt B x^T,
    y = S'^T C + D x."""
    S = torch.exp(dt * A) * S + dt * torch.outer(B, x)
    return S, S.T @ C + D * x


def dual_scan(S, dt, x, A, B, C, D):
    """S [heads, states, values], dt [T, heads], x [T, heads, values], A and D [heads], B and C [T, groups, states]; head h reads group
    h // (heads / groups).  Returns (S after the last token, y)."""
    S, y = S.clone(), torch.empty_like(x)
    per = S.shape[0] // B.shape[1]
    for t in range(len(x)):
        for h in range(S.shape[0]):
            S[h], y[t, h] = dual_step(S[h], dt[t, h], x[t, h], A[h], B[t, h // per], C[t, h // per], D[h])
    return S, y


def route_groups(z, correction, top, count, keep, scale):
    """z [experts] -> (chosen experts, weights).  Sigmoid scores; choices are made on scores + correction: the `keep` groups (of `count`
    equal ones of neighbours) whose two largest choice scores have the largest sum, then the `top` largest among their experts.  The
    weights are scale times the scores themselves."""
    s = torch.sigmoid(z)
    choice = s + correction
    groups = choice.view(count, -1)
    best = groups.sort(dim=-1, descending=True).values[:, :2].sum(-1)
    kept = torch.argsort(best, descending=True, stable=True)[:keep]
    open_ = torch.full_like(groups, float("-inf"))
    open_[kept] = groups[kept]
    idx = torch.argsort(open_.view(-1), descending=True, stable=True)[:top]
    return idx, s[idx] * scale


@dataclass
class LayerState:
    canon: Optional[torch.Tensor] = None  # last normed rows (input convolution)
    k: Optional[torch.Tensor] = None      # attention
    v: Optional[torch.Tensor] = None
    S: Optional[torch.Tensor] = None      # recurrence [heads, states, values]
    tail: Optional[torch.Tensor] = None   # last inputs of its convolution

    def extend(self, k, v):
        self.k = k if self.k is None else torch.cat([self.k, k])
        self.v = v if self.v is None else torch.cat([self.v, v])


class VizonexOracle:
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

    def attention(self, i, h, pos, state):
        m, p, w = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w
        T, H, G = len(h), m["heads"], m["kv_heads"]
        q = self.r(rms_norm(self.lin(h, p + "q"), w[p + "q.norm"], self.eps)).view(T, H, m["dim"])
        k = self.r(rms_norm(self.lin(h, p + "k"), w[p + "k.norm"], self.eps)).view(T, G, m["dim"])
        state[i].extend(k, self.lin(h, p + "v").view(T, G, m["vdim"]))
        size = (m.get("mask") or {}).get("size")
        return self.r(chunk_attention_core(q, state[i].k, state[i].v, pos, m["scale"], w[p + "temp"], w[p + "sink"], size)).reshape(T, H * m["vdim"])

    def mamba2(self, i, h, pos, state):
        m, p, w, st = self.c["layers"][i]["mixer"], f"l{i}.mix.", self.w, state[i]
        T, H, V, N, G = len(h), m["heads"], m["vdim"], m["state"], m["groups"]
        I = H * V
        z, xbc, dt = self.lin(h, p + "in").split([I, I + 2 * G * N, H], dim=1)
        if st.S is None:
            st.S, st.tail = torch.zeros(H, N, V, dtype=self.dtype), torch.zeros(m["conv"] - 1, I + 2 * G * N, dtype=self.dtype)
        xbc, st.tail = causal_conv(xbc, st.tail, w[p + "conv"], w[p + "conv.b"])
        x, B, C = self.r(silu(xbc)).split([I, G * N, G * N], dim=1)
        st.S, y = dual_scan(st.S, softplus(dt + w[p + "dt_bias"]), x.view(T, H, V), -torch.exp(w[p + "A_log"]), B.view(T, G, N), C.view(T, G, N), w[p + "D"])
        return self.r(rms_norm_parts(y.reshape(T, I) * silu(z), w[p + "norm"], self.eps, m["norm_groups"]))

    def expert(self, h, p, limit):
        return self.lin(self.r(clamped_gate(h @ self.w[p + ".gate"].T, h @ self.w[p + ".up"].T, limit)), p + ".down")

    def feed_forward(self, i, h):
        mlp, p, w = self.c["layers"][i]["mlp"], f"l{i}.mlp", self.w
        if mlp.get("kind", "dense") == "dense":
            return self.lin(self.r(gelu_tanh(h @ w[p + ".gate"].T) * (h @ w[p + ".up"].T)), p + ".down")
        r, y = mlp["router"], torch.zeros_like(h)
        g = r.get("groups") or {"count": 1, "keep": 1}
        z = h @ w[p + ".router"].T
        for t in range(len(h)):
            for e, s in zip(*route_groups(z[t], w[p + ".correction"], r["top"], g["count"], g["keep"], r["scale"])):
                y[t] += s * self.expert(h[t:t + 1], f"{p}.e{int(e)}", mlp["expert"]["limit"])[0]
        if mlp.get("shared"):
            y = y + self.expert(h, p + ".shared", mlp["shared"]["limit"])
        return y

    def layer(self, i, x, pos, state):
        w, r, e, p, st = self.w, self.r, self.c["layers"][i], f"l{i}.", state[i]
        h = r(rms_norm(x, w[p + "norm1"], self.eps))
        if st.canon is None:
            st.canon = torch.zeros(self.c["canon"]["taps"] - 1, x.shape[1], dtype=self.dtype)
        y, st.canon = causal_conv(h, st.canon, w[p + "canon1"])
        out = w[p + "ls1"] * self.lin(getattr(self, e["type"])(i, r(h + y), pos, state), p + "mix.o")
        if e.get("mlp") is not None:
            out = out + w[p + "ls2"] * self.feed_forward(i, h)
        return x + out

    def forward(self, tokens, state, start, streams=None):
        """Logits of `tokens`, which follow `start` earlier ones that `state` has seen."""
        tokens = torch.as_tensor(tokens, dtype=torch.long)
        pos = torch.arange(start, start + len(tokens))
        x = self.w["embed"][tokens] + self.w["pos"][pos]
        for i in range(len(self.c["layers"])):
            x = self.layer(i, x, pos, state)
            if streams is not None:
                streams.append(x)
        return self.r(rms_norm(x, self.w["final.norm"], self.eps)) @ self.w["head"].T

    def generate(self, prompt, n):
        """Greedy continuation: n tokens after the prompt."""
        state, toks = self.new_state(), list(prompt)
        logits = self.forward(toks, state, 0)[-1]
        for _ in range(n):
            toks.append(int(logits.argmax()))
            logits = self.forward(toks[-1:], state, len(toks) - 1)[-1]
        return toks
