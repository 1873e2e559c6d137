"""Plain CPU statement of the Gukidra decoder (TEST INFRASTRUCTURE ONLY, like oracle/model.py).

One function per mechanism, fp32 torch on the host, no cache, no state pool and no batching: a sequence is always
recomputed whole, attention is a dense [T, T + blocks] matrix per head, block means are taken from the dense keys and values,
and the matrix memory is a Python loop over the tokens, so nothing here can share a fault with the engine's pools, kernels
or scheduler.  Weights arrive as a dict of tensors under the checkpoint's own names (`embed`, `l<i>.norm1`, `l<i>.mix.q`,
`l<i>.mix.q.norm`, `l<i>.mix.i.b`, `l<i>.mlp.gate`, ..., `final.norm`); the configuration is the checkpoint's config.json as a
dict.

Notation: T tokens, W the model width, H query heads (or memory heads), G key/value heads, D the key size, E the value size,
N the window, P the tokens of a block.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    x = x.float()
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def one_plus_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """Unit RMS times (1 + weight)."""
    return rms(x, eps) * (1.0 + weight.float())


def head_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    """x [T, heads, D]: every head to unit RMS, times a weight [D] all heads share."""
    return rms(x, eps) * weight.float()


def turn_halves(x: torch.Tensor, dims: int, base: float, back: bool = False) -> torch.Tensor:
    """x [T, heads, size]: element i < dims / 2 and element i + dims / 2 of every head are turned as a pair by the angle
    position * base^(-2i / dims) (by minus that with `back`); elements from dims on pass."""
    T = x.shape[0]
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64).float()
    ang = torch.arange(T, dtype=torch.float32).view(T, 1, 1) * f
    c, s = torch.cos(ang), torch.sin(ang) * (-1.0 if back else 1.0)
    x = x.float().clone()
    a, b = x[..., : dims // 2].clone(), x[..., dims // 2: dims].clone()
    x[..., : dims // 2] = a * c - b * s
    x[..., dims // 2: dims] = b * c + a * s
    return x


def block_means(x: torch.Tensor, pool: int) -> torch.Tensor:
    """x [T, G, size] -> [T // pool, G, size]: the mean of every whole block of `pool` tokens."""
    n = x.shape[0] // pool
    return x[: n * pool].view(n, pool, *x.shape[1:]).mean(1)


def pooled_window_mask(T: int, window: int, pool: int) -> torch.Tensor:
    """[T, T + T // pool] bool: which tokens and which blocks a position sees -- the last `window` tokens up to itself, and
    the blocks whose last token is at least `window` back."""
    i = torch.arange(T).view(T, 1)
    j = torch.arange(T).view(1, T)
    tokens = (j <= i) & (i - j < window)
    last = (torch.arange(T // pool).view(1, -1) + 1) * pool - 1
    return torch.cat([tokens, last <= i - window], 1)


def softmax_with_one(scores: torch.Tensor) -> torch.Tensor:
    """exp(s) / (1 + sum exp(s)) over the last axis; hidden entries are -inf."""
    m = torch.clamp(scores.amax(-1, keepdim=True), min=0.0)
    e = torch.exp(scores - m)
    return e / (torch.exp(-m) + e.sum(-1, keepdim=True))


def attention_kv(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float):
    """Keys (normed, turned) and values (turned) as a layer caches them: [T, G, D], [T, G, E]."""
    T, G, D, E = h.shape[0], m["kv_heads"], m["dim"], m["vdim"]
    k = head_norm((h.float() @ w[pre + "k"].float().t()).view(T, G, D), w[pre + "k.norm"], eps)
    v = (h.float() @ w[pre + "v"].float().t()).view(T, G, E)
    return turn_halves(k, m["rot"]["dims"], m["rot"]["base"]), turn_halves(v, E, m["rot"]["base"])


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float, kv) -> torch.Tensor:
    """kv: the (keys, values) of this layer, or of the layer whose cache it reads."""
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    h = h.float()
    q = head_norm((h @ w[pre + "q"].float().t()).view(T, H, D), w[pre + "q.norm"], eps)
    q = turn_halves(q, m["rot"]["dims"], m["rot"]["base"])
    window, pool = m["mask"]["size"], m["mask"]["pool"]
    k, v = (torch.cat([x, block_means(x, pool)], 0) for x in kv)
    of = torch.arange(H) // (H // G)
    s = torch.einsum("ihd,jhd->hij", q, k[:, of]) * m["scale"]
    s = s.masked_fill(~pooled_window_mask(T, window, pool).unsqueeze(0), float("-inf"))
    o = (softmax_with_one(s) @ v[:, of].transpose(0, 1)).transpose(0, 1)                # [T, H, E]
    o = turn_halves(o, E, m["rot"]["base"], back=True)
    o = o * torch.sigmoid(h @ w[pre + "g"].float().t()).view(T, H, 1)
    return o.reshape(T, H * E) @ w[pre + "o"].float().t()


def soft_cap(x: torch.Tensor, cap: float) -> torch.Tensor:
    return cap * torch.tanh(x / cap)


def memory_gates(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict):
    """(log input gate, log forget gate), each [T, H]."""
    h, cap = h.float(), float(m["gate_cap"])
    i = soft_cap(h @ w[pre + "i"].float().t() + w[pre + "i.b"].float(), cap)
    f = soft_cap(h @ w[pre + "f"].float().t() + w[pre + "f.b"].float(), cap)
    return i, torch.nn.functional.logsigmoid(f)


def matrix_memory_scan(q, k, v, log_i, log_f):
    """q, k [T, H, D], v [T, H, E], gates [T, H] -> [T, H, E]: S and n from zero, the running maximum m from 0."""
    T, H, D = q.shape
    E = v.shape[-1]
    S, n, m = torch.zeros(H, D, E), torch.zeros(H, D), torch.zeros(H)
    out = torch.zeros(T, H, E)
    for t in range(T):
        m_new = torch.maximum(log_f[t] + m, log_i[t])
        keep, add = torch.exp(log_f[t] + m - m_new), torch.exp(log_i[t] - m_new)
        m = m_new
        S = keep.view(H, 1, 1) * S + add.view(H, 1, 1) * (k[t].unsqueeze(-1) * v[t].unsqueeze(1))
        n = keep.view(H, 1) * n + add.view(H, 1) * k[t]
        num = (S * q[t].unsqueeze(-1)).sum(1)
        den = torch.maximum((n * q[t]).sum(-1).abs(), torch.exp(-m)) + 1e-6
        out[t] = num / den.view(H, 1)
    return out


def mlstm_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    h = h.float()
    q = (h @ w[pre + "q"].float().t()).view(T, H, D) * D ** -0.5
    k = (h @ w[pre + "k"].float().t()).view(T, H, D)
    v = (h @ w[pre + "v"].float().t()).view(T, H, E)
    o = rms(matrix_memory_scan(q, k, v, *memory_gates(h, w, pre, m)), eps)
    o = o.reshape(T, H * E) * w[pre + "norm"].float() * torch.sigmoid(h @ w[pre + "g"].float().t())
    return o @ w[pre + "o"].float().t()


def dense_feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str) -> torch.Tensor:
    h = h.float()
    a, b = h @ w[pre + "gate"].float().t(), h @ w[pre + "up"].float().t()
    return (torch.nn.functional.silu(a) * b) @ w[pre + "down"].float().t()


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], streams: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; `streams` collects the stream after every layer.  A sublayer reads the stream as it
    is and its OUTPUT is normed: x <- x + norm1(mixer(x)), x <- x + norm2(ff(x))."""
    eps = float(cfg["norm"]["eps"])
    x = w["embed"][torch.tensor(tokens)].float() * float(cfg["embedding"]["scale"])
    kept = {}                                                          # keys and values of every layer that makes its own
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        if layer["type"] == "attention":
            src = m.get("kv_from")
            if src is None:
                kept[i] = attention_kv(x, w, pre + "mix.", m, eps)
            y = attention_mixer(x, w, pre + "mix.", m, eps, kept[i if src is None else src])
        else:
            y = mlstm_mixer(x, w, pre + "mix.", m, eps)
        x = x + one_plus_norm(y, w[pre + "norm1"], eps)
        if layer.get("mlp") is not None:
            x = x + one_plus_norm(dense_feed_forward(x, w, pre + "mlp."), w[pre + "norm2"], eps)
        if streams is not None:
            streams.append(x.clone())
    return one_plus_norm(x, w["final.norm"], eps) @ w["embed"].float().t()


def forward_layers(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int]):
    """(logits, the stream after every layer)."""
    streams: list = []
    return forward(cfg, w, tokens, streams), streams


def random_weights(cfg: dict, seed: int = 0) -> Dict[str, torch.Tensor]:
    """Random bf16 weights under the checkpoint's names, scaled so that every sublayer matters and nothing saturates."""
    gen = torch.Generator().manual_seed(seed)
    W, V = cfg["width"], cfg["vocab"]

    def mat(n_out, n_in, gain=1.0):
        return (torch.randn(n_out, n_in, generator=gen) * gain / math.sqrt(n_in)).to(torch.bfloat16)

    def vec(n, scale=0.1, shift=0.0):
        return (torch.randn(n, generator=gen) * scale + shift).to(torch.bfloat16)

    w = {"embed": (torch.randn(V, W, generator=gen) / math.sqrt(W)).to(torch.bfloat16), "final.norm": vec(W)}
    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        H, D, E = m["heads"], m["dim"], m["vdim"]
        w[pre + "norm1"] = vec(W)
        w[pre + "mix.q"] = mat(H * D, W)
        w[pre + "mix.o"] = mat(W, H * E)
        if layer["type"] == "attention":
            G = m["kv_heads"]
            w[pre + "mix.q.norm"] = vec(D, 0.2, 1.5)
            w[pre + "mix.g"] = mat(H, W)
            if m.get("kv_from") is None:
                w[pre + "mix.k"] = mat(G * D, W)
                w[pre + "mix.v"] = mat(G * E, W)
                w[pre + "mix.k.norm"] = vec(D, 0.2, 1.5)
        else:
            # (keys that lean towards the token's own query: a read-out of near-zero q . k keeps its direction only up to rounding
            # once every head is brought to unit RMS, and the comparison would be one of signs)
            w[pre + "mix.k"] = (0.8 * w[pre + "mix.q"].float() + 0.6 * mat(H * D, W).float()).to(torch.bfloat16)
            w[pre + "mix.v"] = mat(H * E, W)
            w[pre + "mix.g"] = mat(H * E, W)
            w[pre + "mix.norm"] = vec(H * E, 0.1, 1.0)
            w[pre + "mix.i"] = mat(H, W)
            w[pre + "mix.i.b"] = vec(H, 0.5, -1.0)
            w[pre + "mix.f"] = mat(H, W)
            w[pre + "mix.f.b"] = vec(H, 1.0, 3.0)
        mlp = layer.get("mlp")
        if mlp is not None:
            w[pre + "norm2"] = vec(W)
            w[pre + "mlp.gate"] = mat(mlp["ff"], W)
            w[pre + "mlp.up"] = mat(mlp["ff"], W)
            w[pre + "mlp.down"] = mat(W, mlp["ff"])
    return w
