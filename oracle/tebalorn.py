"""Plain CPU statement of the Tebalorn decoder (TEST INFRASTRUCTURE ONLY, like oracle/model.py).

One function per mechanism, fp32 torch on the host, no cache, no state pool and no batching: a sequence is always
recomputed whole, attention is a dense [T, T] matrix per head, both linear recurrences are Python loops over the tokens and
every expert is a feed-forward of its own, so nothing here can share a fault with the engine's pools, kernels or scheduler.
Weights arrive as a dict of tensors under the checkpoint's own names (`embed`, `side.embed`, `l<i>.norm1`, `l<i>.mix.q`,
`l<i>.mix.a2.b`, `l<i>.mlp.e<j>.gate`, `l<i>.side.proj`, ..., `final.norm`, `head`); the configuration is the checkpoint's
config.json as a dict.

Notation: T tokens, W the model width, H heads, G key/value heads, D the key size, E the value size, X experts of which each
token takes K, P the size of a layer's part of the token-side table.
"""
from __future__ import annotations

import math
from typing import Dict, List, Optional

import torch


def linear(x: torch.Tensor, weight: torch.Tensor) -> torch.Tensor:
    return x.float() @ weight.float().t()


def rms(x: torch.Tensor, eps: float) -> torch.Tensor:
    x = x.float()
    return x / torch.sqrt((x * x).mean(-1, keepdim=True) + eps)


def rms_norm(x: torch.Tensor, weight: torch.Tensor, eps: float) -> torch.Tensor:
    return rms(x, eps) * weight.float()


def gelu_tanh(z: torch.Tensor) -> torch.Tensor:
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


# ---- per-channel decay -------------------------------------------------------------------------------------------------
def channel_decay(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict) -> torch.Tensor:
    """alpha [T, H, D] = sigmoid(A2 A1 h + b) ^ (1 / tau)."""
    z = linear(linear(h, w[pre + "a1"]), w[pre + "a2"]) + w[pre + "a2.b"].float()
    return torch.exp(torch.nn.functional.logsigmoid(z) / float(m["tau"])).view(h.shape[0], m["heads"], m["dim"])


def decayed_outer_products(q: torch.Tensor, k: torch.Tensor, v: torch.Tensor, alpha: torch.Tensor) -> torch.Tensor:
    """q, k, alpha [T, H, D], v [T, H, E] -> [T, H, E]: per head S (D x E) from zero, S <- alpha_t (rows) * S + k_t v_t^T, then
    the row S^T q_t."""
    T, H, D = q.shape
    S = torch.zeros(H, D, v.shape[-1])
    out = torch.zeros(T, H, v.shape[-1])
    for t in range(T):
        S = alpha[t].unsqueeze(-1) * S + k[t].unsqueeze(-1) * v[t].unsqueeze(1)
        out[t] = (S * q[t].unsqueeze(-1)).sum(1)
    return out


def gla_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    q = linear(h, w[pre + "q"]).view(T, H, D) * D ** -0.5
    k = linear(h, w[pre + "k"]).view(T, H, D)
    v = linear(h, w[pre + "v"]).view(T, H, E)
    o = rms_norm(decayed_outer_products(q, k, v, channel_decay(h, w, pre, m)), w[pre + "norm"], eps)
    o = o.reshape(T, H * E) * torch.nn.functional.silu(linear(h, w[pre + "g"]))
    return linear(o, w[pre + "o"])


def lightning_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float) -> torch.Tensor:
    """One constant decay per head, q, k and v through silu; the norm spans all heads."""
    T = h.shape[0]
    H, D, E = m["heads"], m["dim"], m["vdim"]
    silu = torch.nn.functional.silu
    q = silu(linear(h, w[pre + "q"])).view(T, H, D)
    k = silu(linear(h, w[pre + "k"])).view(T, H, D)
    v = silu(linear(h, w[pre + "v"])).view(T, H, E)
    decay = torch.tensor(m["decay"], dtype=torch.float64).float().view(1, H, 1).expand(T, H, D)
    o = rms_norm(decayed_outer_products(q, k, v, decay).reshape(T, H * E), w[pre + "norm"], eps)
    return linear(o * torch.sigmoid(linear(h, w[pre + "g"])), w[pre + "o"])


# ---- attention ---------------------------------------------------------------------------------------------------------
def yarn_frequencies(rot: dict):
    """(frequency of every pair, the factor on cos and sin)."""
    dims, base = int(rot["dims"]), float(rot["base"])
    f = torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)], dtype=torch.float64)
    sc = rot.get("scaling")
    if not sc:
        return f, 1.0

    def where(turns):
        return dims * math.log(sc["original"] / (2 * math.pi * turns)) / (2 * math.log(base))

    lo, hi = max(math.floor(where(sc["fast"])), 0), min(math.ceil(where(sc["slow"])), dims - 1)
    ramp = ((torch.arange(dims // 2, dtype=torch.float64) - lo) / max(hi - lo, 0.001)).clamp(0.0, 1.0)
    return f / sc["factor"] * ramp + f * (1 - ramp), 0.1 * math.log(sc["factor"]) + 1.0


def rotate_halves(x: torch.Tensor, rot: dict) -> torch.Tensor:
    """x [T, heads, D]: elements i and i + dims / 2 of the first rot['dims'] are a pair turned by position * frequency_i."""
    T, half = x.shape[0], int(rot["dims"]) // 2
    f, m = yarn_frequencies(rot)
    ang = torch.arange(T, dtype=torch.float32).view(T, 1, 1) * f.float()
    c, s = torch.cos(ang) * m, torch.sin(ang) * m
    x = x.float().clone()
    a, b = x[..., :half].clone(), x[..., half: 2 * half].clone()
    x[..., :half] = a * c - b * s
    x[..., half: 2 * half] = b * c + a * s
    return x


def chunk_mask(T: int, size: int) -> torch.Tensor:
    """[T, T] bool: j <= i inside the same chunk of `size` positions (0: every j <= i)."""
    i, j = torch.arange(T).view(T, 1), torch.arange(T).view(1, T)
    return (j <= i) & (i // size == j // size) if size else j <= i


def softmax_with_sink(s: torch.Tensor, sink: torch.Tensor) -> torch.Tensor:
    """s [H, T, T] (hidden entries -inf): exp(s) / (exp(sink_h) + sum exp(s)) over the last axis."""
    sink = sink.float().view(-1, 1, 1)
    top = torch.maximum(s.amax(-1, keepdim=True), sink)
    e = torch.exp(s - top)
    return e / (torch.exp(sink - top) + e.sum(-1, keepdim=True))


def attention_mixer(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, m: dict, eps: float) -> torch.Tensor:
    T = h.shape[0]
    H, G, D, E = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    q = rotate_halves(linear(h, w[pre + "q"]).view(T, H, D), m["rot"])
    k = rotate_halves(linear(h, w[pre + "k"]).view(T, G, D), m["rot"])
    v = linear(h, w[pre + "v"]).view(T, G, E)
    of = torch.arange(H) // (H // G)
    s = torch.einsum("ihd,jhd->hij", q, k[:, of]) * m["scale"]
    s = s.masked_fill(~chunk_mask(T, (m.get("mask") or {}).get("size", 0)).unsqueeze(0), float("-inf"))
    o = (softmax_with_sink(s, w[pre + "sink"]) @ v[:, of].transpose(0, 1)).transpose(0, 1)
    return linear(o.reshape(T, H * E), w[pre + "o"])


MIXERS = {"gla": gla_mixer, "lightning": lightning_mixer, "attention": attention_mixer}


# ---- feed-forward ------------------------------------------------------------------------------------------------------
def gated(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, act) -> torch.Tensor:
    return linear(act(linear(h, w[pre + "gate"])) * linear(h, w[pre + "up"]), w[pre + "down"])


def expert_weights(h: torch.Tensor, router: torch.Tensor, top: int) -> torch.Tensor:
    """[T, X]: softmax over each token's `top` largest router logits, 0 for the other experts."""
    z = linear(h, router)
    best = z.topk(top, -1)
    return torch.zeros_like(z).scatter(-1, best.indices, torch.softmax(best.values, -1))


def mixture(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, mlp: dict) -> torch.Tensor:
    silu = torch.nn.functional.silu
    p = expert_weights(h, w[pre + "router"], mlp["router"]["top"])
    y = torch.zeros(h.shape[0], w[pre + "e0.down"].shape[0])
    for e in range(mlp["router"]["experts"]):
        y = y + p[:, e: e + 1] * gated(h, w, f"{pre}e{e}.", silu)
    return y + gated(h, w, pre + "shared.", silu) if mlp.get("shared") else y


def feed_forward(h: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, mlp: Optional[dict]) -> torch.Tensor:
    if mlp is None:
        return torch.zeros_like(h)
    return gated(h, w, pre, torch.relu) if mlp["kind"] == "dense" else mixture(h, w, pre, mlp)


# ---- per-layer token input ----------------------------------------------------------------------------------------------
def side_input(x: torch.Tensor, e: torch.Tensor, w: Dict[str, torch.Tensor], pre: str, eps: float) -> torch.Tensor:
    """What the layer's part e [T, P] of the token-side table adds to the stream x behind the sublayers."""
    y = linear(gelu_tanh(linear(x, w[pre + "gate"])) * e.float(), w[pre + "proj"])
    return rms_norm(y, w[pre + "norm"], eps)


def forward(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int], streams: Optional[list] = None) -> torch.Tensor:
    """Logits [T, vocab] of one sequence; `streams` collects the stream after every layer.  Both sublayers of a layer read
    one norm of the stream."""
    eps, P = float(cfg["norm"]["eps"]), int(cfg["token_side"]["dim"])
    ids = torch.tensor(tokens)
    x = w["embed"][ids].float() * float(cfg["embedding"]["scale"])
    for i, layer in enumerate(cfg["layers"]):
        pre = f"l{i}."
        h = rms_norm(x, w[pre + "norm1"], eps)
        x = x + MIXERS[layer["type"]](h, w, pre + "mix.", layer["mixer"], eps) + feed_forward(h, w, pre + "mlp.", layer.get("mlp"))
        x = x + side_input(x, w["side.embed"][ids][:, i * P: (i + 1) * P], w, pre + "side.", eps)
        if streams is not None:
            streams.append(x.clone())
    return linear(rms_norm(x, w["final.norm"], eps), w["head"]) * float(cfg["logit_scale"])


def forward_layers(cfg: dict, w: Dict[str, torch.Tensor], tokens: List[int]):
    """(logits, the stream after every layer)."""
    streams: list = []
    return forward(cfg, w, tokens, streams), streams


def random_weights(cfg: dict, seed: int = 0, rank: int = 8) -> Dict[str, torch.Tensor]:
    """Random bf16 weights under the checkpoint's names, scaled so that every sublayer matters and nothing saturates.  rank: the
    size between the two matrices of a per-channel decay."""
    gen = torch.Generator().manual_seed(seed)
    W, V, P, L = cfg["width"], cfg["vocab"], cfg["token_side"]["dim"], len(cfg["layers"])

    def mat(n_out, n_in, gain=1.0):
        return (torch.randn(n_out, n_in, generator=gen) * gain / math.sqrt(n_in)).to(torch.bfloat16)

    def vec(n, scale=0.1, shift=1.0):
        return (torch.randn(n, generator=gen) * scale + shift).to(torch.bfloat16)

    w = {"embed": mat(V, W), "head": mat(V, W), "final.norm": vec(W),
         "side.embed": torch.randn(V, L * P, generator=gen).to(torch.bfloat16)}

    def ffn(pre, ff):
        w[pre + "gate"], w[pre + "up"], w[pre + "down"] = mat(ff, W), mat(ff, W), mat(W, ff)

    for i, layer in enumerate(cfg["layers"]):
        pre, m = f"l{i}.", layer["mixer"]
        H, D, E = m["heads"], m["dim"], m["vdim"]
        G = m.get("kv_heads", H)
        w[pre + "norm1"], w[pre + "side.norm"] = vec(W), vec(W, 0.05, 0.3)
        w[pre + "side.gate"], w[pre + "side.proj"] = mat(P, W), mat(W, P)
        w[pre + "mix.q"], w[pre + "mix.k"], w[pre + "mix.v"] = mat(H * D, W), mat(G * D, W), mat(G * E, W)
        w[pre + "mix.o"] = mat(W, H * E)
        if layer["type"] == "attention":
            w[pre + "mix.sink"] = vec(H, 0.5, 0.5)
        else:
            # (keys that lean towards the token's own query: a read-out of near-zero q . k keeps its direction only up to rounding
            # once it is brought to unit RMS, and the comparison would be one of signs)
            w[pre + "mix.k"] = (0.8 * w[pre + "mix.q"].float() + 0.6 * w[pre + "mix.k"].float()).to(torch.bfloat16)
            w[pre + "mix.g"] = mat(H * E, W)
            w[pre + "mix.norm"] = vec(E if layer["type"] == "gla" else H * E)
        if layer["type"] == "gla":
            w[pre + "mix.a1"], w[pre + "mix.a2"], w[pre + "mix.a2.b"] = mat(rank, W), mat(H * D, rank, 2.0), vec(H * D, 1.0, 1.0)
        mlp = layer.get("mlp")
        if mlp is None:
            continue
        if mlp["kind"] == "dense":
            ffn(pre + "mlp.", mlp["ff"])
            continue
        w[pre + "mlp.router"] = mat(mlp["router"]["experts"], W, 2.0)
        for e in range(mlp["router"]["experts"]):
            ffn(f"{pre}mlp.e{e}.", mlp["expert"]["ff"])
        if mlp.get("shared"):
            ffn(pre + "mlp.shared.", mlp["shared"]["ff"])
    return w
