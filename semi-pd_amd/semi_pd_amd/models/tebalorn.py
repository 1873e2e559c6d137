"""Tebalorn: a parallel-block decoder -- mixer and feed-forward read ONE norm of the stream and their results are added together --
with an input per layer and token from a table of its own behind them, and three mixers: two linear attentions with decays and
rotary attention local to chunks of positions.

On an fp32 stream x (n(v) = v / sqrt(mean(v^2) + eps) * w):
    x = embed[token] * scale
    h = n_1(x);   x <- x + mixer(h) + ff(h)   (a layer may have no ff);
    x <- x + n_s(W_p (gelu(W_s x) * table[token, layer]));   logits = head n_f(x) * logit_scale
gla, H heads, keys D, values E: csrc/linear_attention.hip with a decay per key channel, sigmoid(A2 (A1 h) + b)^(1 / tau), queries
    times D^(-1/2); every head's read-out normed (one weight for all heads), times silu(W_g h), W_o.
lightning: the same recurrence with a constant decay per head, q, k and v through silu, no scale; one norm over all heads, times
    sigmoid(W_g h), W_o.
attention, H heads over G key/value heads: the first rot.dims elements of q and k turned in pairs (i, i + dims / 2) with stretched
    frequencies; a query sees the keys of its own chunk of mask.size positions; exp(sink_h) in the softmax denominator; W_o.
ff: W_down (relu(W_gate h) * W_up h); or a mixture of silu-gated experts (softmax over the chosen router logits) plus a shared one.

Because both sublayers read h and both results go into one sum, a layer has ONE input GEMM (the mixer's columns, then gate | up of
the dense feed-forward or of the shared expert) and ONE output GEMM over [mixer's heads | activated feed-forward].  Launches per
layer: GEMM in, the mixer (preparation + attention, or the recurrence) and the gated activation into the columns of the output
GEMM's input, [router, experts], GEMM out, sum into the stream (with the token's expert rows, unsummed) + a copy in the activation
type, GEMM(W_s), gelu * table row, GEMM(W_p), seam (norm, sum, the next layer's norm).
"""
from __future__ import annotations

import os
from dataclasses import dataclass, field
from typing import Any, Dict, List, Optional, Tuple

import torch
from torch import nn

from semi_pd_amd import ops
from semi_pd_amd.distributed import get_tensor_model_parallel_world_size
from semi_pd_amd.layers.attention_backend import RadixAttention
from semi_pd_amd.layers.basic import (LogitsProcessor, MergedColumnParallelLinear, OutputRMSNorm, ParallelLMHead, RowParallelLinear,
                                      StreamRMSNorm, VocabParallelEmbedding, dense_linear)
from semi_pd_amd.layers.moe import GatedMoE
from semi_pd_amd.models.penozen import stretched_frequencies
from semi_pd_amd.models.tibenex import RotationConfig


@dataclass
class ChannelDecayConfig:
    """Linear attention with a decay per key channel ("gla")."""
    heads: int
    dim: int
    vdim: int
    tau: float
    rank: int = 16                # size between the two matrices of the decay: the checkpoint's tensor shapes give it


@dataclass
class HeadDecayConfig:
    """Linear attention with a constant decay per head ("lightning")."""
    heads: int
    dim: int
    vdim: int
    decay: List[float]


@dataclass
class ChunkAttentionConfig:
    heads: int
    kv_heads: int
    dim: int
    vdim: int
    scale: float
    rot: RotationConfig
    chunk: int                    # positions of a chunk of the mask; 0: every earlier position is visible


@dataclass
class TebalornLayerConfig:
    kind: str                     # "gla" | "lightning" | "attention"
    mixer: Any
    ff: int = 0                   # dense feed-forward, or the shared expert next to `experts`; 0: none
    ff_act: str = "relu"          # of `ff`
    experts: int = 0              # 0: no mixture
    top: int = 0
    expert_ff: int = 0


def _known(d: Optional[dict], keys, where: str) -> dict:
    d = d or {}
    unknown = set(d) - set(keys)
    if unknown:
        raise ValueError(f"{where}: keys {sorted(unknown)} are not supported")
    return d


@dataclass
class TebalornConfig:
    vocab_size: int = 32000
    hidden_size: int = 1024
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    logit_scale: float = 1.0
    side_dim: int = 64            # a layer's part of the token-side table
    layers: List[TebalornLayerConfig] = field(default_factory=list)
    architectures: tuple = ("Tebalorn",)
    supports_float32 = True       # every kernel of its path is templated on the element type (ServerArgs --dtype float32)

    def __post_init__(self):
        if self.side_dim < 1:
            raise ValueError(f"Tebalorn: a token-side table of {self.side_dim} elements per layer")
        for i, lc in enumerate(self.layers):
            m, where = lc.mixer, f"Tebalorn layer {i}"
            if lc.experts and not 0 < lc.top <= lc.experts:
                raise ValueError(f"{where}: top {lc.top} of {lc.experts} experts")
            if lc.kind == "gla" and m.tau <= 0:
                raise ValueError(f"{where}: tau {m.tau}")
            if lc.kind == "lightning" and (len(m.decay) != m.heads or not all(0.0 <= d <= 1.0 for d in m.decay)):
                raise ValueError(f"{where}: decays {m.decay} of {m.heads} heads")
            if lc.kind == "attention":
                if m.heads % m.kv_heads:
                    raise ValueError(f"{where}: {m.heads} heads over {m.kv_heads} key/value heads")
                if m.rot.dims > m.dim:
                    raise ValueError(f"{where}: {m.rot.dims} turned elements of a head of {m.dim}")
                if m.chunk < 0:
                    raise ValueError(f"{where}: chunks of {m.chunk} positions")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    def read_tensor_shapes(self, shapes: Dict[str, Tuple[int, ...]]) -> None:
        """Sizes that only the checkpoint's tensors give: the rank of every per-channel decay."""
        for i, lc in enumerate(self.layers):
            if lc.kind == "gla" and f"l{i}.mix.a1" in shapes:
                lc.mixer.rank = int(shapes[f"l{i}.mix.a1"][0])

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "TebalornConfig":
        """The checkpoint's config.json: vocab, width, norm.eps, embedding.scale, logit_scale, token_side.dim and one entry per layer
        (type, mixer {...}, mlp {kind: dense, ff} or {kind: moe, expert {ff}, router {experts, top}, shared {ff}} or null)."""
        layers = []
        for i, entry in enumerate(d["layers"]):
            kind, m = entry.get("type"), entry["mixer"]
            where = f"Tebalorn layer {i}"
            if kind == "gla":
                _known(m, ("heads", "dim", "vdim", "tau"), where)
                mixer: Any = ChannelDecayConfig(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), tau=float(m["tau"]))
            elif kind == "lightning":
                _known(m, ("heads", "dim", "vdim", "decay"), where)
                mixer = HeadDecayConfig(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), decay=[float(x) for x in m["decay"]])
            elif kind == "attention":
                _known(m, ("heads", "kv_heads", "dim", "vdim", "scale", "rot", "mask"), where)
                mask = _known(m.get("mask"), ("size",), where + " mask")
                mixer = ChunkAttentionConfig(heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=int(m["dim"]),
                                             vdim=int(m.get("vdim", m["dim"])), scale=float(m["scale"]),
                                             rot=RotationConfig.from_dict(m.get("rot"), int(m["dim"]), where),
                                             chunk=int(mask.get("size") or 0))
            else:
                raise ValueError(f"{where}: mixer type {kind!r} is not supported (gla, lightning, attention)")
            lc = TebalornLayerConfig(kind, mixer)
            mlp = entry.get("mlp")
            if mlp is not None and mlp.get("kind") == "dense":
                _known(mlp, ("kind", "ff"), where + " feed-forward")
                lc.ff = int(mlp["ff"])
            elif mlp is not None and mlp.get("kind") == "moe":
                _known(mlp, ("kind", "expert", "router", "shared"), where + " feed-forward")
                lc.expert_ff = int(_known(mlp["expert"], ("ff",), where + " expert")["ff"])
                router = _known(mlp["router"], ("experts", "top"), where + " router")
                lc.experts, lc.top = int(router["experts"]), int(router["top"])
                if mlp.get("shared") is not None:
                    lc.ff, lc.ff_act = int(_known(mlp["shared"], ("ff",), where + " shared expert")["ff"]), "silu"
            elif mlp is not None:
                raise ValueError(f"{where}: feed-forward kind {mlp.get('kind')!r} is not supported (dense, moe)")
            layers.append(lc)
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)), logit_scale=float(d.get("logit_scale", 1.0)),
                   side_dim=int(d["token_side"]["dim"]), layers=layers)


def tebalorn_uniform(vocab_size: int, hidden_size: int, pattern: str, ff: int, heads: int, kv_heads: int, dim: int, vdim: int, chunk: int,
                     linear_heads: int, linear_dim: int, linear_vdim: int, side_dim: int, experts: int = 0, top: int = 0,
                     expert_ff: int = 0, shared_ff: int = 0, rank: int = 16, norm_eps: float = 1e-6) -> TebalornConfig:
    """A configuration from a pattern of layer kinds: 'g' decay per channel, 'l' decay per head, 'a' attention; an upper-case letter
    has the mixture instead of the dense feed-forward (benchmarks, tests)."""
    layers = []
    for ch in pattern:
        if ch in "gG":
            kind, mixer = "gla", ChannelDecayConfig(linear_heads, linear_dim, linear_vdim, 16.0, rank)
        elif ch in "lL":
            kind, mixer = "lightning", HeadDecayConfig(linear_heads, linear_dim, linear_vdim,
                                                       [1.0 - 2.0 ** (-3.0 - 6.0 * i / max(linear_heads, 1)) for i in range(linear_heads)])
        else:
            kind, mixer = "attention", ChunkAttentionConfig(heads, kv_heads, dim, vdim, dim ** -0.5, RotationConfig(dim, 10000.0), chunk)
        lc = TebalornLayerConfig(kind, mixer, ff)
        if ch.isupper():
            lc = TebalornLayerConfig(kind, mixer, shared_ff, "silu", experts, top, expert_ff)
        layers.append(lc)
    return TebalornConfig(vocab_size=vocab_size, hidden_size=hidden_size, norm_eps=norm_eps, embedding_scale=hidden_size ** 0.5,
                          logit_scale=1.0, side_dim=side_dim, layers=layers)


def pad8(n: int) -> int:
    """Rows of a merged projection's parts: brought to a multiple of 8 with zeros, so that every part starts on a 16-byte boundary."""
    return -(-n // 8) * 8


def mixer_parts(lc: TebalornLayerConfig) -> List[Tuple[str, int]]:
    """(checkpoint leaf, rows) of the mixer's parts of a layer's input projection, in order."""
    m = lc.mixer
    H, D, E = m.heads, m.dim, m.vdim
    if lc.kind == "attention":
        return [("q", H * D), ("k", m.kv_heads * D), ("v", m.kv_heads * E)]
    parts = [("q", H * D), ("k", H * D), ("v", H * E), ("g", H * E)]
    return parts + [("a1", m.rank)] if lc.kind == "gla" else parts


def _portions(forward_batch):
    """(q_start, q_len) of an extend batch, (None, None) of a decode batch: how the kernels find a row's request."""
    if forward_batch.forward_mode.is_decode():
        return None, None
    return forward_batch.extend_start_loc, forward_batch.extend_seq_lens


class TebalornLinearAttention(nn.Module):
    """Both linear attentions: what follows the input projection and comes before the output projection."""

    def __init__(self, lc: TebalornLayerConfig, offsets: Dict[str, int], eps: float, state_id: int, dtype):
        super().__init__()
        m = lc.mixer
        self.mc, self.kind, self.eps, self.state_id, self.offsets = m, lc.kind, eps, state_id, offsets
        H, D, E = m.heads, m.dim, m.vdim
        if lc.kind == "gla":
            self.a2 = nn.Parameter(torch.empty(H * D, m.rank, dtype=dtype), requires_grad=False)
            self.a2_bias = nn.Parameter(torch.zeros(H * D, dtype=torch.float32), requires_grad=False)
            self.out_norm = nn.Parameter(torch.ones(E, dtype=dtype), requires_grad=False)
        else:
            self.register_buffer("powers", ops.decay_powers(m.decay), persistent=False)
            self.out_norm = nn.Parameter(torch.ones(H * E, dtype=dtype), requires_grad=False)

    def forward(self, p: torch.Tensor, out: torch.Tensor, forward_batch, angles) -> None:
        m, o = self.mc, self.offsets
        q_start, q_len = _portions(forward_batch)
        if self.kind == "gla":
            how = dict(a_off=o["a1"], a2=self.a2, a2_bias=self.a2_bias, tau=m.tau)
        else:
            how = dict(powers=self.powers, qkv_silu=True)
        ops.linear_attention(p, [o[x] for x in ("q", "k", "v", "g")], m.heads, m.dim, m.vdim, m.dim ** -0.5 if self.kind == "gla" else 1.0,
                             self.out_norm, self.kind == "lightning", "silu" if self.kind == "gla" else "sigmoid", self.eps,
                             forward_batch.state_pool.get_state_buffer(self.state_id), forward_batch.state_indices,
                             forward_batch.seq_lens, q_start, q_len, out=out,
                             form=int(os.environ.get("SEMIPD_LINEAR_ATTENTION_FORM", "0")), **how)


class TebalornAttention(nn.Module):
    def __init__(self, lc: TebalornLayerConfig, offsets: Dict[str, int], region: int):
        super().__init__()
        m = lc.mixer
        self.mc, self.offsets = m, offsets
        self.sink = nn.Parameter(torch.zeros(m.heads, dtype=torch.float32), requires_grad=False)
        self.attn = RadixAttention(m.heads, m.dim, m.scale, m.kv_heads, region, v_head_dim=m.vdim, chunk_size=m.chunk)

    def forward(self, p: torch.Tensor, out: torch.Tensor, forward_batch, angles) -> None:
        m = self.mc
        k_buf, v_buf = forward_batch.token_to_kv_pool.get_kv_buffer(self.attn.layer_id)
        ops.head_norm_rope_kv_store(p, m.heads, m.kv_heads, m.dim, m.vdim, self.offsets["k"], self.offsets["v"], None, None, 0.0,
                                    angles.get(m.rot), m.rot.dims, None, k_buf, v_buf, forward_batch.out_cache_loc)
        forward_batch.attn_backend.forward_local(p[:, : m.heads * m.dim], self.attn, forward_batch, sink=self.sink, out=out)


class RotationAngles:
    """The angle tables of one forward pass: cos and sin of every row's position for each rotation the layers name, computed when
    first asked for."""

    def __init__(self, freqs: Dict[str, Tuple[torch.Tensor, float]], positions: torch.Tensor):
        self.freqs, self.positions = freqs, positions
        self.tables: Dict[str, torch.Tensor] = {}

    def get(self, rot: RotationConfig) -> Optional[torch.Tensor]:
        if rot.dims == 0:
            return None
        key = repr(rot)
        if key not in self.tables:
            freq, factor = self.freqs[key]
            self.tables[key] = ops.angle_table(self.positions, freq, factor)
        return self.tables[key]


class TokenSideInput(nn.Module):
    """What a layer's part of a token-side table adds to the stream: norm(W_p (gelu(W_s x) * table[token, part]))."""

    def __init__(self, hidden_size: int, dim: int, layer_id: int, eps: float, dtype):
        super().__init__()
        self.dim, self.col = dim, layer_id * dim
        self.gate = nn.Parameter(torch.empty(dim, hidden_size, dtype=dtype), requires_grad=False)
        self.proj = nn.Parameter(torch.empty(hidden_size, dim, dtype=dtype), requires_grad=False)
        self.norm = OutputRMSNorm(hidden_size, eps, 0.0, dtype)

    def forward(self, s: torch.Tensor, x: torch.Tensor, ids: torch.Tensor, table: torch.Tensor, next_norm: StreamRMSNorm) -> torch.Tensor:
        """s: the stream in the activation type; x: the fp32 stream (updated in place).  Returns next_norm(x)."""
        e = ops.gelu_mul_rows(dense_linear(s, self.gate), ids, table, self.col)
        return self.norm.seam(dense_linear(e, self.proj), x, next_norm)


class TebalornDecoderLayer(nn.Module):
    def __init__(self, config: TebalornConfig, layer_id: int, region: Optional[int], state_id: Optional[int], dtype):
        super().__init__()
        lc = config.layers[layer_id]
        W, eps = config.hidden_size, config.norm_eps
        parts = mixer_parts(lc) + ([("gate", lc.ff), ("up", lc.ff)] if lc.ff else [])
        sizes = [pad8(n) for _, n in parts]
        self.offsets = {leaf: sum(sizes[:i]) for i, (leaf, _) in enumerate(parts)}
        self.ff, self.ff_act = lc.ff, lc.ff_act
        self.o_size = lc.mixer.heads * lc.mixer.vdim
        self.in_proj = MergedColumnParallelLinear(W, sizes, params_dtype=dtype)
        self.out_proj = RowParallelLinear(self.o_size + lc.ff, W, params_dtype=dtype)      # columns: the heads, the feed-forward
        self.norm1 = StreamRMSNorm(W, eps, 0.0, dtype)
        if lc.kind == "attention":
            self.mix = TebalornAttention(lc, self.offsets, region)
        else:
            self.mix = TebalornLinearAttention(lc, self.offsets, eps, state_id, dtype)
        self.moe = GatedMoE(lc.experts, lc.top, W, lc.expert_ff, params_dtype=dtype) if lc.experts else None
        self.side = TokenSideInput(W, config.side_dim, layer_id, eps, dtype)

    def forward(self, x: torch.Tensor, h: torch.Tensor, forward_batch, ids, table, angles, next_norm: StreamRMSNorm) -> torch.Tensor:
        """x: the fp32 stream (updated in place); h = norm1(x) in the activation type.  Returns next_norm(x)."""
        p = self.in_proj(h)
        both = torch.empty((p.shape[0], self.o_size + self.ff), dtype=p.dtype, device=p.device)
        self.mix(p, both[:, : self.o_size], forward_batch, angles)
        if self.ff:
            gate, up = self.offsets["gate"], self.offsets["up"]
            ops.glu(p[:, gate:], self.ff, self.ff_act, out=both[:, self.o_size:], up_off=up - gate)
        rows = self.moe.expert_rows(h) if self.moe is not None else None
        s = ops.add_stream(self.out_proj(both), x, rows)
        return self.side(s, x, ids, table, next_norm)


class TebalornForCausalLM(nn.Module):
    def __init__(self, config: TebalornConfig, dtype=torch.bfloat16):
        super().__init__()
        if get_tensor_model_parallel_world_size() != 1:
            raise ValueError("Tebalorn runs on one GPU per replica (tensor parallelism over its per-layer head counts and its "
                             "recurrent state is not implemented)")
        if not config.layers:
            raise ValueError("Tebalorn: the configuration lists no layers")
        self.config = config
        W, L = config.hidden_size, len(config.layers)
        self.embed = VocabParallelEmbedding(config.vocab_size, W, params_dtype=dtype)
        self.side_table = nn.Parameter(torch.empty(config.vocab_size, L * config.side_dim, dtype=dtype), requires_grad=False)
        # pool regions: one per attention layer; state columns: one per linear-attention layer
        self._regions: List[ChunkAttentionConfig] = []
        self._state_widths: List[int] = []
        self._freqs: Dict[str, Tuple[str, float]] = {}
        layers = []
        for i, lc in enumerate(config.layers):
            region = state_id = None
            if lc.kind == "attention":
                region = len(self._regions)
                self._regions.append(lc.mixer)
                rot = lc.mixer.rot
                if rot.dims and repr(rot) not in self._freqs:
                    freq, factor = stretched_frequencies(rot.dims, rot.base, rot.scaling)
                    name = f"freq_{len(self._freqs)}"
                    self._freqs[repr(rot)] = (name, factor)
                    self.register_buffer(name, freq, persistent=False)
            else:
                state_id = len(self._state_widths)
                self._state_widths.append(lc.mixer.heads * lc.mixer.dim * lc.mixer.vdim)
            layers.append(TebalornDecoderLayer(config, i, region, state_id, dtype))
        self.layers = nn.ModuleList(layers)
        self.final_norm = StreamRMSNorm(W, config.norm_eps, 0.0, dtype)
        self.head = ParallelLMHead(config.vocab_size, W, params_dtype=dtype)
        self.logits_processor = LogitsProcessor(config.vocab_size, logit_scale=config.logit_scale)
        self.layer_probe = None      # tests: a callable (layer index, fp32 stream) run after every layer
        for p in self.parameters():
            p.requires_grad_(False)

    def post_load_weights(self):
        for layer in self.layers:
            if layer.moe is not None:
                layer.moe.post_load_weights()

    @property
    def kv_geometry(self):
        """One region per attention layer (a model without such layers keeps one token-sized dummy region)."""
        ms = self._regions
        if not ms:
            return dict(kind="mha", num_kv_heads=[1], head_dim=[8], v_head_dim=[8], num_heads=[1], num_layers=1, values_in_keys=[True])
        return dict(kind="mha", num_kv_heads=[m.kv_heads for m in ms], head_dim=[m.dim for m in ms], v_head_dim=[m.vdim for m in ms],
                    num_heads=[m.heads for m in ms], num_layers=len(ms))

    @property
    def state_geometry(self) -> List[int]:
        """Columns of a request's state row: per linear-attention layer the matrices S [H, D, E]."""
        return list(self._state_widths)

    @torch.no_grad()
    def forward(self, input_ids, positions, forward_batch):
        x = ops.embed_stream(input_ids, self.embed.weight, self.config.embedding_scale)
        angles = RotationAngles({k: (getattr(self, n), f) for k, (n, f) in self._freqs.items()}, forward_batch.positions)
        h = self.layers[0].norm1.read_stream(x)
        n = len(self.layers)
        for i, layer in enumerate(self.layers):
            h = layer(x, h, forward_batch, input_ids, self.side_table, angles, self.layers[i + 1].norm1 if i + 1 < n else self.final_norm)
            if self.layer_probe is not None:
                self.layer_probe(i, x)
        return self.logits_processor(input_ids, h, self.head, forward_batch)
