"""Gukidra: a decoder that norms what its sublayers RETURN, mixes tokens by windowed attention with pooled blocks behind the
window or by a matrix memory with exponential gates, and lets attention layers read each other's cache.

On an fp32 stream x (n(v) = v / sqrt(mean(v^2) + eps) * (1 + w)):
    x = embed[token] * scale;   x <- x + n_1(mixer(x));   x <- x + n_2(ff(x))  (a layer may have no ff);   logits = embed n_f(x)
attention, H heads over G key/value heads, key size D, value size E:
    q and k to unit RMS per head times a weight all heads share, their first rot.dims elements turned by the position in pairs
    (i, i + dims / 2); the VALUES turned as well, over the whole head, and cached so.  A query sees the last `window`
    positions and, in the same softmax, one mean key and mean value for every block of `pool` positions that has left the
    window as a whole; the softmax denominator has 1 added.  A head's result is turned back by the query's own angles (so that
    it depends on distances only), times sigmoid((W_g x)_h), W_o.
    kv_from: the layer has queries only and reads the rows (and takes block means of its own block size) of an earlier layer.
mlstm, H heads, keys D, values E: csrc/matrix_memory.hip; every head's read-out to unit RMS, a weight, sigmoid(W_g x), W_o.

Launches per layer: GEMM(q | k | v | gate [| i | f]), norm + rotation + pool store (+ block means), attention with the turn and
the gate in its epilogue -- or the memory, division + norm + gate --, GEMM(o), seam (norm, sum, the stream in the activation
type), GEMM(gate | up) + silu * up, GEMM(down), seam.  Angle tables are computed once per pass and shared by the layers.
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
from semi_pd_amd.layers.basic import (LogitsProcessor, MergedColumnParallelLinear, OutputRMSNorm, RowParallelLinear, SiluAndMul,
                                      StreamRMSNorm, VocabParallelEmbedding, gate_up_silu)


@dataclass
class GukidraAttentionConfig:
    heads: int
    kv_heads: int
    dim: int                      # query / key size per head
    vdim: int                     # value size per head
    scale: float
    rot_dims: int                 # leading elements of a query / key head that are turned
    rot_base: float               # the values turn with it as well
    window: int                   # positions seen one by one; 0: all of them
    pool: int                     # positions of a block behind the window; 0: no blocks
    kv_from: Optional[int] = None  # the layer whose keys and values this one reads


@dataclass
class GukidraMemoryConfig:
    heads: int
    dim: int
    vdim: int
    gate_cap: float


@dataclass
class GukidraLayerConfig:
    kind: str                     # "attention" | "mlstm"
    mixer: Any
    ff: int = 0                   # 0: the layer has no feed-forward


def _known(d: Optional[dict], keys, where: str) -> dict:
    d = d or {}
    unknown = set(d) - set(keys)
    if unknown:
        raise ValueError(f"{where}: keys {sorted(unknown)} are not supported")
    return d


@dataclass
class GukidraConfig:
    vocab_size: int = 32000
    hidden_size: int = 1024
    norm_eps: float = 1e-6
    embedding_scale: float = 1.0
    layers: List[GukidraLayerConfig] = field(default_factory=list)
    architectures: tuple = ("Gukidra",)
    supports_float32 = True       # every kernel of its path is templated on the element type (ServerArgs --dtype float32)

    def __post_init__(self):
        for i, lc in enumerate(self.layers):
            m, where = lc.mixer, f"Gukidra layer {i}"
            if lc.kind != "attention":
                if m.gate_cap <= 0:
                    raise ValueError(f"{where}: gate cap {m.gate_cap}")
                continue
            if m.heads % m.kv_heads:
                raise ValueError(f"{where}: {m.heads} heads over {m.kv_heads} key/value heads")
            if m.rot_dims % 2 or not 0 <= m.rot_dims <= m.dim or m.vdim % 2:
                raise ValueError(f"{where}: {m.rot_dims} turned elements of a head of {m.dim}, value heads of {m.vdim}")
            if m.window < 0 or m.pool < 0 or (m.pool and not m.window):
                raise ValueError(f"{where}: window {m.window}, blocks of {m.pool}")
            if m.kv_from is None:
                continue
            src = self.layers[m.kv_from] if 0 <= m.kv_from < i else None
            if src is None or src.kind != "attention" or src.mixer.kv_from is not None:
                raise ValueError(f"{where}: kv_from {m.kv_from} is not an earlier attention layer with keys and values of its own")
            if (src.mixer.kv_heads, src.mixer.dim, src.mixer.vdim) != (m.kv_heads, m.dim, m.vdim):
                raise ValueError(f"{where}: key/value heads of layer {m.kv_from} have another shape")

    @property
    def num_hidden_layers(self) -> int:
        return len(self.layers)

    @classmethod
    def from_dict(cls, d: Dict[str, Any]) -> "GukidraConfig":
        """The checkpoint's config.json: vocab, width, norm.eps, embedding.scale and one entry per layer (type, mixer {...}, mlp
        {kind: dense, ff} or null)."""
        layers = []
        for i, entry in enumerate(d["layers"]):
            kind, m = entry.get("type"), entry["mixer"]
            where = f"Gukidra layer {i}"
            if kind == "attention":
                _known(m, ("heads", "kv_heads", "dim", "vdim", "scale", "rot", "mask", "kv_from"), where)
                rot = _known(m.get("rot"), ("base", "dims"), where + " rotation")
                mask = _known(m.get("mask"), ("size", "pool"), where + " mask")
                mixer: Any = GukidraAttentionConfig(
                    heads=int(m["heads"]), kv_heads=int(m.get("kv_heads", m["heads"])), dim=int(m["dim"]),
                    vdim=int(m.get("vdim", m["dim"])), scale=float(m["scale"]), rot_dims=int(rot.get("dims", m["dim"])),
                    rot_base=float(rot.get("base", 10000.0)), window=int(mask.get("size") or 0), pool=int(mask.get("pool") or 0),
                    kv_from=None if m.get("kv_from") is None else int(m["kv_from"]))
            elif kind == "mlstm":
                _known(m, ("heads", "dim", "vdim", "gate_cap"), where)
                mixer = GukidraMemoryConfig(heads=int(m["heads"]), dim=int(m["dim"]), vdim=int(m["vdim"]), gate_cap=float(m["gate_cap"]))
            else:
                raise ValueError(f"{where}: mixer type {kind!r} is not supported (attention, mlstm)")
            mlp = entry.get("mlp")
            if mlp is not None and mlp.get("kind", "dense") != "dense":
                raise ValueError(f"{where}: feed-forward kind {mlp.get('kind')!r} is not supported (dense only)")
            layers.append(GukidraLayerConfig(kind, mixer, ff=int(mlp["ff"]) if mlp is not None else 0))
        return cls(vocab_size=int(d["vocab"]), hidden_size=int(d["width"]), norm_eps=float(d["norm"]["eps"]),
                   embedding_scale=float((d.get("embedding") or {}).get("scale", 1.0)), layers=layers)


def gukidra_uniform(vocab_size: int, hidden_size: int, pattern: str, ff: int, heads: int, kv_heads: int, dim: int, vdim: int,
                    window: int, pool: int, memory_heads: int, memory_dim: int, memory_vdim: int, rot_dims: int = 0,
                    gate_cap: float = 15.0, norm_eps: float = 1e-6) -> GukidraConfig:
    """A configuration from a pattern of layer kinds: 'a' attention, 's' attention over the cache of the last 'a' layer, 'm' matrix
    memory (benchmarks, tests)."""
    layers: List[GukidraLayerConfig] = []
    last = None
    for i, ch in enumerate(pattern):
        if ch == "m":
            layers.append(GukidraLayerConfig("mlstm", GukidraMemoryConfig(memory_heads, memory_dim, memory_vdim, gate_cap), ff))
            continue
        layers.append(GukidraLayerConfig("attention", GukidraAttentionConfig(
            heads, kv_heads, dim, vdim, dim ** -0.5, rot_dims or dim, 10000.0, window, pool, last if ch == "s" else None), ff))
        if ch == "a":
            last = i
    return GukidraConfig(vocab_size=vocab_size, hidden_size=hidden_size, norm_eps=norm_eps, embedding_scale=1.0, layers=layers)


def _portions(forward_batch):
    """(q_start, q_len) of an extend batch, (None, None) of a decode batch: how the kernels find a row's request."""
    if forward_batch.forward_mode.is_decode():
        return None, None
    return forward_batch.extend_start_loc, forward_batch.extend_seq_lens


class GukidraAngles:
    """The angle tables of one forward pass: cos and sin of every row's position for each set of frequencies the layers name
    ((turned elements, base): the queries and keys, and the values), computed when first asked for."""

    def __init__(self, freqs: Dict[Tuple[int, float], torch.Tensor], positions: torch.Tensor):
        self.freqs, self.positions = freqs, positions
        self.tables: Dict[Tuple[int, float], torch.Tensor] = {}

    def get(self, dims: int, base: float) -> Optional[torch.Tensor]:
        if dims == 0:
            return None
        key = (dims, base)
        if key not in self.tables:
            self.tables[key] = ops.angle_table(self.positions, self.freqs[key])
        return self.tables[key]


class GukidraAttention(nn.Module):
    def __init__(self, hidden_size: int, mc: GukidraAttentionConfig, eps: float, region: int, block_sizes: List[int], dtype):
        """region: the pool region of the layer whose rows this one reads (its own, or kv_from's); block_sizes: the block sizes
        whose means this layer keeps up to date when it stores rows (its own and those of the layers that read its cache)."""
        super().__init__()
        self.mc, self.eps, self.own = mc, eps, mc.kv_from is None
        H, G, D, E = mc.heads, mc.kv_heads, mc.dim, mc.vdim
        sizes = [H * D, G * D, G * E, H] if self.own else [H * D, H]
        self.k_off, self.v_off = H * D, (H + G) * D
        self.g_off = sum(sizes[:-1])
        self.in_proj = MergedColumnParallelLinear(hidden_size, sizes + [-sum(sizes) % 8], params_dtype=dtype)
        self.out_proj = RowParallelLinear(H * E, hidden_size, params_dtype=dtype)
        self.q_norm = nn.Parameter(torch.ones(D, dtype=dtype), requires_grad=False)
        self.k_norm = nn.Parameter(torch.ones(D, dtype=dtype), requires_grad=False) if self.own else None
        self.register_buffer("sink", torch.zeros(H, dtype=torch.float32), persistent=False)     # exp(0): the one in the denominator
        self.block_sizes = list(block_sizes)
        self.attn = RadixAttention(H, D, mc.scale, G, region, v_head_dim=E, window=mc.window, pool=mc.pool)

    def forward(self, h: torch.Tensor, forward_batch, angles: GukidraAngles) -> torch.Tensor:
        mc = self.mc
        H, G, D, E = mc.heads, mc.kv_heads, mc.dim, mc.vdim
        p = self.in_proj(h)
        turn_qk, turn_v = angles.get(mc.rot_dims, mc.rot_base), angles.get(E, mc.rot_base)
        lid = self.attn.layer_id
        if self.own:
            pool = forward_batch.token_to_kv_pool
            k_buf, v_buf = pool.get_kv_buffer(lid)
            q_start, q_len = _portions(forward_batch)
            r2t = forward_batch.req_to_token_pool.req_to_token
            first = pool.get_block_means(lid, self.block_sizes[0]) if self.block_sizes else None
            ops.head_norm_rope_kv_store(p, H, G, D, E, self.k_off, self.v_off, self.q_norm, self.k_norm, self.eps, turn_qk, mc.rot_dims,
                                        turn_v, k_buf, v_buf, forward_batch.out_cache_loc, first, forward_batch.positions, r2t,
                                        forward_batch.req_pool_indices, forward_batch.seq_lens, q_start, q_len)
            for size in self.block_sizes[1:]:
                ops.block_means(k_buf, v_buf, pool.get_block_means(lid, size), r2t, forward_batch.req_pool_indices,
                                forward_batch.seq_lens, q_start, q_len, p.shape[0])
        else:
            ops.head_norm_rope_kv_store(p, H, 0, D, E, 0, 0, self.q_norm, None, self.eps, turn_qk, mc.rot_dims, None, None, None, None)
        o = forward_batch.attn_backend.forward_pooled_window(p[:, : H * D], self.attn, forward_batch, sink=self.sink,
                                                             gate=p[:, self.g_off: self.g_off + H], turn=turn_v)
        return self.out_proj(o)


class GukidraMemory(nn.Module):
    def __init__(self, hidden_size: int, mc: GukidraMemoryConfig, eps: float, state_id: int, dtype):
        super().__init__()
        self.mc, self.eps, self.state_id = mc, eps, state_id
        H, D, E = mc.heads, mc.dim, mc.vdim
        sizes = [H * D, H * D, H * E, H * E, H, H]
        self.offsets = [sum(sizes[:i]) for i in range(len(sizes))]
        self.in_proj = MergedColumnParallelLinear(hidden_size, sizes + [-sum(sizes) % 8], params_dtype=dtype)
        self.out_proj = RowParallelLinear(H * E, hidden_size, params_dtype=dtype)
        self.i_bias = nn.Parameter(torch.zeros(H, dtype=torch.float32), requires_grad=False)
        self.f_bias = nn.Parameter(torch.zeros(H, dtype=torch.float32), requires_grad=False)
        self.out_norm = nn.Parameter(torch.ones(H * E, dtype=dtype), requires_grad=False)

    def forward(self, h: torch.Tensor, forward_batch, angles) -> torch.Tensor:
        mc = self.mc
        q_start, q_len = _portions(forward_batch)
        o = ops.matrix_memory(self.in_proj(h), self.offsets, mc.heads, mc.dim, mc.vdim, self.i_bias, self.f_bias, mc.gate_cap,
                              self.out_norm, self.eps, forward_batch.state_pool.get_state_buffer(self.state_id),
                              forward_batch.state_indices, forward_batch.seq_lens, q_start, q_len,
                              form=int(os.environ.get("SEMIPD_MATRIX_MEMORY_FORM", "0")))
        return self.out_proj(o)


class GukidraMLP(nn.Module):
    def __init__(self, hidden_size: int, ff: int, dtype):
        super().__init__()
        self.gate_up_proj = MergedColumnParallelLinear(hidden_size, [ff, ff], params_dtype=dtype)
        self.down_proj = RowParallelLinear(ff, hidden_size, params_dtype=dtype)
        self.act_fn = SiluAndMul(any_width=True)

    def forward(self, x):
        return self.down_proj(gate_up_silu(x, self.gate_up_proj, self.act_fn))


class GukidraDecoderLayer(nn.Module):
    def __init__(self, config: GukidraConfig, layer_id: int, region: Optional[int], block_sizes, state_id: Optional[int], dtype):
        super().__init__()
        lc = config.layers[layer_id]
        W, eps = config.hidden_size, config.norm_eps
        if lc.kind == "attention":
            self.mix = GukidraAttention(W, lc.mixer, eps, region, block_sizes, dtype)
        else:
            self.mix = GukidraMemory(W, lc.mixer, eps, state_id, dtype)
        self.norm1 = OutputRMSNorm(W, eps, 1.0, dtype)
        self.mlp = GukidraMLP(W, lc.ff, dtype) if lc.ff else None
        self.norm2 = OutputRMSNorm(W, eps, 1.0, dtype) if lc.ff else None

    def forward(self, x: torch.Tensor, h: torch.Tensor, forward_batch, angles, last_norm: Optional[StreamRMSNorm]) -> torch.Tensor:
        """x: the fp32 stream (updated in place); h: x in the activation type.  Returns the new h (last_norm: that norm of x)."""
        y = self.mix(h, forward_batch, angles)
        if self.mlp is None:
            return self.norm1.seam(y, x, last_norm)
        return self.norm2.seam(self.mlp(self.norm1.seam(y, x)), x, last_norm)


class GukidraForCausalLM(nn.Module):
    def __init__(self, config: GukidraConfig, dtype=torch.bfloat16):
        super().__init__()
        if get_tensor_model_parallel_world_size() != 1:
            raise ValueError("Gukidra runs on one GPU per replica (tensor parallelism over its per-layer head counts and its "
                             "recurrent state is not implemented)")
        if not config.layers:
            raise ValueError("Gukidra: the configuration lists no layers")
        self.config = config
        W = config.hidden_size
        self.embed = VocabParallelEmbedding(config.vocab_size, W, params_dtype=dtype)
        # pool regions: one per attention layer with keys and values of its own, with the means of every block size its readers
        # name; state columns: one per matrix-memory layer
        regions = {i: n for n, i in enumerate(i for i, lc in enumerate(config.layers)
                                              if lc.kind == "attention" and lc.mixer.kv_from is None)}
        self._regions = [config.layers[i].mixer for i in regions]
        self._block_sizes: List[List[int]] = [[] for _ in regions]
        for i, lc in enumerate(config.layers):
            if lc.kind == "attention" and lc.mixer.pool:
                sizes = self._block_sizes[regions[i if lc.mixer.kv_from is None else lc.mixer.kv_from]]
                if lc.mixer.pool not in sizes:
                    sizes.append(lc.mixer.pool)
        self._state_widths: List[int] = []
        freq_keys, layers = [], []
        for i, lc in enumerate(config.layers):
            region = blocks = state_id = None
            if lc.kind == "attention":
                region = regions[i if lc.mixer.kv_from is None else lc.mixer.kv_from]
                blocks = self._block_sizes[region]
                freq_keys += [(lc.mixer.rot_dims, lc.mixer.rot_base), (lc.mixer.vdim, lc.mixer.rot_base)]
            else:
                state_id = len(self._state_widths)
                self._state_widths.append(ops.matrix_memory_state_width(lc.mixer.heads, lc.mixer.dim, lc.mixer.vdim))
            layers.append(GukidraDecoderLayer(config, i, region, blocks, state_id, dtype))
        self.layers = nn.ModuleList(layers)
        self._freq_names: Dict[Tuple[int, float], str] = {}
        for dims, base in freq_keys:
            if dims and (dims, base) not in self._freq_names:
                name = f"freq_{len(self._freq_names)}"
                self._freq_names[(dims, base)] = name
                self.register_buffer(name, torch.tensor([base ** (-2.0 * i / dims) for i in range(dims // 2)],
                                                        dtype=torch.float64).float(), persistent=False)
        self.final_norm = StreamRMSNorm(W, config.norm_eps, 1.0, dtype)
        self.logits_processor = LogitsProcessor(config.vocab_size)
        self.layer_probe = None      # tests: a callable (layer index, fp32 stream) run after every layer
        for p in self.parameters():
            p.requires_grad_(False)

    @property
    def kv_geometry(self):
        """One region per attention layer with keys and values of its own, and the block sizes whose means lie next to its rows
        (a model without such layers keeps one token-sized dummy region)."""
        ms = self._regions
        if not ms:
            return dict(kind="mha", num_kv_heads=[1], head_dim=[8], v_head_dim=[8], num_heads=[1], num_layers=1, values_in_keys=[True])
        return dict(kind="mha", num_kv_heads=[m.kv_heads for m in ms], head_dim=[m.dim for m in ms], v_head_dim=[m.vdim for m in ms],
                    num_heads=[m.heads for m in ms], num_layers=len(ms), block_means=[list(s) for s in self._block_sizes])

    @property
    def state_geometry(self) -> List[int]:
        """Columns of a request's state row: per matrix-memory layer S [H, D, E] | n [H, D] | m [H]."""
        return list(self._state_widths)

    @torch.no_grad()
    def forward(self, input_ids, positions, forward_batch):
        x, h = ops.embed_stream(input_ids, self.embed.weight, self.config.embedding_scale, want_copy=True)
        angles = GukidraAngles({k: getattr(self, n) for k, n in self._freq_names.items()}, forward_batch.positions)
        n = len(self.layers)
        for i, layer in enumerate(self.layers):
            h = layer(x, h, forward_batch, angles, self.final_norm if i + 1 == n else None)
            if self.layer_probe is not None:
                self.layer_probe(i, x)
        return self.logits_processor(input_ids, h, self.embed, forward_batch)
