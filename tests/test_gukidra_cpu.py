"""Host-side pieces of the Gukidra integration: configuration reader, checkpoint name mapping, the pool's block means next to
the rows, the columns of the state rows, and the plain model's own invariants (tests/test_gpu_gukidra.py compares the engine
with it)."""
import json

import pytest
import torch

from oracle import gukidra as O


def _attn(heads, kv_heads, dim, vdim, dims, size, pool, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 0.3, "rot": {"base": 700.0, "dims": dims},
         "mask": {"size": size, "pool": pool}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def _memory(heads, dim, vdim, cap):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _with(layer, ff):
    return dict(layer, mlp=None if ff is None else {"kind": "dense", "ff": ff})


CFG = {"architecture": "Gukidra", "vocab": 90, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 6.5},
       "layers": [_with(_memory(3, 6, 10, 7.5), 20), _with(_attn(4, 2, 12, 8, 6, 11, 4), None), _with(_memory(1, 16, 8, 3.0), None),
                  _with(_attn(6, 2, 12, 8, 6, 7, 3, kv_from=1), 12), _with(_attn(3, 1, 8, 12, 8, 5, 2), 8)]}


def test_config_reader_takes_every_size_from_the_file():
    from semi_pd_amd.model_loader import config_from_hf_dict
    c = config_from_hf_dict(CFG)
    assert type(c).__name__ == "GukidraConfig" and c.architectures == ("Gukidra",) and c.supports_float32
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embedding_scale, c.num_hidden_layers) == (90, 48, 1e-5, 6.5, 5)
    assert [l.kind for l in c.layers] == ["mlstm", "attention", "mlstm", "attention", "attention"]
    assert [l.ff for l in c.layers] == [20, 0, 0, 12, 8]
    a = c.layers[3].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.rot_dims, a.rot_base, a.window, a.pool, a.kv_from) == \
        (6, 2, 12, 8, 0.3, 6, 700.0, 7, 3, 1)
    assert c.layers[1].mixer.kv_from is None
    m = c.layers[0].mixer
    assert (m.heads, m.dim, m.vdim, m.gate_cap) == (3, 6, 10, 7.5)
    for path, value in ((("layers", 0, "type"), "delta"), (("layers", 3, "mlp", "kind"), "moe"), (("layers", 1, "mixer", "kv_heads"), 3),
                        (("layers", 1, "mixer", "rot", "dims"), 5), (("layers", 1, "mixer", "rot", "dims"), 14),
                        (("layers", 1, "mixer", "rot", "scaling"), {}), (("layers", 1, "mixer", "vdim"), 7),
                        (("layers", 1, "mixer", "mask", "first"), 2), (("layers", 1, "mixer", "mask", "size"), 0),
                        (("layers", 0, "mixer", "gate_cap"), 0.0), (("layers", 0, "mixer", "conv"), 4),
                        (("layers", 3, "mixer", "kv_from"), 0), (("layers", 3, "mixer", "kv_from"), 4), (("layers", 4, "mixer", "kv_from"), 3),
                        (("layers", 3, "mixer", "dim"), 8)):
        bad = json.loads(json.dumps(CFG))
        node = bad
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = value
        with pytest.raises(ValueError):
            config_from_hf_dict(bad)


def test_checkpoint_names_reach_every_parameter_and_merge_the_projections():
    from semi_pd_amd.model_executor.model_runner import build_model
    from semi_pd_amd.model_loader import config_from_hf_dict, load_weights
    c = config_from_hf_dict(CFG)
    w = O.random_weights(CFG, seed=2)
    with torch.device("cpu"):
        model = build_model(c, torch.float32)
    loaded = load_weights(model, c, w.items())
    params = dict(model.named_parameters())
    assert set(loaded) == set(params)
    # the merged projections, brought to a multiple of 8 rows with zeros
    for i, parts in ((0, "qkvgif"), (1, "qkvg"), (3, "qg")):
        full = torch.cat([w[f"l{i}.mix.{n}"] for n in parts]).float()
        got = params[f"layers.{i}.mix.in_proj.weight"]
        assert got.shape[0] % 8 == 0 and got.shape[0] - full.shape[0] < 8
        assert torch.equal(got[: full.shape[0]], full) and not got[full.shape[0]:].any()
    assert model.layers[0].mix.offsets == [0, 18, 36, 66, 96, 99] and model.layers[3].mix.g_off == 72 and model.layers[1].mix.g_off == 88
    pre = "layers.0.mix."
    assert torch.equal(params[pre + "i_bias"], w["l0.mix.i.b"].float()) and params[pre + "f_bias"].dtype == torch.float32
    assert torch.equal(params[pre + "out_norm"], w["l0.mix.norm"].float())
    assert torch.equal(params["layers.1.mix.q_norm"], w["l1.mix.q.norm"].float()) and params["layers.1.mix.k_norm"].shape == (12,)
    assert "layers.3.mix.k_norm" not in params
    assert torch.equal(params["layers.3.mlp.gate_up_proj.weight"], torch.cat([w["l3.mlp.gate"], w["l3.mlp.up"]]).float())
    assert torch.equal(params["layers.3.norm2.weight"], w["l3.norm2"].float()) and torch.equal(params["final_norm.weight"], w["final.norm"].float())
    assert not any(n.startswith("layers.1.norm2") or n.startswith("layers.1.mlp") for n in params)   # no feed-forward, no second norm
    # one pool region per layer with keys and values of its own, with the block sizes of all its readers
    geo = model.kv_geometry
    assert geo["num_kv_heads"] == [2, 1] and geo["head_dim"] == [12, 8] and geo["v_head_dim"] == [8, 12] and geo["block_means"] == [[4, 3], [2]]
    assert model.layers[3].mix.attn.layer_id == 0 and model.layers[3].mix.attn.pool == 3 and model.layers[3].mix.attn.window == 7
    assert model.state_geometry == [3 * 6 * 10 + 3 * 6 + 3, 16 * 8 + 16 + 1]
    for extra in ("l3.mix.k", "l3.mix.v", "l3.mix.k.norm", "l1.mlp.gate", "l1.mix.i.b", "l0.mix.q.norm", "l0.mix.sink", "l5.norm1", "head"):
        with pytest.raises(KeyError):
            load_weights(model, c, list(w.items()) + [(extra, torch.zeros(1))])
    short = dict(w)
    del short["l0.mix.f"]
    with pytest.raises(RuntimeError):
        load_weights(model, c, short.items())


def test_pool_with_block_means_next_to_the_rows():
    from semi_pd_amd.mem_cache.memory_pool import MHATokenToKVPool, mean_piece
    assert [mean_piece(d, p) for d, p in ((96, 16), (128, 16), (128, 8), (96, 3), (20, 1), (8, 64), (256, 2))] == [8, 8, 16, 32, 32, 8, 128]
    pool = MHATokenToKVPool(10, 1, torch.float32, [2, 1], [12, 64], 2, "cpu", v_head_dim=[8, 40], block_means=[[4, 3], [2]])
    assert not pool.uniform and pool.block_sizes == [[3, 4], [2]]
    block, km, vm = pool.get_block_means(1, 2)
    assert block == 2 and km.shape == (1, 11, 32) and vm.shape == (1, 11, 32) and pool.get_block_means(0, 0) is None
    assert pool.get_block_means(0, 4)[1].shape == (2, 11, 8) and pool.get_block_means(0, 3)[2].shape == (2, 11, 8)
    # every buffer lies in the one slab and none overlaps another
    bufs = pool.k_buffer + pool.v_buffer + [m for layer in pool.means for pair in layer.values() for m in pair]
    spans = sorted((t.data_ptr(), t.data_ptr() + t.numel() * 4) for t in bufs)
    assert len(spans) == 10 and all(a[1] <= b[0] for a, b in zip(spans, spans[1:]))
    assert spans[0][0] >= pool.slab.data_ptr() and spans[-1][1] <= pool.slab.data_ptr() + pool.slab.numel()
    k_bytes, v_bytes = pool.get_kv_size_bytes()
    assert k_bytes == 11 * (2 * 12 + 64 + 2 * 8 + 2 * 8 + 32) * 4 and v_bytes == 11 * (2 * 8 + 40 + 2 * 8 + 2 * 8 + 32) * 4
    plain = MHATokenToKVPool(10, 1, torch.float32, 2, 8, 3, "cpu")
    assert plain.uniform and plain.means == [{}, {}, {}]


def test_plain_model_invariants():
    w = O.random_weights(CFG, seed=3)
    g = torch.Generator().manual_seed(0)
    toks = torch.randint(0, CFG["vocab"], (40,), generator=g).tolist()
    full, layers = O.forward_layers(CFG, w, toks)
    assert full.shape == (40, 90) and len(layers) == 5
    torch.testing.assert_close(O.forward(CFG, w, toks[:17]), full[:17], rtol=1e-4, atol=1e-4)      # causal, blocks included
    # what a window of 5 with blocks of 3 shows position 12: tokens 8 .. 12, blocks [0, 2] and [3, 5]; [6, 8] reaches into it
    mask = O.pooled_window_mask(14, 5, 3)
    assert mask[12].nonzero().flatten().tolist() == [8, 9, 10, 11, 12, 14, 15] and mask[13].nonzero().flatten().tolist() == [9, 10, 11, 12, 13, 14, 15, 16]
    assert mask[0].nonzero().flatten().tolist() == [0] and not mask[6, 14:].any() and mask[7, 14:].tolist() == [True, False, False, False]
    # softmax with one more term of score 0
    s = torch.tensor([[0.0, float("-inf"), 2.0], [-50.0, -60.0, -70.0]])
    e = torch.exp(s)
    torch.testing.assert_close(O.softmax_with_one(s), e / (1 + e.sum(-1, keepdim=True)))
    # turning and turning back; a value seen from its own position comes out as it was, so shifting positions changes nothing
    x = torch.randn(6, 2, 12, generator=g)
    torch.testing.assert_close(O.turn_halves(O.turn_halves(x, 12, 50.0), 12, 50.0, back=True), x, rtol=1e-5, atol=1e-5)
    part = O.turn_halves(x, 8, 50.0)
    assert torch.equal(part[..., 8:], x[..., 8:]) and torch.equal(part[0], x[0])
    torch.testing.assert_close(part.norm(dim=-1), x.norm(dim=-1))
    torch.testing.assert_close(part[3, 0, 1], x[3, 0, 1] * torch.cos(torch.tensor(3 * 50.0 ** -0.25)) - x[3, 0, 5] * torch.sin(torch.tensor(3 * 50.0 ** -0.25)))
    # the memory: with forget gates open and equal input gates it sums k v^T; one token reads back its own value
    T, D = 5, 4
    k, v = torch.eye(T, D).view(T, 1, D), torch.randn(T, 1, 3, generator=g)
    q = torch.ones(T, 1, D)
    out = O.matrix_memory_scan(q, k, v, torch.zeros(T, 1), torch.zeros(T, 1))
    want = torch.stack([v[: min(t + 1, 4), 0].sum(0) / max(min(t + 1, 4), 1) for t in range(T)])
    torch.testing.assert_close(out[:, 0], want, rtol=1e-4, atol=1e-4)
    # a running maximum that starts at 0: a first token with a very negative input gate leaves next to nothing
    low = O.matrix_memory_scan(q[:1], k[:1], v[:1], torch.full((1, 1), -30.0), torch.full((1, 1), -1e-3))
    assert low.abs().max() < 1e-11
    # another layer's rows: changing layer 1's values moves layer 3 even when layer 1's own output is cut off
    w2 = dict(w)
    w2["l1.mix.o"] = torch.zeros_like(w["l1.mix.o"])
    w3 = dict(w2)
    w3["l1.mix.v"] = w["l1.mix.v"] * 2
    a, b = O.forward_layers(CFG, w2, toks)[1], O.forward_layers(CFG, w3, toks)[1]
    assert torch.equal(a[2], b[2]) and not torch.allclose(a[3], b[3])


def test_command_line_of_a_model_folder(tmp_path):
    """A Gukidra folder on the command line: the class comes from config.json; float32 is accepted (every kernel of the path
    takes it); the trace runner wants a device; a checkout without a library builds the sources this model calls."""
    import argparse
    from semi_pd_amd import _lib
    from semi_pd_amd.entrypoints import trace_replay
    from semi_pd_amd.server_args import add_cli_args, from_cli_args
    with open(tmp_path / "config.json", "w") as f:
        json.dump(CFG, f)
    ap = argparse.ArgumentParser()
    add_cli_args(ap)
    sa = from_cli_args(ap.parse_args(["--model-path", str(tmp_path), "--dtype", "float32", "--skip-tokenizer-init"]))
    assert type(sa.model_config).__name__ == "GukidraConfig" and sa.torch_dtype == torch.float32
    assert {"matrix_memory.hip", "attention_prep.hip", "local_attention.hip"} <= set(_lib.MODEL_SOURCES["Gukidra"])
    if not torch.cuda.is_available():
        assert trace_replay.main(["--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(tmp_path / "o"),
                                  "--max-tokens", "64"]) == 2
