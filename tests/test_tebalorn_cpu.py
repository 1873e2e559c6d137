"""Host-side pieces of the Tebalorn integration: configuration reader with sizes from tensor shapes, checkpoint name mapping into the
merged projections, pool regions and state columns, and the plain model's own invariants (tests/test_gpu_tebalorn.py compares the
engine with it)."""
import json

import pytest
import torch

from oracle import tebalorn as O

CFG = {"architecture": "Tebalorn", "vocab": 90, "width": 48, "norm": {"eps": 1e-5}, "embedding": {"scale": 6.5}, "logit_scale": 0.3,
       "token_side": {"dim": 10},
       "layers": [
           {"type": "gla", "mixer": {"heads": 3, "dim": 6, "vdim": 10, "tau": 8.0}, "mlp": {"kind": "dense", "ff": 20}},
           {"type": "attention", "mixer": {"heads": 4, "kv_heads": 2, "dim": 12, "vdim": 8, "scale": 0.3, "mask": {"size": 11},
                                           "rot": {"base": 700.0, "dims": 6, "scaling": {"factor": 3.0, "original": 64, "fast": 8.0, "slow": 0.5}}},
            "mlp": None},
           {"type": "lightning", "mixer": {"heads": 2, "dim": 16, "vdim": 8, "decay": [0.5, 0.99]},
            "mlp": {"kind": "moe", "router": {"experts": 5, "top": 2}, "expert": {"ff": 12}, "shared": {"ff": 28}}},
           {"type": "attention", "mixer": {"heads": 3, "kv_heads": 1, "dim": 8, "vdim": 12, "scale": 0.4, "mask": None, "rot": {"base": 90.0, "dims": 8}},
            "mlp": {"kind": "moe", "router": {"experts": 3, "top": 3}, "expert": {"ff": 7}}},
       ]}


def _config(d=CFG):
    from semi_pd_amd.model_loader import config_from_hf_dict
    return config_from_hf_dict(d)


def test_config_reader_takes_every_size_from_the_file():
    c = _config()
    assert type(c).__name__ == "TebalornConfig" and c.architectures == ("Tebalorn",) and c.supports_float32
    assert (c.vocab_size, c.hidden_size, c.norm_eps, c.embedding_scale, c.logit_scale, c.side_dim, c.num_hidden_layers) == \
        (90, 48, 1e-5, 6.5, 0.3, 10, 4)
    assert [l.kind for l in c.layers] == ["gla", "attention", "lightning", "attention"]
    assert [(l.ff, l.ff_act, l.experts, l.top, l.expert_ff) for l in c.layers] == \
        [(20, "relu", 0, 0, 0), (0, "relu", 0, 0, 0), (28, "silu", 5, 2, 12), (0, "relu", 3, 3, 7)]
    m = c.layers[0].mixer
    assert (m.heads, m.dim, m.vdim, m.tau) == (3, 6, 10, 8.0)
    assert c.layers[2].mixer.decay == [0.5, 0.99]
    a = c.layers[1].mixer
    assert (a.heads, a.kv_heads, a.dim, a.vdim, a.scale, a.chunk, a.rot.dims, a.rot.base) == (4, 2, 12, 8, 0.3, 11, 6, 700.0)
    assert a.rot.scaling == {"factor": 3.0, "original": 64.0, "fast": 8.0, "slow": 0.5}
    assert c.layers[3].mixer.chunk == 0 and c.layers[3].mixer.rot.scaling is None
    for path, value in ((("layers", 0, "type"), "delta"), (("layers", 0, "mlp", "kind"), "gated"), (("layers", 1, "mixer", "kv_heads"), 3),
                        (("layers", 1, "mixer", "rot", "dims"), 5), (("layers", 1, "mixer", "rot", "dims"), 14),
                        (("layers", 1, "mixer", "rot", "scaling"), {"factor": 2.0}), (("layers", 1, "mixer", "mask", "first"), 2),
                        (("layers", 1, "mixer", "mask", "size"), -1), (("layers", 0, "mixer", "tau"), 0.0), (("layers", 0, "mixer", "conv"), 4),
                        (("layers", 2, "mixer", "decay"), [0.5]), (("layers", 2, "mixer", "decay"), [0.5, 1.5]),
                        (("layers", 2, "mlp", "router", "top"), 6), (("layers", 2, "mlp", "router", "groups"), 2),
                        (("layers", 2, "mlp", "expert", "limit"), 7.0), (("layers", 2, "mlp", "shared", "gate"), True),
                        (("token_side", "dim"), 0)):
        bad = json.loads(json.dumps(CFG))
        node = bad
        for k in path[:-1]:
            node = node[k]
        node[path[-1]] = value
        with pytest.raises(ValueError):
            _config(bad)


def test_sizes_that_only_the_tensors_give(tmp_path):
    from safetensors.torch import save_file
    from semi_pd_amd.model_loader import load_hf_config, safetensors_shapes
    (tmp_path / "config.json").write_text(json.dumps(CFG))
    assert load_hf_config(str(tmp_path)).layers[0].mixer.rank == 16                # no tensors: a default
    w = O.random_weights(CFG, seed=1, rank=5)
    half = len(w) // 2
    for i, part in enumerate((list(w)[:half], list(w)[half:])):
        save_file({k: w[k] for k in part}, str(tmp_path / f"model-{i}.safetensors"))
    assert load_hf_config(str(tmp_path)).layers[0].mixer.rank == 5
    assert safetensors_shapes(str(tmp_path)) == {k: tuple(v.shape) for k, v in w.items()}


def test_checkpoint_names_reach_every_parameter_and_merge_the_projections():
    from semi_pd_amd.model_executor.model_runner import build_model
    from semi_pd_amd.model_loader import load_weights
    c = _config()
    w = O.random_weights(CFG, seed=2, rank=7)
    c.read_tensor_shapes({k: tuple(v.shape) for k, v in w.items()})
    with torch.device("cpu"):
        model = build_model(c, torch.float32)
    loaded = load_weights(model, c, w.items())
    params = dict(model.named_parameters())
    assert set(loaded) == set(params)
    # one input projection per layer: the mixer's parts, then gate | up, each on a multiple of 8 rows with zeros behind it
    for i, parts in ((0, ("mix.q", "mix.k", "mix.v", "mix.g", "mix.a1", "mlp.gate", "mlp.up")), (1, ("mix.q", "mix.k", "mix.v")),
                     (2, ("mix.q", "mix.k", "mix.v", "mix.g", "mlp.shared.gate", "mlp.shared.up")), (3, ("mix.q", "mix.k", "mix.v"))):
        got = params[f"layers.{i}.in_proj.weight"]
        offsets = model.layers[i].offsets
        at = 0
        for n in parts:
            t = w[f"l{i}.{n}"].float()
            assert offsets[n.rsplit(".", 1)[-1]] == at and at % 8 == 0
            assert torch.equal(got[at: at + t.shape[0]], t) and not got[at + t.shape[0]: at + t.shape[0] + -t.shape[0] % 8].any()
            at += t.shape[0] + -t.shape[0] % 8
        assert got.shape[0] == at
    # one output projection: the heads' columns, then the feed-forward's
    assert torch.equal(params["layers.0.out_proj.weight"], torch.cat([w["l0.mix.o"], w["l0.mlp.down"]], 1).float())
    assert torch.equal(params["layers.2.out_proj.weight"], torch.cat([w["l2.mix.o"], w["l2.mlp.shared.down"]], 1).float())
    assert torch.equal(params["layers.1.out_proj.weight"], w["l1.mix.o"].float())
    assert params["layers.0.mix.a2"].shape == (18, 7) and params["layers.0.mix.a2_bias"].dtype == torch.float32
    assert torch.equal(params["layers.0.mix.a2_bias"], w["l0.mix.a2.b"].float())
    assert torch.equal(params["layers.0.mix.out_norm"], w["l0.mix.norm"].float()) and params["layers.2.mix.out_norm"].shape == (16,)
    assert torch.equal(params["layers.1.mix.sink"], w["l1.mix.sink"].float())
    assert torch.equal(params["layers.2.moe.w13"][3], torch.cat([w["l2.mlp.e3.gate"], w["l2.mlp.e3.up"]]).float())
    assert torch.equal(params["layers.3.moe.w_down"][2], w["l3.mlp.e2.down"].float()) and params["layers.2.moe.router"].dtype == torch.float32
    assert torch.equal(params["side_table"], w["side.embed"].float()) and torch.equal(params["layers.3.side.norm.weight"], w["l3.side.norm"].float())
    geo = model.kv_geometry
    assert geo["num_kv_heads"] == [2, 1] and geo["head_dim"] == [12, 8] and geo["v_head_dim"] == [8, 12]
    assert [model.layers[i].mix.attn.layer_id for i in (1, 3)] == [0, 1] and model.layers[1].mix.attn.chunk_size == 11
    assert model.state_geometry == [3 * 6 * 10, 2 * 16 * 8] and model.layers[2].mix.state_id == 1
    for extra in ("l1.mlp.gate", "l1.mix.g", "l0.mix.sink", "l2.mix.a1", "l2.mlp.gate", "l0.mlp.router", "l3.mlp.e3.gate", "l3.mlp.shared.up", "l0.norm2",
                  "l0.side.bias", "l4.norm1", "bigram"):
        with pytest.raises(KeyError):
            load_weights(model, c, list(w.items()) + [(extra, torch.zeros(1))])
    for gone in ("l0.mix.a1", "l2.mlp.shared.up", "l0.mlp.down"):
        short = dict(w)
        del short[gone]
        with pytest.raises(RuntimeError):
            load_weights(model, c, short.items())


def test_powers_of_a_heads_decay():
    from semi_pd_amd import ops
    t = ops.decay_powers([0.999, 1.0, 0.0, 0.25])
    assert t.shape == (4, 65) and (t[:, 0] == 1).all() and (t[1] == 1).all() and (t[2, 1:] == 0).all()
    assert t[3, 3] == 0.25 ** 3 and t[0, 1] == torch.tensor(0.999)
    torch.testing.assert_close(t[0, 64], torch.tensor(float(torch.tensor(0.999)) ** 64))


def test_plain_model_invariants():
    w = O.random_weights(CFG, seed=3)
    g = torch.Generator().manual_seed(0)
    toks = torch.randint(0, CFG["vocab"], (40,), generator=g).tolist()
    full, layers = O.forward_layers(CFG, w, toks)
    assert full.shape == (40, 90) and len(layers) == 4
    torch.testing.assert_close(O.forward(CFG, w, toks[:17]), full[:17], rtol=1e-4, atol=1e-4)      # causal
    mask = O.chunk_mask(9, 4)
    assert mask[3].nonzero().flatten().tolist() == [0, 1, 2, 3] and mask[4].nonzero().flatten().tolist() == [4]
    assert mask[8].nonzero().flatten().tolist() == [8] and O.chunk_mask(9, 0)[8].all()
    # softmax with a sink: a term more in the denominator, however large or small
    s = torch.tensor([[[0.0, float("-inf"), 2.0], [-50.0, -60.0, -70.0]], [[1.0, 1.0, 1.0], [90.0, 0.0, 0.0]]])
    sink = torch.tensor([0.5, 80.0])
    e = torch.exp(s.double())
    torch.testing.assert_close(O.softmax_with_sink(s, sink), (e / (torch.exp(sink.double()).view(2, 1, 1) + e.sum(-1, keepdim=True))).float())
    # rotation: norms kept up to the factor, what lies behind dims passes, position 0 only scaled
    rot = {"dims": 8, "base": 50.0}
    x = torch.randn(6, 2, 12, generator=g)
    y = O.rotate_halves(x, rot)
    assert torch.equal(y[..., 8:], x[..., 8:]) and torch.equal(y[0], x[0])
    torch.testing.assert_close(y[..., :8].norm(dim=-1), x[..., :8].norm(dim=-1))
    torch.testing.assert_close(y[3, 0, 1], x[3, 0, 1] * torch.cos(torch.tensor(3 * 50.0 ** -0.25)) - x[3, 0, 5] * torch.sin(torch.tensor(3 * 50.0 ** -0.25)))
    f, m = O.yarn_frequencies(dict(rot, scaling={"factor": 4.0, "original": 40, "fast": 3.0, "slow": 0.1}))
    f0, _ = O.yarn_frequencies(rot)
    assert m > 1.1 and torch.allclose(f[0], f0[0]) and (f <= f0 + 1e-12).all() and (f >= f0 / 4 - 1e-12).all() and f[-1] < f0[-1]
    # the recurrence without decay sums k v^T; with a decay of 0 it forgets everything but the token itself
    T, D = 5, 4
    k, v = torch.eye(T, D).view(T, 1, D), torch.randn(T, 1, 3, generator=g)
    q = torch.ones(T, 1, D)
    out = O.decayed_outer_products(q, k, v, torch.ones(T, 1, D))
    torch.testing.assert_close(out[:, 0], torch.stack([v[: min(t + 1, 4), 0].sum(0) for t in range(T)]))
    torch.testing.assert_close(O.decayed_outer_products(q, k, v, torch.zeros(T, 1, D))[:4], v[:4])
    # expert weights: a softmax over the chosen logits only
    h, r = torch.randn(7, 5, generator=g), torch.randn(6, 5, generator=g)
    p = O.expert_weights(h, r, 2)
    assert ((p > 0).sum(-1) == 2).all() and torch.allclose(p.sum(-1), torch.ones(7))
    z = h @ r.t()
    torch.testing.assert_close(p.max(-1).values, torch.sigmoid(z.topk(2, -1).values[:, 0] - z.topk(2, -1).values[:, 1]))
    # both sublayers read the same norm: taking the mixer out leaves the feed-forward's part as it was
    w2 = dict(w, **{"l0.mix.o": torch.zeros_like(w["l0.mix.o"]), "l0.side.norm": torch.zeros_like(w["l0.side.norm"])})
    x0 = w["embed"][torch.tensor(toks)].float() * 6.5
    h0 = O.rms_norm(x0, w["l0.norm1"], 1e-5)
    torch.testing.assert_close(O.forward_layers(CFG, w2, toks)[1][0], x0 + O.feed_forward(h0, w, "l0.mlp.", CFG["layers"][0]["mlp"]))


def test_command_line_of_a_model_folder(tmp_path):
    """A Tebalorn folder on the command line: the class comes from config.json; float32 is accepted (every kernel of the path
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
    assert type(sa.model_config).__name__ == "TebalornConfig" and sa.torch_dtype == torch.float32
    assert {"linear_attention.hip", "attention_prep.hip", "local_attention.hip"} <= set(_lib.MODEL_SOURCES["Tebalorn"])
    if not torch.cuda.is_available():
        assert trace_replay.main(["--model", str(tmp_path), "--dtype", "bfloat16", "--out", str(tmp_path / "o"),
                                  "--max-tokens", "64"]) == 2
