"""Tebalorn on the GPU against the plain host statement (oracle/tebalorn.py): every mechanism alone, then whole models through
the replay scheduler (whole prompts, token-by-token decoding, portions down to two tokens, unequal requests side by side,
slots and state rows that change hands, planted keys at the edges of chunks, far tokens in the recurrences) and greedy generation
through the Engine."""
import json
import math
import os

import pytest
import torch

from oracle import tebalorn as O

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
TOL = {torch.float32: dict(rtol=3e-5, atol=3e-5), torch.bfloat16: dict(rtol=3e-2, atol=3e-2), torch.float16: dict(rtol=4e-3, atol=4e-3)}


def _batch(parts):
    """parts: [(slot, lo, hi)] -> (slots, lengths after the step, q_start, q_len) on the device."""
    slots = torch.tensor([s for s, _, _ in parts], device=DEV)
    lens = torch.tensor([hi for _, _, hi in parts], device=DEV)
    n = torch.tensor([hi - lo for _, lo, hi in parts], dtype=torch.int32, device=DEV)
    return slots, lens, (torch.cumsum(n, 0) - n).int(), n


# ----------------------------------------------------------------------------------------------- two sublayers into one stream
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("rows,width,n", [(1, 8, 0), (5, 100, 3), (37, 256, 1), (3, 4104, 6), (2, 9001, 2)])
def test_sum_into_the_stream(dtype, rows, width, n):
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(width)
    y, x = torch.randn(rows, width, generator=g).to(dtype), 3 * torch.randn(rows, width, generator=g)
    more = torch.randn(rows, n, width, generator=g).to(dtype) if n else None
    wide = torch.randn(rows, width + 16, generator=g).to(dtype).to(DEV)
    wide[:, 8: 8 + width] = y.to(DEV)
    want = x + y.float() + (more.float().sum(1) if n else 0.0)
    stream = x.to(DEV)
    out = ops.add_stream(wide[:, 8: 8 + width], stream, more.to(DEV) if n else None)
    torch.testing.assert_close(stream.cpu(), want, rtol=1e-6, atol=2e-6)                  # the stream keeps fp32
    assert torch.equal(out, stream.to(dtype))
    if n:
        stream = x.to(DEV)
        out = ops.add_stream(None, stream, more.to(DEV))
        torch.testing.assert_close(stream.cpu(), x + more.float().sum(1), rtol=1e-6, atol=2e-6)
    stream = x.to(DEV)
    assert torch.equal(ops.add_stream(None, stream, None, dtype=dtype), stream.to(dtype)) and torch.equal(stream.cpu(), x)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
def test_token_side_input(dtype):
    """gelu(W_s x) times the token's row of a layer's part of the table; then the whole input with its norm, and the next norm."""
    from semi_pd_amd import ops
    from semi_pd_amd.layers.basic import StreamRMSNorm
    from semi_pd_amd.models.tebalorn import TokenSideInput
    g = torch.Generator().manual_seed(1)
    for T, V, L, P, W in ((9, 40, 3, 24, 72), (33, 50, 2, 7, 50), (2, 11, 1, 1, 8), (5, 300, 4, 128, 2056)):
        z = (3 * torch.randn(T, P, generator=g)).to(dtype)
        z.view(-1)[0] = -9.0
        table = torch.randn(V, L * P, generator=g).to(dtype)
        ids = torch.randint(0, V, (T,), generator=g)
        ids[0], ids[-1] = V - 1, 0
        for layer in range(L):
            got = ops.gelu_mul_rows(z.to(DEV), ids.to(DEV), table.to(DEV), layer * P)
            want = O.gelu_tanh(z.float()) * table[ids].float()[:, layer * P: (layer + 1) * P]
            torch.testing.assert_close(got.float().cpu(), want, **TOL[dtype])
        layer = L - 1
        m = TokenSideInput(W, P, layer, 1e-3, dtype)
        w = {"gate": torch.randn(P, W, generator=g).to(dtype) / math.sqrt(W), "proj": torch.randn(W, P, generator=g).to(dtype),
             "norm": (1 + 0.2 * torch.randn(W, generator=g)).to(dtype)}
        m.gate.data, m.proj.data, m.norm.weight.data = w["gate"], w["proj"], w["norm"]
        nxt = StreamRMSNorm(W, 1e-5, 0.0, dtype)
        m, nxt = m.to(DEV), nxt.to(DEV)
        s = torch.randn(T, W, generator=g).to(dtype)
        x = s.float()
        want = x + O.side_input(s, table[ids][:, layer * P: (layer + 1) * P], w, "", 1e-3)
        stream = x.to(DEV)
        h = m(s.to(DEV), stream, ids.to(DEV), table.to(DEV), nxt)
        tol = dict(rtol=2e-4, atol=2e-4) if dtype == torch.float32 else dict(rtol=3e-2, atol=4e-2)
        torch.testing.assert_close(stream.cpu(), want, **tol)
        torch.testing.assert_close(h.float().cpu(), O.rms(stream.cpu(), 1e-5), **TOL[dtype])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("act", ["relu", "silu"])
@pytest.mark.parametrize("rows,ff,groups,off", [(3, 40, 1, 8), (17, 13, 1, 3), (5, 24, 6, 0), (9, 10, 4, 2), (200, 1032, 1, 16)])
def test_gated_activation_over_column_ranges(dtype, act, rows, ff, groups, off):
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(ff)
    gap = 8 if groups == 1 else 0                                      # up need not follow gate directly
    x = (2 * torch.randn(rows, off + groups * 2 * ff + gap, generator=g)).to(dtype)
    f = torch.relu if act == "relu" else torch.nn.functional.silu
    blocks = [x[:, off + e * 2 * ff:].float() for e in range(groups)]
    want = torch.cat([f(b[:, :ff]) * b[:, ff + gap: 2 * ff + gap] for b in blocks], 1)
    wide = torch.full((rows, groups * ff + 24), 7.0, dtype=dtype, device=DEV)
    xd = x.to(DEV)
    ops.glu(xd[:, off:], ff, act, out=wide[:, 8: 8 + groups * ff], up_off=ff + gap, groups=groups)
    torch.testing.assert_close(wide[:, 8: 8 + groups * ff].float().cpu(), want, **TOL[dtype])
    assert (wide[:, :8] == 7.0).all() and (wide[:, 8 + groups * ff:] == 7.0).all()
    if groups > 1:                                                     # with routing: the experts a row does not use come out zero
        k = 2
        ids = torch.stack([torch.randperm(groups, generator=g)[:k] for _ in range(rows)]).int()
        wts = torch.rand(rows, k, generator=g)
        full = torch.zeros(rows, groups).scatter(1, ids.long(), wts)
        got = ops.glu(xd[:, off:], ff, act, groups=groups, topk_weights=wts.to(DEV), topk_ids=ids.to(DEV))
        torch.testing.assert_close(got.float().cpu(), want * full.repeat_interleave(ff, 1), **TOL[dtype])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("T,W,F,E,K", [(5, 64, 32, 4, 2), (70, 72, 40, 12, 3), (33, 128, 128, 8, 8), (130, 50, 18, 5, 1), (600, 128, 64, 6, 3)])
def test_mixture_of_gated_experts(dtype, T, W, F, E, K):
    from semi_pd_amd.layers.moe import GatedMoE
    g = torch.Generator().manual_seed(W + E)
    h = torch.randn(T, W, generator=g).to(dtype)
    w = {"router": 2 * torch.randn(E, W, generator=g) / math.sqrt(W)}
    for e in range(E):
        w[f"e{e}.gate"], w[f"e{e}.up"] = ((torch.randn(F, W, generator=g) / math.sqrt(W)).to(dtype) for _ in range(2))
        w[f"e{e}.down"] = (torch.randn(W, F, generator=g) / math.sqrt(F)).to(dtype)
    m = GatedMoE(E, K, W, F, params_dtype=dtype)
    m.router.data = w["router"]
    m.w13.data = torch.stack([torch.cat([w[f"e{e}.gate"], w[f"e{e}.up"]]) for e in range(E)])
    m.w_down.data = torch.stack([w[f"e{e}.down"] for e in range(E)])
    m = m.to(DEV)
    m.post_load_weights()
    want = O.mixture(h, w, "", {"router": {"experts": E, "top": K}})
    rows = m.expert_rows(h.to(DEV))
    assert rows.shape[1] == (1 if m.side_by_side() else K)
    tol = dict(rtol=1e-4, atol=1e-4) if dtype == torch.float32 else dict(rtol=3e-2, atol=4e-2)
    torch.testing.assert_close(rows.float().sum(1).cpu(), want, **tol)
    torch.testing.assert_close(m(h.to(DEV)).float().cpu(), want, **tol)
    wts, ids = m.route(h.to(DEV))
    full = torch.zeros(T, E).scatter(1, ids.long().cpu(), wts.cpu())
    torch.testing.assert_close(full, O.expert_weights(h, w["router"], K), rtol=1e-4, atol=1e-5)
    assert (wts.sum(1) - 1).abs().max() < 1e-5


# ----------------------------------------------------------------------------------------------- rotation and chunk attention
def _scaling(factor=4.0, original=32.0, fast=2.0, slow=0.25):
    return {"factor": factor, "original": original, "fast": fast, "slow": slow}


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("H,G,D,E,rot,scaling", [(4, 2, 64, 48, 64, True), (3, 3, 20, 13, 10, False), (4, 1, 96, 160, 32, True), (1, 1, 8, 8, 0, False),
                                                 (6, 2, 48, 80, 16, True), (2, 1, 256, 24, 256, False)])
def test_rotation_without_norms_and_store(dtype, H, G, D, E, rot, scaling):
    """Queries in place, keys and values (as they are) into scattered slots; everything else untouched."""
    from semi_pd_amd import ops
    from semi_pd_amd.models.penozen import stretched_frequencies
    g = torch.Generator().manual_seed(D + E)
    spec = {"dims": rot, "base": 700.0, "scaling": _scaling() if scaling else None}
    T, N, width = 41, 90, (H + G) * D + G * E + 16
    width += -width % 8
    raw = torch.randn(T, width, generator=g).to(dtype)
    q, k = raw[:, : H * D].view(T, H, D), raw[:, H * D: (H + G) * D].reshape(T, G, D)
    v = raw[:, (H + G) * D: (H + G) * D + G * E].reshape(T, G, E)
    want_q, want_k = (O.rotate_halves(x, spec) if rot else x.float() for x in (q, k))
    pos, loc = torch.arange(T, device=DEV), (torch.randperm(N, generator=g)[:T] + 1)
    angles = None
    if rot:
        freq, factor = stretched_frequencies(rot, 700.0, spec["scaling"])
        assert (factor != 1.0) == scaling
        angles = ops.angle_table(pos, freq.to(DEV), factor)
    kp, vp = torch.full((N + 1, G, D), 3.0, dtype=dtype, device=DEV), torch.full((N + 1, G, E), 3.0, dtype=dtype, device=DEV)
    x = raw.to(DEV)
    ops.head_norm_rope_kv_store(x, H, G, D, E, H * D, (H + G) * D, None, None, 0.0, angles, rot, None, kp, vp, loc.to(DEV))
    torch.testing.assert_close(x[:, : H * D].float().cpu().view(T, H, D), want_q, **TOL[dtype])
    assert torch.equal(x[:, H * D:].cpu(), raw[:, H * D:])
    torch.testing.assert_close(kp.cpu()[loc].float(), want_k, **TOL[dtype])
    assert torch.equal(vp.cpu()[loc], v)
    free = [i for i in range(N + 1) if i not in set(loc.tolist())]
    assert (kp.cpu()[free] == 3.0).all() and (vp.cpu()[free] == 3.0).all()


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,E,chunk", [(4, 2, 64, 72, 50), (3, 1, 20, 12, 7), (8, 2, 96, 40, 64), (2, 2, 32, 160, 33), (4, 2, 64, 48, 0), (2, 1, 8, 8, 1)])
def test_chunk_attention_with_planted_keys(dtype, H, G, D, E, chunk):
    """Every query near an edge is lined up with the first key of its own chunk, the last key of the chunk in front, or its own key,
    whose value stands out: an edge that is one off, or a sink that is left out, moves the result by it.  The result goes into a
    column range of a wider row."""
    from semi_pd_amd.layers.attention_backend import HipAttnBackend, RadixAttention
    from semi_pd_amd.model_executor.forward_batch_info import ForwardMode
    g = torch.Generator().manual_seed(H * 1000 + D + chunk)
    T, other, scale = 210, 75, D ** -0.5
    sink = torch.linspace(-1.0, 3.0, H)
    seqs = {}
    for r, n in ((1, T), (0, other)):
        q, k, v = (torch.randn(n, h, d, generator=g) for h, d in ((H, D), (G, D), (G, E)))
        for x, i in enumerate(range(n - 1, max(n - 60, 0), -7)):
            start = i // chunk * chunk if chunk else 0
            j = (start, start - 1, i)[x % 3]
            if j >= 0:
                k[j] = 0.9 * q[i].view(G, H // G, D)[:, 0]
                v[j] = 4.0 if x % 2 else -4.0
        seqs[r] = [t.to(dtype) for t in (q, k, v)]
    perm = torch.randperm(400, generator=g) + 1
    table = torch.zeros(3, 256, dtype=torch.int32)
    table[1, :T], table[0, :other] = perm[:T].int(), perm[T: T + other].int()
    kp, vp = torch.zeros(401, G, D, dtype=dtype), torch.zeros(401, G, E, dtype=dtype)
    truth = {}
    for r, n in ((1, T), (0, other)):
        q, k, v = (x.float() for x in seqs[r])
        kp[table[r, :n].long()], vp[table[r, :n].long()] = seqs[r][1], seqs[r][2]
        of = torch.arange(H) // (H // G)
        s = (torch.einsum("ihd,jhd->hij", q, k[:, of]) * scale).masked_fill(~O.chunk_mask(n, chunk).unsqueeze(0), float("-inf"))
        truth[r] = (O.softmax_with_sink(s, sink) @ v[:, of].transpose(0, 1)).transpose(0, 1).reshape(n, H * E)
    kp, vp, table, sink = kp.to(DEV), vp.to(DEV), table.to(DEV), sink.to(DEV)
    layer = RadixAttention(H, D, scale, G, 0, v_head_dim=E, chunk_size=chunk)

    class Pool:
        get_key_buffer = staticmethod(lambda layer_id: kp)
        get_value_buffer = staticmethod(lambda layer_id: vp)

    backend = HipAttnBackend.__new__(HipAttnBackend)
    backend.req_to_token, backend.model_runner = table, None

    def check(parts, decode=False):
        rows, lens, start, n = _batch(parts)
        fb = type("FB", (), dict(forward_mode=ForwardMode.DECODE if decode else ForwardMode.EXTEND, token_to_kv_pool=Pool, req_pool_indices=rows,
                                 seq_lens=lens, extend_start_loc=start, extend_seq_lens=n,
                                 extend_seq_lens_cpu=[hi - lo for _, lo, hi in parts]))()
        q = torch.cat([seqs[r][0][lo:hi] for r, lo, hi in parts]).reshape(-1, H * D).to(DEV)
        both = torch.full((q.shape[0], H * E + 24), 9.0, dtype=dtype, device=DEV)
        backend.forward_local(q, layer, fb, sink=sink, out=both[:, : H * E])
        want = torch.cat([truth[r][lo:hi] for r, lo, hi in parts])
        torch.testing.assert_close(both[:, : H * E].float().cpu(), want, **TOL[dtype])
        assert (both[:, H * E:] == 9.0).all()

    check([(1, 0, T)])
    check([(0, 0, other), (1, 0, T)])
    check([(1, 100, T), (0, 74, 75)])                            # a cached prefix beside a single token
    check([(1, 207, 209), (0, 30, 75)])
    for i in range(T - 62, T, 3):
        check([(1, i, i + 1), (0, min(i - T + 62, 74), min(i - T + 62, 74) + 1)], decode=True)


# ----------------------------------------------------------------------------------------------- linear attention
def _linear_truth(p, sizes, H, D, E, alpha, silu, q_scale, nw, together, gate, eps, dtype):
    q, k, v, g = torch.split(p[:, : sum(sizes[:4])].float(), sizes[:4], 1)
    T = p.shape[0]
    if silu:                                                     # (held in the activation type, as a projection is)
        q, k, v = (torch.nn.functional.silu(x).to(dtype).float() for x in (q, k, v))
    o = O.decayed_outer_products(q.reshape(T, H, D) * q_scale, k.reshape(T, H, D), v.reshape(T, H, E), alpha)
    o = O.rms_norm(o.reshape(T, H * E), nw, eps) if together else O.rms_norm(o, nw, eps).reshape(T, H * E)
    return o * (torch.sigmoid(g) if gate == "sigmoid" else torch.nn.functional.silu(g))


def _forms(dtype, D, E):
    """Which forms take a shape: 0 picks one, 1 token by token, 2 the matrix-core form."""
    return [0, 1] + ([2] if dtype == torch.bfloat16 and D % 8 == 0 and E % 8 == 0 and D <= 256 else [])


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("kind,H,D,E,tau,shift", [
    ("channel", 3, 40, 24, 16.0, 1.0), ("channel", 2, 64, 72, 4.0, 0.0), ("channel", 4, 128, 96, 16.0, 2.0), ("channel", 1, 256, 160, 8.0, 3.0),
    ("channel", 2, 20, 12, 1.0, 1.0), ("channel", 1, 200, 33, 16.0, 1.0), ("channel", 2, 48, 136, 1.0, -6.0),
    ("head", 3, 40, 24, 0, 0), ("head", 4, 64, 64, 0, 0), ("head", 2, 128, 72, 0, 0), ("head", 5, 256, 40, 0, 0), ("head", 2, 13, 7, 0, 0),
    ("head", 1, 16, 1100, 0, 0)])
def test_linear_attention_over_portions_and_decode_steps(dtype, kind, H, D, E, tau, shift):
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(D * 7 + E)
    eps, T, rank = 1e-5, 170, 12 if D % 16 else 37
    sizes = [H * D, H * D, H * E, H * E, rank]
    offs = [sum(sizes[:i]) for i in range(5)]
    width = sum(sizes) + -sum(sizes) % 8
    together, gate = kind == "head", "sigmoid" if kind == "head" else "silu"
    nw = (1 + 0.2 * torch.randn(H * E if together else E, generator=g)).to(dtype)
    seqs = {s: torch.randn(n, width, generator=g).to(dtype) for s, n in ((1, T), (3, 40))}
    if kind == "channel":
        a2, bias = (torch.randn(H * D, rank, generator=g) * 2 / math.sqrt(rank)).to(dtype), shift + 1.5 * torch.randn(H * D, generator=g)
        if shift < 0:                                            # channels that are gone within a token beside slow ones
            bias[::5] = -40.0
            bias[1::5] = 6.0
        how = dict(a_off=offs[4], a2=a2.to(DEV), a2_bias=bias.to(DEV), tau=tau)
        q_scale = D ** -0.5

        def alpha(x):
            z = x[:, offs[4]: offs[4] + rank].float() @ a2.float().t() + bias
            return torch.exp(torch.nn.functional.logsigmoid(z) / tau).view(-1, H, D)
    else:
        decay = [0.999, 0.6, 1.0, 0.05, 0.9][:H]
        how = dict(powers=ops.decay_powers(decay).to(DEV), qkv_silu=True)
        q_scale = 1.0

        def alpha(x):
            return torch.tensor(decay).view(1, H, 1).expand(x.shape[0], H, D)
    want = {s: _linear_truth(x, sizes, H, D, E, alpha(x), kind == "head", q_scale, nw, together, gate, eps, dtype) for s, x in seqs.items()}
    seqs[2], want[2] = seqs[3], want[3]
    tol = dict(rtol=2e-4, atol=2e-4) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)
    for form in _forms(dtype, D, E):
        slab = torch.full((5, H * D * E + 8), 77.0, device=DEV)                        # rows full of something else
        state = slab[:, 4: 4 + H * D * E]

        def run(parts, decode=False):
            x = torch.cat([seqs[s][lo:hi] for s, lo, hi in parts]).to(DEV)
            slots, lens, start, n = _batch(parts)
            both = torch.full((x.shape[0], H * E + 16), 5.0, dtype=dtype, device=DEV)
            ops.linear_attention(x, offs[:4], H, D, E, q_scale, nw.to(DEV), together, gate, eps, state, slots, lens,
                                 None if decode else start, None if decode else n, out=both[:, : H * E], form=form, **how)
            torch.testing.assert_close(both[:, : H * E].float().cpu(), torch.cat([want[s][lo:hi] for s, lo, hi in parts]), **tol)
            assert (both[:, H * E:] == 5.0).all()

        run([(1, 0, T)])                                             # chunk by chunk
        run([(3, 0, 2), (1, 0, 70)])                                 # the row changes hands: what it held is not looked at
        run([(1, 70, 71), (3, 2, 3)], decode=True)
        run([(1, 71, 72), (3, 3, 4)])                                # single tokens in a prompt batch
        run([(3, 4, 6), (1, 72, 137)])
        run([(3, 6, 40)])
        for i in range(137, 150):
            run([(1, i, i + 1)], decode=True)
        run([(1, 150, T)])
        for i in range(20):                                          # from the first token on, one by one
            run([(2, i, i + 1)], decode=True)
        run([(2, 20, 40)])
        assert (slab[:, :4] == 77.0).all() and (slab[:, 4 + H * D * E:] == 77.0).all() and (slab[4] == 77.0).all()


@pytest.mark.parametrize("kind", ["channel", "head"])
def test_linear_attention_keeps_a_far_token(kind):
    """Slow decays and one token with a large key: 700 tokens on, in chunks and token by token, the read-out of a query lined up
    with that token's key is that token's value."""
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(0)
    H, D, E, T, rank = 1, 64, 32, 720, 8
    for dtype in (torch.bfloat16, torch.float32):
        sizes = [D, D, E, E, rank]
        offs = [sum(sizes[:i]) for i in range(5)]
        p = 0.05 * torch.randn(T, sum(sizes), generator=g)
        key, val = 4.0 + torch.rand(D, generator=g), 4.0 + 2 * torch.randn(E, generator=g)
        p[3, D: 2 * D], p[3, 2 * D: 2 * D + E] = 40 * key, val
        p[-8:, :D] = key
        p = p.to(dtype)
        nw = torch.ones(E, dtype=dtype, device=DEV)
        if kind == "channel":
            a2, bias = torch.zeros(D, rank, dtype=dtype), torch.full((D,), 6.0)
            how = dict(a_off=offs[4], a2=a2.to(DEV), a2_bias=bias.to(DEV), tau=16.0)
            alpha = torch.exp(torch.nn.functional.logsigmoid(bias) / 16.0).view(1, 1, D).expand(T, 1, D)
        else:
            how = dict(powers=ops.decay_powers([0.9997]).to(DEV), qkv_silu=True)
            alpha = torch.tensor(0.9997).view(1, 1, 1).expand(T, 1, D)
        args = (kind == "head", "sigmoid" if kind == "head" else "silu", 1e-6)
        want = _linear_truth(p, sizes, H, D, E, alpha, kind == "head", 1.0, nw.cpu(), *args, dtype)
        state = torch.zeros(2, D * E, device=DEV)
        slots, lens, start, n = _batch([(1, 0, 716)])
        ops.linear_attention(p[:716].to(DEV), offs[:4], H, D, E, 1.0, nw, *args, state, slots, lens, start, n, **how)
        for i in range(716, T):
            slots, lens, _, _ = _batch([(1, i, i + 1)])
            out = ops.linear_attention(p[i: i + 1].to(DEV), offs[:4], H, D, E, 1.0, nw, *args, state, slots, lens, None, None, **how).float().cpu()
            torch.testing.assert_close(out, want[i: i + 1], rtol=2e-2, atol=2e-2)
            gate = p[i, 2 * D + E: 2 * D + 2 * E].float()
            gate = torch.sigmoid(gate) if kind == "head" else torch.nn.functional.silu(gate)
            v = torch.nn.functional.silu(val) if kind == "head" else val
            assert torch.nn.functional.cosine_similarity(out[0] / gate, v, dim=0) > 0.99


@pytest.mark.parametrize("kind", ["channel", "head"])
@pytest.mark.parametrize("D,E,B", [(32, 16, 150), (128, 136, 70), (256, 136, 30)])
def test_linear_attention_over_many_requests_at_once(kind, D, E, B):
    """More requests in a prompt batch than a wave has lanes, of 1 to 130 tokens each: every chunk finds its request.  So many columns
    of state that workgroups take 64 of them (the last one of 136 keeps 8), first over fresh state rows, then behind them."""
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(4)
    H, rank = 2, 8
    sizes = [H * D, H * D, H * E, H * E, rank]
    offs = [sum(sizes[:i]) for i in range(5)]
    lens = [(7 * i * i) % 130 + 1 for i in range(B)]
    seqs = [torch.randn(n, sum(sizes), generator=g).to(torch.bfloat16) for n in lens]
    a2, bias = torch.randn(H * D, rank, generator=g).to(torch.bfloat16), torch.randn(H * D, generator=g)
    nw = torch.ones(E if kind == "channel" else H * E, dtype=torch.bfloat16)
    how = dict(a_off=offs[4], a2=a2.to(DEV), a2_bias=bias.to(DEV), tau=16.0) if kind == "channel" else \
        dict(powers=ops.decay_powers([0.9, 0.99]).to(DEV), qkv_silu=True)
    state = torch.full((B + 1, H * D * E), 3.0, device=DEV)
    args = (kind == "head", "silu" if kind == "channel" else "sigmoid", 1e-5)
    cut = [n * 2 // 3 if b % 3 else 0 for b, n in enumerate(lens)]                 # the first part of some, then the rest of all
    parts = [(b + 1, 0, cut[b]) for b in range(B) if cut[b]]
    where = _batch(parts)
    first = ops.linear_attention(torch.cat([seqs[s - 1][:hi] for s, _, hi in parts]).to(DEV), offs[:4], H, D, E, 1.0, nw.to(DEV), *args, state, *where,
                                 form=2, **how).float().cpu()
    slots, total, start, n = _batch([(b + 1, cut[b], lens[b]) for b in range(B)])
    rest = ops.linear_attention(torch.cat([x[c:] for x, c in zip(seqs, cut)]).to(DEV), offs[:4], H, D, E, 1.0, nw.to(DEV), *args, state, slots, total,
                                start, n, form=2, **how).float().cpu()
    at1 = at2 = 0
    for b in range(B):
        n1, n2 = cut[b], lens[b] - cut[b]
        if b % 11 == 0 or b > B - 8 or 60 < b < 68:
            x = seqs[b]
            z = x[:, offs[4]:].float() @ a2.float().t() + bias
            alpha = torch.exp(torch.nn.functional.logsigmoid(z) / 16.0).view(-1, H, D) if kind == "channel" else \
                torch.tensor([0.9, 0.99]).view(1, H, 1).expand(lens[b], H, D)
            want = _linear_truth(x, sizes, H, D, E, alpha, kind == "head", 1.0, nw, *args, torch.bfloat16)
            torch.testing.assert_close(torch.cat([first[at1: at1 + n1], rest[at2: at2 + n2]]), want, rtol=2e-2, atol=2e-2)
        at1, at2 = at1 + n1, at2 + n2


# ----------------------------------------------------------------------------------------------- whole models
def _attn(heads, kv_heads, dim, vdim, dims, size, base=300.0, scaling=None):
    rot = {"base": base, "dims": dims}
    if scaling:
        rot["scaling"] = scaling
    return {"type": "attention", "mixer": {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": 1.3 * dim ** -0.5, "rot": rot,
                                           "mask": {"size": size}}}


def _gla(heads, dim, vdim, tau=16.0):
    return {"type": "gla", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "tau": tau}}


def _lightning(decay, dim, vdim):
    return {"type": "lightning", "mixer": {"heads": len(decay), "dim": dim, "vdim": vdim, "decay": decay}}


def _dense(ff):
    return {"kind": "dense", "ff": ff}


def _moe(experts, top, ff, shared):
    return {"kind": "moe", "router": {"experts": experts, "top": top}, "expert": {"ff": ff}, "shared": None if shared is None else {"ff": shared}}


def _config(vocab, width, side, layers, eps=1e-5, scale=5.0, logit_scale=0.7):
    return {"architecture": "Tebalorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale},
            "logit_scale": logit_scale, "token_side": {"dim": side}, "layers": [dict(m, mlp=f) for m, f in layers]}


CONFIGS = {
    # every mixer with a dense feed-forward, a mixture or none; two rotations; a chunk of 40
    "mixed": _config(200, 96, 16, [(_gla(3, 40, 24, 4.0), _dense(64)), (_attn(4, 2, 64, 48, 32, 40, scaling=_scaling()), _moe(6, 2, 32, 48)),
                                   (_lightning([0.97, 0.5, 1.0], 32, 40), None), (_attn(2, 1, 32, 64, 32, 64), _dense(40)),
                                   (_lightning([0.999], 64, 72), _moe(5, 3, 24, 40)), (_gla(2, 64, 32), _moe(4, 2, 16, None))]),
    "minimal": _config(65, 8, 1, [(_gla(1, 8, 8), None), (_attn(1, 1, 8, 8, 8, 1), _dense(8)), (_lightning([0.9], 8, 8), _moe(1, 1, 8, 8))], scale=1.0,
                       logit_scale=1.0),
    "awkward": _config(77, 50, 5, [(_attn(3, 1, 20, 12, 10, 7), _dense(18)), (_gla(3, 13, 7, 1.0), _moe(3, 2, 10, 14)),
                                   (_lightning([0.8, 0.99], 9, 11), _dense(21)), (_attn(2, 2, 36, 10, 4, 13), None)], scale=3.3),
    "attention_only": _config(130, 64, 24, [(_attn(4, 4, 32, 32, 16, 16), _dense(64)), (_attn(8, 2, 32, 40, 32, 48, scaling=_scaling(2.0)), _moe(8, 4, 32, 32))]),
    "linear_only": _config(130, 64, 8, [(_gla(4, 16, 32), _dense(64)), (_lightning([0.9, 0.995], 128, 40), _moe(8, 8, 16, 16))]),
    "wide": _config(96, 128, 40, [(_gla(1, 256, 64), _dense(64)), (_attn(2, 1, 256, 256, 128, 32), None), (_lightning([0.98], 256, 128), _moe(4, 2, 128, 128))]),
}


def _write_checkpoint(path, cfg, seed, change=None, rank=8):
    from safetensors.torch import save_file
    w = O.random_weights(cfg, seed, rank)
    if change:
        change(w)
    with open(os.path.join(path, "config.json"), "w") as f:
        json.dump(cfg, f)
    save_file({k: v.contiguous() for k, v in w.items()}, os.path.join(path, "model.safetensors"))
    return w


def _scheduler(path, dtype, max_tokens, max_requests=4, graphs=True):
    from semi_pd_amd.entrypoints.engine import _build_runner
    from semi_pd_amd.managers.replay_scheduler import ReplayScheduler
    from semi_pd_amd.semi_pd.utils import InstanceRole
    from semi_pd_amd.server_args import ServerArgs
    sa = ServerArgs(model_path=path, load_format="auto", dtype=dtype, context_length=max_tokens, max_total_tokens=max_tokens,
                    max_running_requests=max_requests, cuda_graph_max_bs=max_requests, disable_cuda_graph=not graphs,
                    skip_tokenizer_init=True, enable_semi_pd=False)
    mr = _build_runner(sa, 0, 0, InstanceRole.OTHER, 29663, max_total_tokens=max_tokens)
    mr.init_attention_backend()
    mr.init_cuda_graphs()
    return ReplayScheduler(sa, mr)


def _tokens(n, vocab, seed):
    g = torch.Generator().manual_seed(seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def _run_schedule(sched, prompts, schedule):
    """schedule: steps of [(request name, token count)]; every position's logits are asked for.  Returns name -> [T, vocab]."""
    at = {n: 0 for n in prompts}
    got = {n: [] for n in prompts}
    for step in schedule:
        entries, end = [], []
        for name, count in step:
            lo, hi = at[name], at[name] + count
            entries.append({"id": name, "tokens": prompts[name][lo:hi], "want": list(range(count))})
            at[name] = hi
            if hi == len(prompts[name]):
                end.append(name)
        logits = sched.replay_step(entries, end).cpu()
        k = 0
        for name, count in step:
            got[name].append(logits[k: k + count])
            k += count
    assert all(at[n] == len(prompts[n]) for n in prompts)
    return {n: torch.cat(v) for n, v in got.items()}


def _rel_err(got, want, outliers=False):
    """Error of the positions (mean taken off, relative to the spread of the position's logits): the largest one; with
    `outliers` (16-bit runs) an outlier counts half as long as 97 of 100 positions stay below the figure returned (a router's close
    call, or the norm of a read-out that nearly cancels, passes 16-bit rounding on enlarged)."""
    d = (got - want) - (got - want).mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / want.std(-1)
    if not outliers:
        return e.max().item()
    return max(e.max().item() / 6, torch.quantile(e, 0.97).item())


LIMIT = {"float32": 4e-5, "bfloat16": 8e-2}


@pytest.fixture(scope="module", params=["float32", "bfloat16"])
def mixed_model(request, tmp_path_factory):
    path = str(tmp_path_factory.mktemp("tebalorn_mixed"))
    cfg = CONFIGS["mixed"]
    w = _write_checkpoint(path, cfg, seed=11)
    # a pool far smaller than the tokens that pass through it: slots, rows and state rows come back and are used again
    sched = _scheduler(path, request.param, max_tokens=448)
    lens = {"a": 150, "b": 1, "c": 97, "d": 2, "e": 64, "f": 131}
    prompts = {n: _tokens(k, cfg["vocab"], seed=ord(n)) for n, k in lens.items()}
    truth = {n: O.forward(cfg, w, t) for n, t in prompts.items()}
    return request.param, sched, prompts, truth, (cfg, w)


def _pools_are_whole(sched):
    assert sched.token_to_kv_pool_allocator.available_size() == 448 and sched.req_to_token_pool.available_size() == 5
    assert sched.model_runner.state_pool.available_size() == 4 and not sched.live


def test_every_layer_matches_the_plain_model(mixed_model):
    dtype, sched, prompts, truth, (cfg, w) = mixed_model
    t = prompts["c"]
    _, layers = O.forward_layers(cfg, w, t)
    seen = []
    sched.model_runner.model.layer_probe = lambda i, x: seen.append(x.detach().float().cpu().clone())
    try:
        sched.replay_step([{"id": "p", "tokens": t, "want": [0]}], ["p"])
    finally:
        sched.model_runner.model.layer_probe = None
    assert len(seen) == len(layers)
    for got, want in zip(seen, layers):
        err = (got - want).pow(2).mean(-1).sqrt() / want.pow(2).mean(-1).sqrt()
        if dtype == "float32":
            assert err.max().item() < 2e-5
        else:
            assert torch.quantile(err, 0.9).item() < 3e-2 and err.max().item() < 0.3
    _pools_are_whole(sched)


def test_whole_prompts_match_the_plain_model(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    for n in prompts:
        got = _run_schedule(sched, {n: prompts[n]}, [[(n, len(prompts[n]))]])
        assert _rel_err(got[n], truth[n], dtype != "float32") < LIMIT[dtype], n
    _pools_are_whole(sched)


def test_decoding_token_by_token_matches_the_prompt_pass(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    # from the very first token on (an empty state), and behind a prompt
    got = _run_schedule(sched, {"a": prompts["a"]}, [[("a", 1)]] * 150)
    assert _rel_err(got["a"], truth["a"], dtype != "float32") < LIMIT[dtype]
    got = _run_schedule(sched, {"f": prompts["f"]}, [[("f", 90)]] + [[("f", 1)]] * 41)
    assert _rel_err(got["f"], truth["f"], dtype != "float32") < LIMIT[dtype]
    _pools_are_whole(sched)


def test_portions_of_every_size_down_to_two(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    for cuts in ([2] * 75, [64, 2, 3, 17, 64], [1, 2, 1, 146], [149, 1], [39, 2, 39, 70], [7] * 21 + [3]):
        assert sum(cuts) == 150
        got = _run_schedule(sched, {"a": prompts["a"]}, [[("a", c)] for c in cuts])
        assert _rel_err(got["a"], truth["a"], dtype != "float32") < LIMIT[dtype], cuts
    _pools_are_whole(sched)


def test_unequal_requests_side_by_side_with_reuse(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    schedule = [[("a", 100), ("b", 1), ("c", 2)],
                [("a", 1), ("c", 60), ("d", 2)],             # b and d end: their rows, slots and state rows go back
                [("a", 1), ("c", 1), ("e", 33), ("f", 2)],   # e and f take them over
                [("c", 34), ("e", 1), ("f", 100)],           # a sits out a step
                [("a", 48), ("e", 30), ("f", 29)]]
    got = _run_schedule(sched, prompts, schedule)
    for n in prompts:
        assert _rel_err(got[n], truth[n], dtype != "float32") < LIMIT[dtype], n
    _pools_are_whole(sched)
    # all four live requests decode side by side through one captured graph
    four = {n: prompts[n][:64] for n in ("a", "c", "e", "f")}
    got = _run_schedule(sched, four, [[(n, 40) for n in four]] + [[(n, 1) for n in four]] * 24)
    for n in four:
        assert _rel_err(got[n], truth[n][:64], dtype != "float32") < LIMIT[dtype], n
    _pools_are_whole(sched)


def test_logits_do_not_depend_on_the_cut_or_the_neighbours(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    alone = _run_schedule(sched, {"c": prompts["c"]}, [[("c", 97)]])["c"]
    cut = _run_schedule(sched, {"c": prompts["c"], "e": prompts["e"]}, [[("c", 50), ("e", 64)], [("c", 47)]])["c"]
    assert _rel_err(cut, alone, dtype != "float32") < (5e-5 if dtype == "float32" else 8e-2)


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name,rank", [("minimal", 1), ("awkward", 3), ("attention_only", 8), ("linear_only", 40), ("wide", 16)])
def test_other_sizes_and_orders(name, rank, dtype, tmp_path):
    cfg = CONFIGS[name]
    w = _write_checkpoint(str(tmp_path), cfg, seed=5, rank=rank)
    sched = _scheduler(str(tmp_path), dtype, max_tokens=256)
    prompts = {"x": _tokens(90, cfg["vocab"], 1), "y": _tokens(37, cfg["vocab"], 2)}
    truth = {n: O.forward(cfg, w, t) for n, t in prompts.items()}
    got = _run_schedule(sched, prompts, [[("x", 60), ("y", 2)], [("x", 1), ("y", 30)], [("x", 1), ("y", 1)], [("x", 28), ("y", 4)]])
    for n in prompts:
        assert _rel_err(got[n], truth[n], dtype != "float32") < LIMIT[dtype], n
    got = _run_schedule(sched, {"x": prompts["x"]}, [[("x", 70)]] + [[("x", 1)]] * 20)
    assert _rel_err(got["x"], truth["x"], dtype != "float32") < LIMIT[dtype]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_padded_rows_of_a_decode_graph_leave_the_pools_alone(dtype, tmp_path):
    """Three requests decode through a graph captured for four: the padded row must not touch what a live request holds."""
    cfg = CONFIGS["linear_only"]
    w = _write_checkpoint(str(tmp_path), cfg, seed=6)
    sched = _scheduler(str(tmp_path), dtype, max_tokens=256)
    assert 3 not in sched.model_runner.graph_runner.capture_bs and 4 in sched.model_runner.graph_runner.capture_bs
    prompts = {n: _tokens(k, cfg["vocab"], i) for i, (n, k) in enumerate((("x", 60), ("y", 45), ("z", 50)))}
    got = _run_schedule(sched, prompts, [[("x", 30), ("y", 15), ("z", 20)]] + [[("x", 1), ("y", 1), ("z", 1)]] * 30)
    for n in prompts:
        assert _rel_err(got[n], O.forward(cfg, w, prompts[n]), dtype != "float32") < LIMIT[dtype], n


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_eager_decode_steps_and_the_plain_kernel_forms(dtype, tmp_path, monkeypatch):
    """Without captured graphs, the attention a wave per row, the recurrences token by token, the experts side by side."""
    monkeypatch.setenv("SEMIPD_LOCAL_ATTN_FORM", "1")
    monkeypatch.setenv("SEMIPD_LINEAR_ATTENTION_FORM", "1")
    monkeypatch.setenv("SEMIPD_MOE_SIDE_BY_SIDE", "1")
    cfg = CONFIGS["mixed"]
    w = _write_checkpoint(str(tmp_path), cfg, seed=8)
    sched = _scheduler(str(tmp_path), dtype, max_tokens=256, graphs=False)
    prompts = {"x": _tokens(80, cfg["vocab"], 1), "y": _tokens(50, cfg["vocab"], 2)}
    got = _run_schedule(sched, prompts, [[("x", 40), ("y", 10)]] + [[("x", 1), ("y", 1)]] * 40)
    for n in prompts:
        assert _rel_err(got[n], O.forward(cfg, w, prompts[n]), dtype != "float32") < LIMIT[dtype], n


def test_a_far_token_decides_the_logits(tmp_path):
    """Slow decays: a token that only the recurrences' states still hold has to change the last position's logits in the engine
    exactly as in the plain model, in the prompt pass, over portions and when decoding; so has a token at the start of the last
    position's attention chunk."""
    cfg = _config(96, 64, 8, [(_gla(2, 32, 32), _dense(64)), (_lightning([0.9995, 0.99], 32, 32), None), (_attn(2, 1, 32, 32, 32, 690), None)])

    def slow(w):
        w["l0.mix.a2.b"] += 4.0
        w["l2.mix.q"] *= 3.0

    w = _write_checkpoint(str(tmp_path), cfg, seed=3, change=slow)
    sched = _scheduler(str(tmp_path), "float32", max_tokens=1408, max_requests=2)
    t = _tokens(700, 96, 9)
    want = O.forward(cfg, w, t)
    moved = []
    for j in (5, 333, 689, 690):
        t2 = list(t)
        t2[j] = (t2[j] + 17) % 96
        moved.append(((O.forward(cfg, w, t2)[-1] - want[-1]).abs().max().item(), j, t2))
    assert moved[0][0] > 1e-3 and min(m[0] for m in moved[2:]) > 1e-3
    for seq in (t, moved[0][2], moved[3][2]):
        truth = O.forward(cfg, w, seq)
        got = _run_schedule(sched, {"p": seq}, [[("p", 640)], [("p", 2)]] + [[("p", 1)]] * 58)
        assert _rel_err(got["p"], truth) < 2 * LIMIT["float32"]
        got = _run_schedule(sched, {"p": seq}, [[("p", 700)]])
        assert _rel_err(got["p"], truth) < 2 * LIMIT["float32"]


def test_long_prompt_and_long_decoding(tmp_path):
    """600 tokens in one portion (many tiles of the prompt attention, many chunks of the recurrences), then 200 decode steps, in
    fp32 against the plain model."""
    cfg = CONFIGS["mixed"]
    w = _write_checkpoint(str(tmp_path), cfg, seed=31)
    sched = _scheduler(str(tmp_path), "float32", max_tokens=832, max_requests=2)
    t = _tokens(800, cfg["vocab"], 77)
    got = _run_schedule(sched, {"p": t}, [[("p", 600)]] + [[("p", 1)]] * 200)
    assert _rel_err(got["p"], O.forward(cfg, w, t)) < LIMIT["float32"]


def _check_generation(cfg, w, prompts, outs, steps):
    exact = total = 0
    for p, o in zip(prompts, outs):
        assert len(o) == steps
        logits = O.forward(cfg, w, p + o)
        for i, tok in enumerate(o):
            row = logits[len(p) + i - 1]
            assert row[tok] >= row.max() - 0.3 * row.std(), (len(p), i)
            exact += int(row.argmax().item() == tok)
            total += 1
    assert exact >= 0.9 * total


def test_greedy_generation_through_the_engine(tmp_path):
    """Prompts of unequal length through Engine.generate (the unified scheduler: chunked prefill, decode graphs, sampler):
    every generated token is the plain model's argmax given the tokens before it, or within a small margin of it."""
    from semi_pd_amd.entrypoints.engine import Engine
    from semi_pd_amd.managers.io_struct import SamplingParams
    from semi_pd_amd.server_args import ServerArgs
    cfg = CONFIGS["mixed"]
    w = _write_checkpoint(str(tmp_path), cfg, seed=21)
    prompts = [_tokens(n, cfg["vocab"], seed=n) for n in (3, 70, 33, 1, 120)]
    sa = ServerArgs(model_path=str(tmp_path), load_format="auto", dtype="bfloat16", context_length=256, max_total_tokens=1024,
                    max_running_requests=8, cuda_graph_max_bs=8, chunked_prefill_size=64, skip_tokenizer_init=True)
    eng = Engine(sa)
    try:
        outs = eng.generate(prompts, SamplingParams(max_new_tokens=24, ignore_eos=True), timeout=300)
    finally:
        eng.shutdown()
    _check_generation(cfg, w, prompts, outs, 24)


def test_greedy_generation_through_the_semi_pd_engine(tmp_path):
    """The same through a prefill and a decode process on one GPU: the rows of every attention layer, the slab of state rows and every
    parameter reach the prefill process through IPC handles; prompts are cut into 48-token portions in the prefill process and
    decoded in the other."""
    from semi_pd_amd.entrypoints.engine import Engine
    from semi_pd_amd.managers.io_struct import SamplingParams
    from semi_pd_amd.server_args import ServerArgs
    cfg = CONFIGS["mixed"]
    w = _write_checkpoint(str(tmp_path), cfg, seed=22)
    prompts = [_tokens(n, cfg["vocab"], seed=100 + n) for n in (5, 90, 47, 130)]
    sa = ServerArgs(model_path=str(tmp_path), load_format="auto", dtype="bfloat16", context_length=256, max_total_tokens=2048,
                    max_running_requests=8, cuda_graph_max_bs=8, chunked_prefill_size=48, skip_tokenizer_init=True,
                    enable_semi_pd=True, cu_mask_mode="env", prefill_cu_percent=50, decode_cu_percent=50, tune_prefill_gemm=False,
                    watchdog_timeout=120.0)
    eng = Engine(sa)
    try:
        outs = eng.generate(prompts, SamplingParams(max_new_tokens=16, ignore_eos=True), timeout=300)
    finally:
        eng.shutdown()
    _check_generation(cfg, w, prompts, outs, 16)
