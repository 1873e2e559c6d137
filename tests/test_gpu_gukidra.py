"""Gukidra on the GPU against the plain host statement (oracle/gukidra.py): every mechanism alone, then whole models through
the replay scheduler (whole prompts, token-by-token decoding, portions down to two tokens, unequal requests side by side,
slots and state rows that change hands, planted keys at every edge of a window and of a block) and greedy generation through
the Engine."""
import json
import os

import pytest
import torch

from oracle import gukidra as O

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
TOL = {torch.float32: dict(rtol=3e-5, atol=3e-5), torch.bfloat16: dict(rtol=3e-2, atol=3e-2), torch.float16: dict(rtol=4e-3, atol=4e-3)}


def _batch(parts):
    """parts: [(slot, lo, hi)] -> (slots, lengths after the step, q_start, q_len) on the device."""
    slots = torch.tensor([s for s, _, _ in parts], device=DEV)
    lens = torch.tensor([hi for _, _, hi in parts], device=DEV)
    n = torch.tensor([hi - lo for _, lo, hi in parts], dtype=torch.int32, device=DEV)
    return slots, lens, (torch.cumsum(n, 0) - n).int(), n


# ----------------------------------------------------------------------------------------------- the seam: norm of the output
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16, torch.float16])
@pytest.mark.parametrize("rows,width", [(1, 8), (5, 100), (37, 256), (3, 4104), (2, 2048), (2, 9000)])
def test_output_norm_seam(dtype, rows, width):
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(width)
    w, w2 = (0.3 * torch.randn(width, generator=g)).to(dtype), (0.3 * torch.randn(width, generator=g)).to(dtype)
    y = (2 * torch.randn(rows, width, generator=g)).to(dtype)
    x = 3 * torch.randn(rows, width, generator=g)
    want = x + O.one_plus_norm(y, w, 1e-5)
    stream = x.to(DEV)
    out = ops.outnorm_stream(y.to(DEV), stream, w.to(DEV), 1e-5, 1.0)
    torch.testing.assert_close(stream.cpu(), want, rtol=1e-5, atol=1e-5)                  # the stream keeps fp32
    torch.testing.assert_close(out.float().cpu(), want, **TOL[dtype])
    stream = x.to(DEV)                                                                    # the next reader's norm in the same launch
    out = ops.outnorm_stream(y.to(DEV), stream, w.to(DEV), 1e-5, 1.0, next_weight=w2.to(DEV), next_eps=1e-3, next_shift=1.0)
    torch.testing.assert_close(stream.cpu(), want, rtol=1e-5, atol=1e-5)
    torch.testing.assert_close(out.float().cpu(), O.one_plus_norm(want, w2, 1e-3), **TOL[dtype])
    stream = x.to(DEV)                                                                    # a plain weight, nothing wanted
    assert ops.outnorm_stream(y.to(DEV), stream, w.to(DEV), 1e-5, 0.0, want_out=False) is None
    torch.testing.assert_close(stream.cpu(), x + O.rms(y, 1e-5) * w.float(), rtol=1e-5, atol=1e-5)
    tiny = torch.full((rows, width), 1e-3).to(dtype)                                      # eps inside the root matters here
    stream = x.to(DEV)
    ops.outnorm_stream(tiny.to(DEV), stream, w.to(DEV), 1e-3, 1.0, want_out=False)
    torch.testing.assert_close(stream.cpu(), x + O.one_plus_norm(tiny, w, 1e-3), rtol=1e-5, atol=1e-5)


def test_embedding_with_a_copy_in_the_activation_type():
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(1)
    table = torch.randn(40, 72, generator=g).to(torch.bfloat16)
    ids = torch.randint(0, 40, (9,), generator=g)
    x, h = ops.embed_stream(ids.to(DEV), table.to(DEV), 7.3, want_copy=True)
    want = table[ids].float() * 7.3
    torch.testing.assert_close(x.cpu(), want)
    assert torch.equal(h.cpu(), want.to(torch.bfloat16))


# ----------------------------------------------------------------------------------------------- preparation and block means
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,D,E,rot,pool", [(8, 4, 64, 32, 32, 8), (3, 3, 20, 12, 20, 5), (4, 1, 96, 160, 96, 16), (1, 1, 8, 8, 2, 1),
                                              (6, 2, 48, 80, 16, 3), (2, 2, 256, 256, 128, 2), (2, 1, 24, 40, 10, 7)])
def test_head_norms_rotation_store_and_block_means(dtype, H, G, D, E, rot, pool):
    """Portions, single tokens in a prompt batch and decode batches; slots scattered over the pool; other slots untouched."""
    from semi_pd_amd import ops
    from semi_pd_amd.mem_cache.memory_pool import mean_piece
    g = torch.Generator().manual_seed(D + E)
    base, eps, N = 700.0, 1e-4, 150
    freq = lambda n: torch.tensor([base ** (-2.0 * i / n) for i in range(n // 2)], dtype=torch.float64).float().to(DEV)
    qw, kw = (1.5 + 0.3 * torch.randn(D, generator=g)).to(dtype), (0.7 + 0.3 * torch.randn(D, generator=g)).to(dtype)
    width = H * D + G * (D + E) + 8
    width += -width % 8
    lens = {0: 61, 2: 33}
    raw = {r: (1.5 * torch.randn(n, width, generator=g)).to(dtype) for r, n in lens.items()}
    want_q = {r: O.turn_halves(O.head_norm(x[:, : H * D].view(-1, H, D), qw, eps), rot, base) for r, x in raw.items()}
    want_k = {r: O.turn_halves(O.head_norm(x[:, H * D: (H + G) * D].reshape(-1, G, D), kw, eps), rot, base) for r, x in raw.items()}
    want_v = {r: O.turn_halves(x[:, (H + G) * D: (H + G) * D + G * E].reshape(-1, G, E), E, base) for r, x in raw.items()}
    perm = torch.randperm(N, generator=g) + 1
    table = torch.zeros(3, 64, dtype=torch.int32)
    table[0, :61], table[2, :33] = perm[:61].int(), perm[61:94].int()
    table_d = table.to(DEV)
    kp, vp = torch.full((N + 1, G, D), 3.0, dtype=dtype, device=DEV), torch.full((N + 1, G, E), 3.0, dtype=dtype, device=DEV)
    km = torch.full((G, N + 1, mean_piece(D, pool)), 5.0, dtype=dtype, device=DEV)
    vm = torch.full((G, N + 1, mean_piece(E, pool)), 5.0, dtype=dtype, device=DEV)

    def run(parts, decode=False):
        x = torch.cat([raw[r][lo:hi] for r, lo, hi in parts]).to(DEV)
        rows, lengths, start, n = _batch(parts)
        pos = torch.cat([torch.arange(lo, hi) for _, lo, hi in parts]).to(DEV)
        loc = torch.cat([table[r, lo:hi] for r, lo, hi in parts]).long().to(DEV)
        keep = x[:, (H + G) * D + G * E:].clone()
        ops.head_norm_rope_kv_store(x, H, G, D, E, H * D, (H + G) * D, qw.to(DEV), kw.to(DEV), eps, ops.angle_table(pos, freq(rot)), rot,
                                    ops.angle_table(pos, freq(E)), kp, vp, loc, (pool, km, vm), pos, table_d, rows, lengths,
                                    None if decode else start, None if decode else n)
        torch.testing.assert_close(x[:, : H * D].float().cpu().view(-1, H, D), torch.cat([want_q[r][lo:hi] for r, lo, hi in parts]), **TOL[dtype])
        assert torch.equal(x[:, (H + G) * D + G * E:], keep)
        if not decode:                   # a layer that only has queries
            x2 = torch.cat([raw[r][lo:hi] for r, lo, hi in parts]).to(DEV)
            ops.head_norm_rope_kv_store(x2, H, 0, D, E, 0, 0, qw.to(DEV), None, eps, ops.angle_table(pos, freq(rot)), rot, None, None, None, None)
            assert torch.equal(x2[:, : H * D], x[:, : H * D]) and torch.equal(x2[:, H * D:].cpu(), torch.cat([raw[r][lo:hi, H * D:] for r, lo, hi in parts]))

    run([(0, 0, 17), (2, 0, 2)])
    run([(2, 2, 3), (0, 17, 18)])                    # single tokens as a prompt batch
    for i in range(15):
        run([(0, 18 + i, 19 + i), (2, 3 + i, 4 + i)], decode=True)
    run([(2, 18, 33), (0, 33, 61)])
    kp_c, vp_c, km_c, vm_c = kp.cpu(), vp.cpu(), km.cpu(), vm.cpu()
    used = set()
    for r, n in lens.items():
        s = table[r, :n].long()
        torch.testing.assert_close(kp_c[s].float(), want_k[r], **TOL[dtype])
        torch.testing.assert_close(vp_c[s].float(), want_v[r], **TOL[dtype])
        used |= set(s.tolist())
        # the means are those of the rows as the pool holds them, one rounding
        for cache, means, size in ((kp_c[s], km_c, D), (vp_c[s], vm_c, E)):
            piece, mean = means.shape[2], O.block_means(cache.float(), pool)
            for b in range(n // pool):
                got = means[:, s[b * pool: (b + 1) * pool]].reshape(G, pool * piece)[:, :size]
                torch.testing.assert_close(got.float(), mean[b], rtol=2 ** -8 if dtype == torch.bfloat16 else 1e-5, atol=1e-6)
            for tok in range(n // pool * pool, n):                              # a block that is not whole has no mean yet
                assert (means[:, s[tok]] == 5.0).all()
    free = [i for i in range(N + 1) if i not in used]
    assert (kp_c[free] == 3.0).all() and (vp_c[free] == 3.0).all() and (km_c[:, free] == 5.0).all() and (vm_c[:, free] == 5.0).all()
    # means of another block size of the same rows, as a second reader of the cache asks for
    other = pool + 1
    km2 = torch.zeros((G, N + 1, mean_piece(D, other)), dtype=dtype, device=DEV)
    vm2 = torch.zeros((G, N + 1, mean_piece(E, other)), dtype=dtype, device=DEV)
    rows, lengths, start, n = _batch([(2, 0, 33), (0, 0, 61)])
    ops.block_means(kp, vp, (other, km2, vm2), table_d, rows, lengths, start, n, 94)
    for r, n_ in lens.items():
        s = table[r, :n_].long()
        mean = O.block_means(vp_c[s].float(), other)
        for b in range(n_ // other):
            got = vm2.cpu()[:, s[b * other: (b + 1) * other]].reshape(G, -1)[:, :E]
            torch.testing.assert_close(got.float(), mean[b], rtol=2 ** -8 if dtype == torch.bfloat16 else 1e-5, atol=1e-6)


# ----------------------------------------------------------------------------------------------- attention
def _attn_truth(q, k, v, kb, vb, gate, scale, window, pool, base):
    """q [T, H, D], k / v [T, G, .], kb / vb [T // pool, G, .] as the pools hold them."""
    T, H, E = q.shape[0], q.shape[1], v.shape[2]
    of = torch.arange(H) // (H // k.shape[1])
    mask = O.pooled_window_mask(T, window, pool) if pool else \
        ((torch.arange(T).view(T, 1) >= torch.arange(T)) & (torch.arange(T).view(T, 1) - torch.arange(T) < (window or T + 1)))
    kk, vv = (k, v) if not pool else (torch.cat([k, kb]), torch.cat([v, vb]))
    s = torch.einsum("ihd,jhd->hij", q, kk[:, of]) * scale
    p = O.softmax_with_one(s.masked_fill(~mask.unsqueeze(0), float("-inf")))
    o = O.turn_halves((p @ vv[:, of].transpose(0, 1)).transpose(0, 1), E, base, back=True)
    return (o * torch.sigmoid(gate.float()).unsqueeze(-1)).reshape(T, H * E)


@pytest.mark.parametrize("dtype,form", [(torch.float32, 0), (torch.bfloat16, 0), (torch.bfloat16, 1), (torch.float16, 0)])
@pytest.mark.parametrize("H,G,D,E,window,pool", [(8, 2, 64, 64, 40, 8), (4, 1, 96, 48, 33, 16), (3, 1, 20, 12, 7, 5), (4, 4, 32, 160, 64, 2),
                                                 (2, 1, 256, 256, 16, 32), (36, 2, 32, 16, 1, 1), (2, 2, 64, 80, 100, 3), (4, 2, 64, 64, 24, 0),
                                                 (4, 2, 64, 64, 0, 0)])
def test_window_with_pooled_blocks(dtype, form, H, G, D, E, window, pool):
    """Random keys and, for a range of queries, planted ones: query i is lined up with the key just inside its window, the
    one just outside, the last token of the last block it sees and the first of the next, so that an edge that is one off
    moves the result by the planted value."""
    from semi_pd_amd import ops
    from semi_pd_amd.mem_cache.memory_pool import mean_piece
    g = torch.Generator().manual_seed(H * 1000 + D + window)
    T, other, base, scale = 210, 75, 90.0, 0.9 * D ** -0.5
    N = 400
    seqs = {}
    for r, n in ((1, T), (0, other)):
        q, k, v = (torch.randn(n, h, d, generator=g) for h, d in ((H, D), (G, D), (G, E)))
        for x, i in enumerate(range(n - 1, max(n - 24, 0), -1)):
            last = (max(0, i - window + 1) // pool) * pool - 1 if pool and window else -1      # last token of the last block seen
            for j in ((i - window + 1, i - window, last, last + 1)[x % 4], 0):
                if 0 <= j <= i and window:
                    k[j, :] = 0.7 * q[i].view(G, H // G, D)[:, 0] * (3.0 if j == last else 1.0)
                    v[j, :] = 4.0 if x % 2 else -4.0
                    break
        seqs[r] = [t.to(dtype) for t in (q, k, v)] + [(2 * torch.randn(n, H, generator=g)).to(dtype)]
    perm = torch.randperm(N, generator=g) + 1
    table = torch.zeros(3, 256, dtype=torch.int32)
    table[1, :T], table[0, :other] = perm[:T].int(), perm[T: T + other].int()
    kp, vp = torch.zeros(N + 1, G, D, dtype=dtype), torch.zeros(N + 1, G, E, dtype=dtype)
    for r, n in ((1, T), (0, other)):
        kp[table[r, :n].long()], vp[table[r, :n].long()] = seqs[r][1], seqs[r][2]
    kp, vp, table = kp.to(DEV), vp.to(DEV), table.to(DEV)
    freq = torch.tensor([base ** (-2.0 * i / E) for i in range(E // 2)], dtype=torch.float64).float().to(DEV)
    sink = torch.zeros(H, device=DEV)
    means = None
    if pool:
        km, vm = (torch.zeros(G, N + 1, mean_piece(d, pool), dtype=dtype, device=DEV) for d in (D, E))
        means = (pool, km, vm)
        rows, lens, start, n = _batch([(1, 0, T), (0, 0, other)])
        ops.block_means(kp, vp, means, table, rows, lens, start, n, T + other)
    truth = {}
    for r, n in ((1, T), (0, other)):
        q, k, v, gate = (x.float() for x in seqs[r])
        kb, vb = (O.block_means(x, pool).to(dtype).float() if pool else None for x in (k, v))
        truth[r] = _attn_truth(q, k, v, kb, vb, gate, scale, window, pool, base)

    def check(parts, decode=False, n_splits=1):
        q = torch.cat([seqs[r][0][lo:hi] for r, lo, hi in parts]).reshape(-1, H * D).to(DEV)
        gate = torch.cat([seqs[r][3][lo:hi] for r, lo, hi in parts]).to(DEV)
        pos = torch.cat([torch.arange(lo, hi) for _, lo, hi in parts]).to(DEV)
        rows, lens, start, n = _batch(parts)
        out = torch.full((q.shape[0], H * E), 9.0, dtype=dtype, device=DEV)
        ops.pooled_window_attention_fwd(q, out, kp, vp, means, table, rows, lens, None if decode else start, None if decode else n,
                                        max(hi - lo for _, lo, hi in parts), scale, window, sink=sink, gate=gate,
                                        turn=ops.angle_table(pos, freq), form=form, n_splits=n_splits)
        want = torch.cat([truth[r][lo:hi] for r, lo, hi in parts])
        tol = TOL[dtype]["atol"]
        torch.testing.assert_close(out.float().cpu(), want, rtol=tol, atol=tol)

    check([(1, 0, T)])
    check([(0, 0, other), (1, 0, T)])
    check([(1, 100, T), (0, 74, 75)])                            # a cached prefix beside a single token
    check([(1, 207, 209), (0, 30, 75)])
    for i in range(T - 26, T):
        check([(1, i, i + 1), (0, min(i - T + 26, 74), min(i - T + 26, 74) + 1)], decode=True)
    for splits in (2, 5, 16):
        check([(0, 74, 75), (1, 209, 210)], decode=True, n_splits=splits)
        check([(1, 130, 131), (0, 0, 1)], decode=True, n_splits=splits)


def test_the_one_in_the_denominator_without_gate_and_turn():
    """One token whose score is s: the result is e^s / (1 + e^s) of its value, whatever the size of s."""
    from semi_pd_amd import ops
    for dtype in (torch.float32, torch.bfloat16):
        q = torch.zeros(3, 32, dtype=dtype, device=DEV)
        q[0, 0], q[1, 0], q[2, 0] = 0.0, 3.0, -40.0
        kp = torch.zeros(4, 1, 32, dtype=dtype, device=DEV)
        kp[1:, 0, 0] = 4.0
        vp = torch.full((4, 1, 16), 2.0, dtype=dtype, device=DEV)
        out = torch.empty(3, 16, dtype=dtype, device=DEV)
        table = torch.tensor([[1], [2], [3]], dtype=torch.int32, device=DEV)
        one = torch.ones(3, dtype=torch.int64, device=DEV)
        ops.pooled_window_attention_fwd(q, out, kp, vp, None, table, torch.arange(3, device=DEV), one, None, None, 1, 1.0, 5,
                                        sink=torch.zeros(1, device=DEV))
        want = 2.0 * torch.sigmoid(torch.tensor([0.0, 12.0, -160.0]))
        torch.testing.assert_close(out[:, 3].float().cpu(), want, rtol=5e-3, atol=1e-6)


# ----------------------------------------------------------------------------------------------- matrix memory
def _memory_truth(p, H, D, E, ib, fb, cap, nw, eps):
    q, k, v, g, i, f = torch.split(p.float(), [H * D, H * D, H * E, H * E, H, H], 1)
    T = p.shape[0]
    li = O.soft_cap(i + ib, cap)
    lf = torch.nn.functional.logsigmoid(O.soft_cap(f + fb, cap))
    o = O.rms(O.matrix_memory_scan(q.view(T, H, D) * D ** -0.5, k.view(T, H, D), v.view(T, H, E), li, lf), eps)
    return o.reshape(T, H * E) * nw.float() * torch.sigmoid(g)


@pytest.mark.parametrize("dtype,form", [(torch.float32, 0), (torch.bfloat16, 0), (torch.bfloat16, 1), (torch.float16, 0)])
@pytest.mark.parametrize("H,D,E,fbias", [(3, 40, 24, 3.0), (2, 64, 72, 5.0), (4, 128, 96, 3.0), (1, 256, 160, 6.0), (2, 20, 12, 1.0),
                                         (1, 8, 8, 0.0), (2, 13, 7, 2.0), (1, 200, 33, 4.0), (2, 16, 1100, 2.0)])
def test_matrix_memory_over_portions_and_decode_steps(dtype, form, H, D, E, fbias):
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(D * 7 + E)
    eps, cap, T = 1e-5, 6.0, 170
    width = 2 * H * D + 2 * H * E + 2 * H
    pad = -width % 8
    ib, fb = torch.randn(H, generator=g), fbias + torch.randn(H, generator=g)
    nw = (1 + 0.2 * torch.randn(H * E, generator=g)).to(dtype)
    seqs = {s: torch.cat([torch.randn(n, width, generator=g), torch.zeros(n, pad)], 1).to(dtype) for s, n in ((1, T), (3, 40))}
    for s in seqs:           # gates that rise and fall: the running maximum moves with single tokens
        seqs[s][:, width - 2 * H: width - H] = (4 * torch.randn(seqs[s].shape[0], H, generator=g)).to(dtype)
    want = {s: _memory_truth(x[:, :width], H, D, E, ib, fb, cap, nw, eps) for s, x in seqs.items()}
    sizes = [H * D, H * D, H * E, H * E, H, H]
    offs = [sum(sizes[:i]) for i in range(6)]
    slab = torch.full((5, ops.matrix_memory_state_width(H, D, E) + 8), 77.0, device=DEV)      # rows full of something else
    state = slab[:, 4: 4 + ops.matrix_memory_state_width(H, D, E)]
    tol = dict(rtol=2e-4, atol=2e-4) if dtype == torch.float32 else dict(rtol=2e-2, atol=2e-2)

    def run(parts, decode=False):
        x = torch.cat([seqs[s][lo:hi] for s, lo, hi in parts]).to(DEV)
        slots, lens, start, n = _batch(parts)
        out = ops.matrix_memory(x, offs, H, D, E, ib.to(DEV), fb.to(DEV), cap, nw.to(DEV), eps, state, slots, lens,
                                None if decode else start, None if decode else n, form=form)
        torch.testing.assert_close(out.float().cpu(), torch.cat([want[s][lo:hi] for s, lo, hi in parts]), **tol)

    run([(1, 0, T)])                                             # chunk by chunk
    run([(3, 0, 2), (1, 0, 70)])                                 # the row changes hands: what it held is not looked at
    run([(1, 70, 71), (3, 2, 3)], decode=True)
    run([(1, 71, 72), (3, 3, 4)])                                # single tokens in a prompt batch
    run([(3, 4, 6), (1, 72, 137)])
    run([(3, 6, 40)])
    for i in range(137, 150):
        run([(1, i, i + 1)], decode=True)
    run([(1, 150, T)])
    seqs[2], want[2] = seqs[3], want[3]                          # from the first token on, one by one
    for i in range(20):
        run([(2, i, i + 1)], decode=True)
    run([(2, 20, 40)])
    assert (slab[:, :4] == 77.0).all() and (slab[:, 4 + state.shape[1]:] == 77.0).all() and (slab[4] == 77.0).all()


def test_matrix_memory_keeps_a_far_token():
    """Forget gates close to one and one token with a high input gate: 700 tokens on, in chunks and token by token, the read-out of
    a query lined up with that token's key is that token's value."""
    from semi_pd_amd import ops
    g = torch.Generator().manual_seed(0)
    H, D, E, T = 1, 64, 32, 720
    for dtype in (torch.bfloat16, torch.float32):
        p = 0.05 * torch.randn(T, 2 * D + 2 * E + 2, generator=g)
        key, val = torch.randn(D, generator=g), torch.randn(E, generator=g)
        p[3, D: 2 * D], p[3, 2 * D: 2 * D + E], p[3, -2] = key, val, 9.0
        p[:, -1] = 12.0
        p[-8:, :D] = key
        p = torch.cat([p, torch.zeros(T, -p.shape[1] % 8)], 1).to(dtype)
        state = torch.zeros(2, ops.matrix_memory_state_width(H, D, E), device=DEV)
        offs = [0, D, 2 * D, 2 * D + E, 2 * D + 2 * E, 2 * D + 2 * E + 1]
        z, nw = torch.zeros(1, device=DEV), torch.ones(E, dtype=dtype, device=DEV)
        want = _memory_truth(p[:, : 2 * D + 2 * E + 2], H, D, E, 0.0, 0.0, 15.0, nw.cpu(), 1e-6)
        slots, lens, start, n = _batch([(1, 0, 716)])
        ops.matrix_memory(p[:716].to(DEV), offs, H, D, E, z, z, 15.0, nw, 1e-6, state, slots, lens, start, n)
        for i in range(716, T):
            slots, lens, _, _ = _batch([(1, i, i + 1)])
            out = ops.matrix_memory(p[i: i + 1].to(DEV), offs, H, D, E, z, z, 15.0, nw, 1e-6, state, slots, lens, None, None).float().cpu()
            torch.testing.assert_close(out, want[i: i + 1], rtol=2e-2, atol=2e-2)
            lined_up = torch.nn.functional.cosine_similarity(out[0] / torch.sigmoid(p[i, 2 * D + E: 2 * D + 2 * E].float()), val, dim=0)
            assert lined_up > 0.99


# ----------------------------------------------------------------------------------------------- whole models
def _attn(heads, kv_heads, dim, vdim, dims, size, pool, base=300.0, kv_from=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5, "rot": {"base": base, "dims": dims},
         "mask": {"size": size, "pool": pool}}
    if kv_from is not None:
        m["kv_from"] = kv_from
    return {"type": "attention", "mixer": m}


def _memory(heads, dim, vdim, cap=10.0):
    return {"type": "mlstm", "mixer": {"heads": heads, "dim": dim, "vdim": vdim, "gate_cap": cap}}


def _layer(mixer, ff):
    return dict(mixer, mlp=None if ff is None else {"kind": "dense", "ff": ff})


def _config(vocab, width, layers, eps=1e-5, scale=5.0):
    return {"architecture": "Gukidra", "vocab": vocab, "width": width, "norm": {"eps": eps}, "embedding": {"scale": scale}, "layers": layers}


CONFIGS = {
    # both mixers with and without a feed-forward, a cache that two other layers read with windows and blocks of their own
    "mixed": _config(200, 96, [_layer(_memory(3, 40, 24), 64), _layer(_attn(4, 2, 64, 48, 32, 40, 8), None),
                               _layer(_attn(6, 2, 64, 48, 32, 23, 4, kv_from=1), 80), _layer(_memory(2, 64, 72, 4.0), None),
                               _layer(_attn(2, 1, 32, 64, 32, 64, 16), 48), _layer(_attn(2, 2, 64, 48, 32, 9, 8, kv_from=1), 40)]),
    "minimal": _config(65, 8, [_layer(_attn(1, 1, 8, 8, 8, 1, 1), None), _layer(_memory(1, 8, 8), None)], scale=1.0),
    "awkward": _config(77, 50, [_layer(_attn(3, 1, 20, 12, 10, 7, 5), 18), _layer(_memory(3, 13, 7, 2.0), 22),
                                _layer(_attn(5, 1, 20, 12, 10, 30, 3, kv_from=0), None), _layer(_attn(2, 2, 36, 10, 4, 11, 13), 6)], scale=3.3),
    "attention_only": _config(130, 64, [_layer(_attn(4, 4, 32, 32, 16, 16, 2), 64), _layer(_attn(8, 4, 32, 32, 16, 48, 6, kv_from=0), 64)]),
    "memory_only": _config(130, 64, [_layer(_memory(4, 16, 32), 64), _layer(_memory(1, 128, 40), None)]),
    "wide": _config(96, 128, [_layer(_attn(2, 1, 256, 256, 128, 32, 8), 64), _layer(_memory(1, 256, 64), None)]),
}


def _write_checkpoint(path, cfg, seed, change=None):
    from safetensors.torch import save_file
    w = O.random_weights(cfg, seed)
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
    `outliers` (16-bit runs) an outlier counts half as long as 97 of 100 positions stay below the figure returned (the norm of
    an output that nearly cancels passes 16-bit rounding on enlarged)."""
    d = (got - want) - (got - want).mean(-1, keepdim=True)
    e = d.pow(2).mean(-1).sqrt() / want.std(-1)
    if not outliers:
        return e.max().item()
    return max(e.max().item() / 2, torch.quantile(e, 0.97).item())


# (16 bits: every sublayer adds about 1 % of rounding to the stream -- its input, the projections, the mixer's output, all rounded
# -- and the mixed model has ten; the fp32 runs carry the weight of the comparison)
LIMIT = {"float32": 4e-5, "bfloat16": 8e-2}


@pytest.fixture(scope="module", params=["float32", "bfloat16"])
def mixed_model(request, tmp_path_factory):
    path = str(tmp_path_factory.mktemp("gukidra_mixed"))
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
            assert torch.quantile(err, 0.97).item() < 5e-2 and err.max().item() < 1e-1
    _pools_are_whole(sched)


def test_whole_prompts_match_the_plain_model(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    for n in prompts:
        got = _run_schedule(sched, {n: prompts[n]}, [[(n, len(prompts[n]))]])
        assert _rel_err(got[n], truth[n], dtype != "float32") < LIMIT[dtype], n
    _pools_are_whole(sched)


def test_decoding_token_by_token_matches_the_prompt_pass(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    # from the very first token on (an empty state, no block yet), and behind a prompt
    got = _run_schedule(sched, {"a": prompts["a"]}, [[("a", 1)]] * 150)
    assert _rel_err(got["a"], truth["a"], dtype != "float32") < LIMIT[dtype]
    got = _run_schedule(sched, {"f": prompts["f"]}, [[("f", 90)]] + [[("f", 1)]] * 41)
    assert _rel_err(got["f"], truth["f"], dtype != "float32") < LIMIT[dtype]
    _pools_are_whole(sched)


def test_portions_of_every_size_down_to_two(mixed_model):
    dtype, sched, prompts, truth, _ = mixed_model
    for cuts in ([2] * 75, [64, 2, 3, 17, 64], [1, 2, 1, 146], [149, 1], [33, 31, 32, 54], [7] * 21 + [3]):
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
@pytest.mark.parametrize("name", ["minimal", "awkward", "attention_only", "memory_only", "wide"])
def test_other_sizes_and_orders(name, dtype, tmp_path):
    cfg = CONFIGS[name]
    w = _write_checkpoint(str(tmp_path), cfg, seed=5)
    sched = _scheduler(str(tmp_path), dtype, max_tokens=256)
    prompts = {"x": _tokens(90, cfg["vocab"], 1), "y": _tokens(37, cfg["vocab"], 2)}
    truth = {n: O.forward(cfg, w, t) for n, t in prompts.items()}
    got = _run_schedule(sched, prompts, [[("x", 60), ("y", 2)], [("x", 1), ("y", 30)], [("x", 1), ("y", 1)], [("x", 28), ("y", 4)]])
    for n in prompts:
        assert _rel_err(got[n], truth[n], dtype != "float32") < LIMIT[dtype], n
    got = _run_schedule(sched, {"x": prompts["x"]}, [[("x", 70)]] + [[("x", 1)]] * 20)
    assert _rel_err(got["x"], truth["x"], dtype != "float32") < LIMIT[dtype]


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("name", ["minimal", "attention_only"])
def test_padded_rows_of_a_decode_graph_leave_the_pools_alone(name, dtype, tmp_path):
    """Three requests decode through a graph captured for four: the padded row (a sequence of one token, which completes a block
    where blocks are of one token) must not touch what the request in row 0 of the table holds."""
    cfg = CONFIGS[name]
    w = _write_checkpoint(str(tmp_path), cfg, seed=6)
    sched = _scheduler(str(tmp_path), dtype, max_tokens=256)
    assert 3 not in sched.model_runner.graph_runner.capture_bs and 4 in sched.model_runner.graph_runner.capture_bs
    prompts = {n: _tokens(k, cfg["vocab"], i) for i, (n, k) in enumerate((("x", 60), ("y", 45), ("z", 50)))}
    got = _run_schedule(sched, prompts, [[("x", 30), ("y", 15), ("z", 20)]] + [[("x", 1), ("y", 1), ("z", 1)]] * 30)
    for n in prompts:
        assert _rel_err(got[n], O.forward(cfg, w, prompts[n]), dtype != "float32") < LIMIT[dtype], n


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_eager_decode_steps_and_the_plain_kernel_forms(dtype, tmp_path, monkeypatch):
    """Without captured graphs, the attention a wave per row and the memory token by token."""
    monkeypatch.setenv("SEMIPD_LOCAL_ATTN_FORM", "1")
    monkeypatch.setenv("SEMIPD_MATRIX_MEMORY_FORM", "1")
    cfg = CONFIGS["mixed"]
    w = _write_checkpoint(str(tmp_path), cfg, seed=8)
    sched = _scheduler(str(tmp_path), dtype, max_tokens=256, graphs=False)
    prompts = {"x": _tokens(80, cfg["vocab"], 1), "y": _tokens(50, cfg["vocab"], 2)}
    got = _run_schedule(sched, prompts, [[("x", 40), ("y", 10)]] + [[("x", 1), ("y", 1)]] * 40)
    for n in prompts:
        assert _rel_err(got[n], O.forward(cfg, w, prompts[n]), dtype != "float32") < LIMIT[dtype], n


def test_a_far_token_decides_the_logits(tmp_path):
    """Sharp scores (large norm weights): a token that only a block mean or the memory still holds has to change the last position's
    logits in the engine exactly as in the plain model, in the prompt pass, over portions and when decoding."""
    cfg = _config(96, 64, [_layer(_attn(4, 2, 32, 32, 8, 24, 4), 64), _layer(_memory(2, 32, 32), None)])

    def sharpen(w):
        w["l0.mix.q.norm"] += 3.0
        w["l0.mix.k.norm"] += 1.0
        w["l1.mix.f.b"] += 5.0

    w = _write_checkpoint(str(tmp_path), cfg, seed=3, change=sharpen)
    sched = _scheduler(str(tmp_path), "float32", max_tokens=1408, max_requests=2)
    t = _tokens(700, 96, 9)
    want = O.forward(cfg, w, t)
    moved = []
    for j in (5, 60, 200, 333, 600):
        t2 = list(t)
        t2[j] = (t2[j] + 17) % 96
        moved.append(((O.forward(cfg, w, t2)[-1] - want[-1]).abs().max().item(), j, t2))
    change, j, t2 = max(moved)
    assert change > 1e-3
    want2 = O.forward(cfg, w, t2)
    for seq, truth in ((t, want), (t2, want2)):
        got = _run_schedule(sched, {"p": seq}, [[("p", 640)], [("p", 2)]] + [[("p", 1)]] * 58)
        assert _rel_err(got["p"], truth) < 2 * LIMIT["float32"]
        got = _run_schedule(sched, {"p": seq}, [[("p", 700)]])
        assert _rel_err(got["p"], truth) < 2 * LIMIT["float32"]


def test_long_prompt_and_long_decoding(tmp_path):
    """600 tokens in one portion (many tiles of the prompt attention, many chunks of the memory), then 200 decode steps, in
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
            assert row[tok] >= row.max() - 0.1 * row.std(), (len(p), i)
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
    """The same through a prefill and a decode process on one GPU: the rows and the block means of every attention layer, the slab
    of state rows and every parameter reach the prefill process through IPC handles; prompts are cut into 48-token portions
    in the prefill process and decoded in the other."""
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
