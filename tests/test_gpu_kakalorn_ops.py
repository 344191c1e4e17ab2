"""Each mechanism of the Kakalorn layers alone, kernel against the plain functions: the convolution added to a mixer's
input carried through pieces and slots; the recurrence whose forget gate
writes, with gates at both ends; the head norm without a gate; windows with kept first positions, learned sinks and keys
as values, with one key made to stand out at every edge (prompt and single-token kernels, plain and matrix-core, page
borders, rotations of a part of the head); latent rows and queries that turn in pairs of neighbours with slowed
frequencies; gates of one number per head; the squared rectifier."""

import pytest
import torch

from tests.plain import kakalorn_plain as plain

pytestmark = pytest.mark.gpu
DEV = "cuda:0"
PAGE = 64
D64 = torch.float64


def _gen(seed):
    return torch.Generator().manual_seed(seed)


def _close(got, want, tol, what=""):
    want = want.to(D64)
    err = float((got.detach().cpu().to(D64) - want).abs().max() / want.abs().max().clamp_min(1e-30))
    assert err < tol, f"{what}: {err:.3g} >= {tol}"


def _i32(values):
    return torch.tensor(values, dtype=torch.int32, device=DEV)


def _pieces(lengths, cuts):
    """Steps that bring sequence ``b`` in pieces: for every step the (sequence, first, count) triples."""
    at = [0] * len(lengths)
    steps = []
    while any(a < n for a, n in zip(at, lengths)):
        step = []
        for b, n in enumerate(lengths):
            if at[b] < n:
                c = min(cuts[(len(steps) + b) % len(cuts)], n - at[b])
                step.append((b, at[b], c))
                at[b] += c
        steps.append(step)
    return steps


def _step(step, starts, slots):
    rows = [i for b, first, c in step for i in range(starts[b] + first, starts[b] + first + c)]
    cu = [0]
    for _, _, c in step:
        cu.append(cu[-1] + c)
    return rows, _i32(cu), _i32([slots[b] for b, _, _ in step]), [c for _, _, c in step]


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 1e-6), (torch.bfloat16, 6e-3)])
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 5, 8, 16])
@pytest.mark.parametrize("n", [5, 72, 1032, 4100])
def test_convolution_added_to_the_input(n, taps, dtype, tol):
    """Four sequences in slots beside slots of others, in pieces of 1 to 40 tokens, single-token steps among them."""
    from rocml_amd import ops
    g = _gen(n + taps)
    lengths, starts, slots = [90, 2, 33, 1], [0, 90, 92, 125], [2, 5, 0, 3]
    T = sum(lengths)
    h = torch.randn(T, n, generator=g).to(dtype)
    w = torch.randn(n, taps, generator=g)
    want = torch.cat([plain.added_conv(h[s:s + c].double(), w.double()) for s, c in zip(starts, lengths)])
    state = torch.zeros(6, taps - 1, n, dtype=dtype, device=DEV) if taps > 1 else None
    if state is not None:
        state[1].fill_(3.0)
    got = torch.zeros(T, n)
    for step in _pieces(lengths, [1, 40, 1, 2, 17]):
        rows, cu, seq_slots, counts = _step(step, starts, slots)
        out = torch.full((len(rows), n), 9.0, dtype=dtype, device=DEV)
        ops.added_conv(h[rows].to(DEV).contiguous(), w.t().contiguous().to(DEV), state, cu, seq_slots, counts, out)
        got[rows] = out.float().cpu()
    _close(got, want, tol, "convolved input")
    if state is not None:
        assert float((state[1].float() - 3.0).abs().max()) == 0.0 and float(state[4].float().abs().max()) == 0.0
        for s, c, slot in zip(starts, lengths, slots):
            kept = torch.cat([torch.zeros(taps - 1, n, dtype=dtype), h[s:s + c]])[-(taps - 1):]
            assert torch.equal(state[slot].cpu(), kept), "the kept rows are the last inputs"


def test_convolution_over_many_sequences_whose_runs_differ():
    from rocml_amd import ops
    g = _gen(3)
    n, taps, lengths = 64, 4, [16, 17, 1, 33, 15, 64, 2, 31, 32, 3]
    starts = [sum(lengths[:i]) for i in range(len(lengths))]
    h, w = torch.randn(sum(lengths), n, generator=g), torch.randn(n, taps, generator=g)
    want = torch.cat([plain.added_conv(h[s:s + c].double(), w.double()) for s, c in zip(starts, lengths)])
    state = torch.zeros(len(lengths), taps - 1, n, device=DEV)
    rows, cu, slots, counts = _step([(b, 0, c) for b, c in enumerate(lengths)], starts, list(reversed(range(len(lengths)))))
    out = torch.empty(len(rows), n, device=DEV)
    ops.added_conv(h.to(DEV), w.t().contiguous().to(DEV), state, cu, slots, counts, out)
    _close(out, want, 1e-6)


@pytest.mark.parametrize("dk,dv,H", [(1, 1, 2), (6, 12, 3), (20, 36, 3), (33, 9, 2), (64, 64, 3), (128, 130, 2), (256, 16, 2), (24, 40, 160)])
def test_recurrence_whose_gate_writes(dk, dv, H):
    """Pieces, slots and single-token steps; lower bounds of zero, of one (nothing is ever written) and next to one, logits
    that open and shut the gate altogether.  160 heads take the kernel of two columns a lane."""
    from rocml_amd import ops
    g = _gen(dk * 100 + dv)
    lengths, starts, slots = [70, 5, 33], [0, 70, 75], [4, 0, 2]
    T = sum(lengths)
    q, z = torch.randn(T, H, dk, generator=g, dtype=D64) * 2, torch.randn(T, H, dk, generator=g, dtype=D64) * 3
    v = torch.randn(T, H, dv, generator=g, dtype=D64)
    lower, bias = torch.rand(H, dk, generator=g, dtype=D64), torch.randn(H, dk, generator=g, dtype=D64)
    lower[0, 0] = 0.0
    lower[-1, -1] = 1.0
    lower[H // 2, 0] = 1.0 - 2.0 ** -12
    z[3], z[10, 0], z[11, 0] = 40.0, 90.0, -90.0
    q, z, v, lower, bias = (t.float().double() for t in (q, z, v, lower, bias))
    want = torch.cat([plain.gated_recurrence(plain.silu(q[s:s + n]), plain.forget_gate(z[s:s + n] + bias, lower), v[s:s + n])
                      for s, n in zip(starts, lengths)])
    state = torch.zeros(6, H, dv, dk, dtype=torch.float32, device=DEV)
    state[1].fill_(7.0)
    got = torch.zeros(T, H * dv)
    lo, bi = lower.reshape(-1).float().to(DEV), bias.reshape(-1).float().to(DEV)
    for col0 in (4, 3):          # rows that start on 16 bytes (where the sizes allow) and rows that do not
        state[[0, 2, 3, 4, 5]] = 0.0
        for step in _pieces(lengths, [1, 40, 2, 7]):
            rows, cu, seq_slots, _ = _step(step, starts, slots)
            mat = torch.cat([torch.zeros(len(rows), col0, dtype=D64), q[rows].reshape(len(rows), -1), z[rows].reshape(len(rows), -1),
                             v[rows].reshape(len(rows), -1)], dim=1).float().to(DEV).contiguous()
            out = torch.empty(len(rows), H * dv, dtype=torch.float32, device=DEV)
            ops.decay_scan(mat, col0, mat, col0 + H * dk, mat, col0 + 2 * H * dk, state, cu, seq_slots, out, H, dk, dv, gate_lower=lo, gate_bias=bi)
            got[rows] = out.cpu()
        _close(got, want.reshape(T, -1), 1e-5, "recurrence")
        assert float((state[1] - 7.0).abs().max()) == 0.0 and float(state[3].abs().max()) == 0.0, "other slots stay as they were"


def test_recurrence_keeps_a_value_for_a_thousand_tokens():
    """A gate that forgets one part in four thousand a token: what was written at the start is still there after 1,000
    tokens, to 32-bit accuracy."""
    from rocml_amd import ops
    g = _gen(1)
    T, H, dk, dv = 1000, 2, 16, 16
    q, v = torch.randn(T, H, dk, generator=g), torch.randn(T, H, dv, generator=g)
    z = torch.full((T, H, dk), 8.3)
    z[:5] = -30.0                                # the first tokens are written whole
    lower = torch.zeros(H, dk)
    want = plain.gated_recurrence(plain.silu(q.double()), plain.forget_gate(z.double(), lower.double()), v.double())
    mat = torch.cat([t.reshape(T, -1) for t in (q, z, v)], dim=1).to(DEV).contiguous()
    state, out = torch.zeros(1, H, dv, dk, device=DEV), torch.empty(T, H * dv, device=DEV)
    ops.decay_scan(mat, 0, mat, H * dk, mat, 2 * H * dk, state, _i32([0, T]), _i32([0]), out, H, dk, dv,
                   gate_lower=lower.reshape(-1).to(DEV), gate_bias=torch.zeros(H * dk, device=DEV))
    _close(out, want.reshape(T, -1), 5e-6)


@pytest.mark.parametrize("heads,dv", [(1, 1), (3, 17), (4, 64), (2, 130), (3, 256), (2, 600)])
def test_head_norm_without_a_gate(heads, dv):
    from rocml_amd import ops
    g = _gen(heads + dv)
    T, eps = 6, 1e-3
    o = torch.randn(T, heads, dv, generator=g, dtype=D64) * 4
    gain = 1 + 0.3 * torch.randn(dv, generator=g, dtype=D64)
    want = plain.norm(o, gain, eps).reshape(T, -1)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 1e-2)):
        out = torch.empty(T, heads * dv, dtype=dtype, device=DEV)
        ops.head_norm_gate(o.reshape(T, -1).float().to(DEV), None, 0, gain.repeat(heads).float().to(DEV), out, heads, eps, gate=None)
        _close(out, want, tol)


# ---- the windowed attention ---------------------------------------------------------------------
def _tables(T, rot):
    from rocml_amd import ops
    f, factor = plain.frequencies(rot)
    cos = torch.empty(T, rot["dims"] // 2, device=DEV)
    sin = torch.empty_like(cos)
    ops.rope_table(_i32(list(range(T))), torch.tensor(f, dtype=D64, device=DEV), cos, sin, factor)
    return cos, sin


def _attend(q, k, bq, bk, qg, kg, eps, rot, dtype, scale, window, keep, sinks, decode_from, seed, fused):
    """``q [T, H, d]``, ``k [T, G, d]`` as projected (without the bias) of one sequence through the library's kernels: the first
    ``decode_from`` positions as one prompt step, the rest one token a step (``fused``: by the kernel that reads the
    projection).  The sequence's pages lie scattered in the pool; pages that are neither kept nor in the window are gone."""
    from rocml_amd import ops
    T, H, d = q.shape
    G = k.shape[1]
    n_pages = (T + PAGE - 1) // PAGE
    perm = torch.randperm(n_pages + 3, generator=_gen(seed))[:n_pages].tolist()
    kc = torch.zeros(n_pages + 3, G, PAGE, d, dtype=dtype, device=DEV)
    vc = torch.zeros(n_pages + 3, G, d, PAGE, dtype=dtype, device=DEV)
    bias = torch.cat([bq.reshape(-1), bk.reshape(-1)]).float().to(DEV)
    cos_all, sin_all = _tables(T, rot)
    qg, kg, sinks = qg.float().to(DEV), kg.float().to(DEV), sinks.float().to(DEV)
    ws = torch.empty(1 << 22, dtype=torch.uint8, device=DEV)
    out = torch.zeros(T, H * d)
    for first, n in [(0, decode_from)] + [(i, 1) for i in range(decode_from, T)]:
        rows = slice(first, first + n)
        pages = [p if i < -(-keep // PAGE) or (i + 1) * PAGE > max(0, first - window + 1) else -1 for i, p in enumerate(perm)]
        table = torch.tensor([pages], dtype=torch.int32, device=DEV)
        qkv = torch.cat([q[rows].reshape(n, -1), k[rows].reshape(n, -1)], dim=1).float().to(DEV).contiguous()
        seq, pos = _i32([0] * n), _i32(list(range(first, first + n)))
        cos, sin = cos_all[rows].contiguous(), sin_all[rows].contiguous()
        o = torch.empty(n, H * d, dtype=dtype, device=DEV)
        splits = ops.decode_splits(G, 256, n_pages) if n == 1 else 0
        if n == 1 and fused:
            ops.attention_decode_fused(qkv, o, kc, vc, table, None, pos, H, G, d, scale, qg, kg, eps, cos, sin, window=window, workspace=ws,
                                       max_len=first + 1, n_splits=splits, bias=bias, sink=True, sinks=sinks, keep_first=keep,
                                       values_are_keys=True)
        else:
            qo = torch.empty(n, H * d, dtype=dtype, device=DEV)
            ops.qk_norm_rope_append(qkv, H, G, d, qg, kg, eps, cos, sin, rot["dims"], qo, kc, vc, table, seq, pos, bias=bias,
                                    values_are_keys=True)
            ops.attention(qo, o, kc, vc, table, seq, pos, H, G, d, scale, window, workspace=ws, cu_seqlens=_i32([0, n]), max_new=n,
                          q_counts=[n], max_len=first + n, n_splits=splits, sink=True, sinks=sinks, keep_first=keep)
        out[rows] = o.float().cpu()
    return out


def _want(q, k, bq, bk, qg, kg, eps, rot, scale, window, keep, sinks):
    T, H, d = q.shape
    G = k.shape[1]
    kb = k + bk
    qn, kn = plain.rotate(plain.norm(q + bq, qg, eps), rot, "halves"), plain.rotate(plain.norm(kb, kg, eps), rot, "halves")
    seen = plain.window_seen(T, window, keep)
    out = []
    for a in range(H):
        g = a // (H // G)
        out.append(plain.softmax_seen((qn[:, a] @ kn[:, g].T) * scale, seen, sinks[a]) @ kb[:, g])
    return torch.cat(out, dim=1)


SHAPES = [(torch.float32, 4, 2, 24, 12, False), (torch.float32, 2, 2, 64, 64, False), (torch.bfloat16, 4, 2, 64, 64, False),
          (torch.bfloat16, 4, 2, 64, 64, True), (torch.bfloat16, 8, 1, 128, 128, True), (torch.bfloat16, 6, 3, 128, 32, True),
          (torch.bfloat16, 3, 3, 48, 48, False), (torch.bfloat16, 6, 2, 96, 96, False), (torch.bfloat16, 2, 1, 256, 128, True),
          (torch.bfloat16, 4, 4, 32, 32, False), (torch.bfloat16, 4, 2, 192, 192, True), (torch.bfloat16, 34, 2, 64, 64, False)]


@pytest.mark.parametrize("dtype,H,G,d,dims,fused", SHAPES)
@pytest.mark.parametrize("window,keep", [(1, 1), (5, 3), (64, 64), (65, 1), (40, 65), (130, 4), (30, 0), (300, 7)])
def test_one_key_stands_out_at_every_edge(dtype, H, G, d, dims, fused, window, keep):
    """One key wins by far over all others wherever it is seen: the last kept position, the first that is not kept, positions on
    both sides of page borders.  Every query that sees it (in the window or kept) gives its value alone, every other gives
    nothing of it; the sink of one head equals its score and takes half.  All queries in a prompt and decoded ones."""
    g = _gen(window * 7 + d + keep)
    T, decode_from = 200, 150
    rot = {"dims": dims, "base": 1e7}
    eps = 1e-5
    q, k = torch.randn(T, H, d, generator=g, dtype=D64), torch.randn(T, G, d, generator=g, dtype=D64)
    bq, bk = 0.3 * torch.randn(H, d, generator=g, dtype=D64), 0.3 * torch.randn(G, d, generator=g, dtype=D64)
    qg, kg = 1 + 0.1 * torch.randn(d, generator=g, dtype=D64), 1 + 0.1 * torch.randn(d, generator=g, dtype=D64)
    # a direction that the rotation leaves alone: the slowest pair (its angle over 200 positions is next to nothing) and
    # whatever lies beyond the rotated part
    u = torch.zeros(d, dtype=D64)
    u[[dims // 2 - 1, dims - 1]] = 1.0
    u[dims:] = 0.5
    u = u / u.norm() * d ** 0.5
    q = 0.3 * q + u
    k = k - (k @ u)[..., None] / d * u                 # nothing along u
    places = sorted({j for j in (0, keep - 1, keep, 63, 64, 100, 127, 128) if 0 <= j < T})
    sinks = torch.full((H,), -25.0, dtype=D64)
    scale = 20.0 / d                                    # a key along u scores about 20
    sinks[0] = 20.0
    for j in places:
        kj = k.clone()
        kj[j] = u * 1.5 + 0.05 * k[j]
        qq, kk, b1, b2, g1, g2 = (t.float().double() for t in (q, kj, bq, bk, qg, kg))
        want = _want(qq, kk, b1, b2, g1, g2, eps, rot, scale, window, keep, sinks)
        got = _attend(qq, kk, b1, b2, g1, g2, eps, rot, dtype, scale, window, keep, sinks, decode_from, window + j, fused)
        err = (got.double() - want).abs().amax(dim=-1) / want.abs().max()
        tol = 2e-5 if dtype == torch.float32 else 4e-2
        assert float(err.max()) < tol, f"key {j}, worst query {int(err.argmax())}: {float(err.max()):.3g}"
        # the key shows: the last query that sees it and the next one differ by the order of its value
        last = j + window - 1
        if j >= keep and last + 1 < T and window > 1:
            assert float((want[last] - want[last + 1]).abs().max()) > 0.3


@pytest.mark.parametrize("H,G,d,dims", [(4, 2, 64, 64), (2, 2, 128, 64)])
def test_prompts_on_top_of_a_cache_and_unequal_sequences(H, G, d, dims):
    """Prompt steps of several tokens on top of cached positions, two sequences with different first positions in one step:
    the matrix-core prompt kernel visits the kept pages and then the window's."""
    from rocml_amd import ops
    g = _gen(d)
    lengths, cuts, window, keep, eps, scale = [420, 330], [[0, 90, 260, 420], [0, 200, 205, 330]], 70, 67, 1e-5, 0.2
    rot = {"dims": dims, "base": 5000.0}
    sinks = torch.randn(H, generator=g, dtype=D64)
    gains = [1 + 0.1 * torch.randn(d, generator=g, dtype=D64) for _ in range(2)]
    bias = [0.3 * torch.randn(H, d, generator=g, dtype=D64), 0.3 * torch.randn(G, d, generator=g, dtype=D64)]
    data, want = [], []
    for n in lengths:
        q, k = torch.randn(n, H, d, generator=g).double(), torch.randn(n, G, d, generator=g).double()
        k[:keep] *= 3.0
        data.append((q, k))
        want.append(_want(q, k, bias[0], bias[1], gains[0], gains[1], eps, rot, scale, window, keep, sinks))
    pages = [list(range(0, 14, 2)), list(range(1, 14, 2))]
    kc = torch.zeros(14, G, PAGE, d, dtype=torch.bfloat16, device=DEV)
    vc = torch.zeros(14, G, d, PAGE, dtype=torch.bfloat16, device=DEV)
    cos_all, sin_all = _tables(max(lengths), rot)
    for step in range(3):
        spans = [(cuts[b][step], cuts[b][step + 1]) for b in range(2)]
        counts = [e - s for s, e in spans]
        qkv = torch.cat([torch.cat([data[b][0][s:e].reshape(e - s, -1), data[b][1][s:e].reshape(e - s, -1)], dim=1)
                         for b, (s, e) in enumerate(spans)]).float().to(DEV).contiguous()
        pos = [p for s, e in spans for p in range(s, e)]
        seq = [b for b in range(2) for _ in range(counts[b])]
        cos, sin = cos_all[pos].contiguous(), sin_all[pos].contiguous()
        qo = torch.empty(len(pos), H * d, dtype=torch.bfloat16, device=DEV)
        table = torch.tensor(pages, dtype=torch.int32, device=DEV)
        ops.qk_norm_rope_append(qkv, H, G, d, gains[0].float().to(DEV), gains[1].float().to(DEV), eps, cos, sin, dims, qo, kc, vc, table,
                                _i32(seq), _i32(pos), bias=torch.cat([b.reshape(-1) for b in bias]).float().to(DEV), values_are_keys=True)
        outs = {}
        for algo in (ops.ATTN_MFMA, ops.ATTN_PLAIN):
            o = torch.empty_like(qo)
            ops.attention(qo, o, kc, vc, table, _i32(seq), _i32(pos), H, G, d, scale, window, algo=algo,
                          workspace=torch.empty(1 << 20, dtype=torch.uint8, device=DEV), cu_seqlens=_i32([0, counts[0], sum(counts)]),
                          max_new=max(counts), q_counts=counts, max_len=max(e for _, e in spans), sink=True, sinks=sinks.float().to(DEV),
                          keep_first=keep)
            outs[algo] = o
        ref = torch.cat([want[b][s:e] for b, (s, e) in enumerate(spans)])
        for algo, o in outs.items():
            _close(o, ref, 3e-2, f"step {step}, algorithm {algo}")


def test_refusals_of_the_attention():
    from rocml_amd import ops
    from rocml_amd.errors import KernelError
    q = torch.zeros(1, 64, dtype=torch.bfloat16, device=DEV)
    kc = torch.zeros(1, 1, PAGE, 64, dtype=torch.bfloat16, device=DEV)
    t = _i32([[0]])
    with pytest.raises(KernelError):
        ops.attention(q, torch.empty_like(q), kc, kc.transpose(2, 3).contiguous(), t, _i32([0]), _i32([0]), 1, 1, 64, 1.0, chunk=8, window=None,
                      keep_first=-1)
    qkv = torch.zeros(1, 128, device=DEV)
    with pytest.raises(KernelError):          # values that are keys have the keys' size
        ops.qk_norm_rope_append(qkv, 1, 1, 64, None, None, 1.0, None, None, 0, q, kc, torch.zeros(1, 1, 32, PAGE, dtype=torch.bfloat16, device=DEV),
                                t, _i32([0]), _i32([0]), v_head_dim=32, values_are_keys=True)


# ---- the latent attention's pieces ----------------------------------------------------------------
@pytest.mark.parametrize("dtype,tol", [(torch.float32, 5e-6), (torch.bfloat16, 1e-2)])
@pytest.mark.parametrize("q_rank,kv_rank,part,scaling", [(20, 24, 8, None), (70, 40, 12, (4.0, 64, 8.0, 1.0)), (300, 512, 64, (8.0, 4096, 32.0, 1.0))])
def test_latent_rows_that_turn_in_neighbours(q_rank, kv_rank, part, scaling, dtype, tol):
    from rocml_amd import ops
    g = _gen(q_rank + part)
    T, eps = 140, 1e-4
    rot = {"dims": part, "base": 3000.0}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    proj = torch.randn(T, q_rank + kv_rank + part + 3, generator=g)
    qg, kg = 1 + 0.2 * torch.randn(q_rank, generator=g), 1 + 0.2 * torch.randn(kv_rank, generator=g)
    P = proj.double()
    want_q = plain.norm(P[:, :q_rank], qg.double(), eps)
    want_c = plain.norm(P[:, q_rank:q_rank + kv_rank], kg.double(), eps)
    want_r = plain.rotate(P[:, None, q_rank + kv_rank:q_rank + kv_rank + part], rot, "neighbours")[:, 0]
    cos, sin = _tables(T, rot)
    cq = torch.empty(T, q_rank, dtype=dtype, device=DEV)
    cache = torch.full((4, PAGE, kv_rank + part), 5.0, dtype=dtype, device=DEV)
    table, seq, pos = _i32([[2, 0, 3]]), _i32([0] * T), _i32(list(range(T)))
    ops.latent_prepare(proj.to(DEV), q_rank, kv_rank, part, part, qg.to(DEV), kg.to(DEV), eps, cos, sin, cq, cache, table, seq, pos,
                       pairing="neighbours")
    rows = torch.cat([cache[p] for p in (2, 0, 3)])[:T]
    _close(cq, want_q, tol, "query latent")
    _close(rows[:, :kv_rank], want_c, tol, "latent")
    _close(rows[:, kv_rank:], want_r, tol, "rotated part")
    # a layer that reads another's rows: its projection holds the query latent (and a gate) alone, nothing is appended
    before = cache.clone()
    narrow = proj[:, :q_rank + 2].contiguous().to(DEV)
    cq2 = torch.empty_like(cq)
    ops.latent_prepare(narrow, q_rank, kv_rank, part, part, qg.to(DEV), None, eps, cos, sin, cq2, cache, table, seq, pos, write_cache=False,
                       pairing="neighbours")
    assert torch.equal(cq, cq2) and torch.equal(before, cache)


@pytest.mark.parametrize("dims,scaling", [(8, None), (2, (3.0, 40, 4.0, 1.0)), (32, (8.0, 128, 16.0, 2.0))])
def test_queries_that_turn_in_neighbours(dims, scaling):
    from rocml_amd import ops
    g = _gen(dims)
    T, H, d, stride, off = 70, 3, 5, 50, 7
    rot = {"dims": dims, "base": 777.0}
    if scaling is not None:
        rot["scaling"] = dict(zip(("factor", "original", "fast", "slow"), scaling))
    q = torch.randn(T, H, d + dims, generator=g)
    want = plain.rotate(q[..., d:].double(), rot, "neighbours")
    cos, sin = _tables(T, rot)
    out = torch.zeros(T, H * stride, device=DEV)
    ops.rope_heads(q.reshape(T, -1).to(DEV), H, d + dims, d, dims, dims, cos, sin, out, stride, off, lead=d, pairing="neighbours")
    got = out.view(T, H, stride)
    _close(got[..., off + d:off + d + dims], want, 2e-6, "rotated")
    assert torch.equal(got[..., off:off + d].cpu(), q[..., :d]) and float(got[..., :off].abs().max()) == 0.0


@pytest.mark.parametrize("T", [1, 9, 16, 40, 150])
def test_gate_of_one_number_per_head(T):
    """As the epilogue of the per-head products, on heads packed from a wider output, and as a kernel of its own."""
    from rocml_amd import ops
    g = _gen(T)
    H, N, K = 3, 40, 64
    x, w = torch.randn(T, H * K, generator=g).bfloat16(), (torch.randn(H, N, K, generator=g) / 8).bfloat16()
    wide = torch.randn(T, H + 9, generator=g) * 2
    gate = torch.sigmoid(wide[:, 6:6 + H].double())
    want = torch.stack([x.view(T, H, K)[:, h].double() @ w[h].double().T * gate[:, h:h + 1] for h in range(H)], dim=1).reshape(T, -1)
    out = torch.empty(T, H * N, dtype=torch.bfloat16, device=DEV)
    ops.gemm_batched(x.to(DEV), K, w.to(DEV), out, N, gate=wide.to(DEV)[:, 6:6 + H])
    _close(out, want, 1e-2, "epilogue of the products")
    y = torch.randn(T, H * 24, generator=g)
    for dtype, tol in ((torch.float32, 1e-6), (torch.bfloat16, 1e-2)):
        yd = y.to(dtype)
        packed = torch.empty(T, H * 10, dtype=dtype, device=DEV)
        ops.gate_heads(yd.to(DEV), 24, wide.to(DEV)[:, 6:6 + H], packed, H, 10)
        _close(packed, (yd.double().view(T, H, 24)[..., :10] * gate[..., None]).reshape(T, -1), tol, "packed heads")
        z = yd.clone().to(DEV)
        ops.sigmoid_gate(z, wide.to(DEV)[:, 6:6 + H], group=24)
        _close(z, (yd.double().view(T, H, 24) * gate[..., None]).reshape(T, -1), tol, "by itself")


# ---- the squared rectifier ------------------------------------------------------------------------
@pytest.mark.parametrize("m", [1, 2, 7, 16, 17, 40, 64, 130, 300])
@pytest.mark.parametrize("n,k", [(96, 72), (1100, 2048), (6144, 1024)])
def test_squared_rectifier_behind_a_product(m, n, k):
    """Every kernel of the product stores the square of the positive sums, also where K is cut into pieces."""
    from rocml_amd import ops
    g = _gen(m + n)
    x, w = torch.randn(m, k, generator=g).bfloat16(), (torch.randn(n, k, generator=g) / k ** 0.5).bfloat16()
    want = torch.relu(x.double() @ w.double().T) ** 2
    ws = torch.empty(64 << 20, dtype=torch.uint8, device=DEV)
    for splits in (0, 1):
        out = torch.full((m, n), -1.0, dtype=torch.bfloat16, device=DEV)
        ops.gemm(x.to(DEV), w.to(DEV), out, workspace=ws, epilogue="relu2", max_splits=splits)
        _close(out, want, 1e-2, f"max_splits {splits}")
    z = torch.empty(m, n, device=DEV)
    ops.gemm(x.to(DEV), w.to(DEV), z, workspace=ws)
    ops.activate(z, z, "relu2")
    _close(z, want, 1e-4, "behind the product")


def test_squared_rectifier_refuses_what_it_cannot_do():
    from rocml_amd import ops
    from rocml_amd.errors import KernelError
    x, w = torch.zeros(4, 12, device=DEV), torch.zeros(8, 12, device=DEV)
    with pytest.raises(KernelError):
        ops.gemm(x, w, torch.empty(4, 8, device=DEV), epilogue="relu2")
    with pytest.raises(KernelError):          # K of 12: not the matrix-core kernels
        ops.gemm(x.bfloat16(), w.bfloat16(), torch.empty(4, 8, dtype=torch.bfloat16, device=DEV), epilogue="relu2")
    with pytest.raises(KernelError):
        ops.activate(x, x, "square")
