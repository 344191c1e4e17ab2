"""Each mechanism of the Nazulorn layers alone, kernel against the plain functions: the copies of the stream with their
links, K pieces and next norm; the recurrence with a decay per token and channel carried through pieces and slots; decays from
a low-rank product; two maps per head with one key made to stand out in one map at every window's edge (prompt and single-token kernels,
plain and matrix-core, page borders, rotations of a part of the head); identity experts, factors on the weights, limited gates."""

import pytest
import torch

from tests.plain import nazulorn_plain as plain

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


# ---- copies of the stream -------------------------------------------------------------------------
@pytest.mark.parametrize("streams", [1, 2, 3, 4, 5, 16])
@pytest.mark.parametrize("n", [5, 72, 1032, 4100, 8200, 20000])
def test_links_between_the_copies(streams, n):
    """Start from equal copies, two updates with the next input, one into the sum; whole outputs, outputs with K pieces to add, and K
    pieces alone; both types of the next input."""
    from rocml_amd import ops
    g = _gen(streams * 31 + n)
    T, eps, m = 3, 1e-4, 0.6

    def r(*shape, std=1.0):
        return torch.randn(*shape, generator=g) * std
    x0, gain = r(T, n), 1 + r(n, std=0.2)
    ins, outs, mixes = [r(streams) for _ in range(3)], [r(streams) for _ in range(3)], [r(streams, streams, std=0.5) for _ in range(3)]
    ys, pieces = [r(T, n) for _ in range(3)], [None, r(2, T, n), r(5, T, n)]
    dev = lambda t: t.float().contiguous().to(DEV)
    for dtype, tol in ((torch.float32, 1e-5), (torch.bfloat16, 8e-3)):
        want = [x0.double() for _ in range(streams)]
        xn = torch.empty(T, n, dtype=dtype, device=DEV)
        ops.stream_links(dev(x0), streams, w_in=dev(ins[0]), gain=dev(gain), eps=eps, normed=xn)
        _close(xn, plain.norm(plain.streams_input(want, ins[0].double()), gain.double(), eps), tol, "first input")
        src = dev(x0)
        copies = torch.empty(T, streams, n, device=DEV)
        total = torch.empty(T, n, device=DEV)
        for k in range(3):
            replace = k == 2
            y = pieces[k].double().sum(0) if replace else ys[k].double() + (0 if pieces[k] is None else pieces[k].double().sum(0))
            want = plain.streams_update(want, y, mixes[k].double(), outs[k].double(), m)
            kw = dict(y=dev(ys[k]), mix=dev(mixes[k]), w_out=dev(outs[k] * m), partials=None if pieces[k] is None else dev(pieces[k]), replace=replace)
            if k < 2:
                ops.stream_links(src, streams, dst=copies, w_in=dev(ins[k + 1]), gain=dev(gain), eps=eps, normed=xn, **kw)
                _close(copies, torch.stack(want, dim=1), 2e-6, f"copies after update {k}")
                _close(xn, plain.norm(plain.streams_input(want, ins[k + 1].double()), gain.double(), eps), tol, f"input after update {k}")
                src = copies
            else:
                before = copies.clone()
                ops.stream_links(copies, streams, total=total, **kw)
                _close(total, sum(want), 3e-6, "sum of the copies")
                assert torch.equal(before, copies), "the last update leaves the copies alone"


def test_the_sum_may_replace_its_source():
    """A model of one sublayer: equal copies in, their sum out, in one buffer."""
    from rocml_amd import ops
    g = _gen(8)
    x, y, mix, out = torch.randn(4, 96, generator=g), torch.randn(4, 96, generator=g), torch.randn(3, 3, generator=g), torch.randn(3, generator=g)
    want = sum(plain.streams_update([x.double()] * 3, y.double(), mix.double(), out.double(), 1.0))
    xd = x.to(DEV)
    ops.stream_links(xd, 3, y=y.to(DEV), mix=mix.to(DEV), w_out=out.to(DEV), total=xd)
    _close(xd, want, 2e-6)


# ---- the recurrence ---------------------------------------------------------------------------------
@pytest.mark.parametrize("H,dk,dv", [(1, 1, 1), (3, 20, 36), (2, 33, 9), (4, 64, 128), (2, 128, 130), (2, 200, 24), (1, 256, 8), (40, 16, 40)])
def test_recurrence_in_pieces_and_slots(H, dk, dv):
    """Four sequences in slots beside slots of others, in pieces of 1 to 40 tokens; decays at both ends (forgetting all and nothing)
    among them; rows that start on 16 bytes and rows that do not."""
    from rocml_amd import ops
    g = _gen(H * 100 + dk)
    lengths, slots = [70, 2, 33, 1], [2, 5, 0, 4]
    starts = [0, 70, 72, 105]
    T = sum(lengths)
    q, k = torch.randn(T, H, dk, generator=g), torch.randn(T, H, dk, generator=g)
    v = torch.randn(T, H, dv, generator=g)
    w = torch.sigmoid(torch.randn(T, H, dk, generator=g) * 3 + 2)
    w[torch.rand(T, H, dk, generator=g) < 0.05] = 1.0
    w[torch.rand(T, H, dk, generator=g) < 0.02] = 0.0
    scale = 0.37
    want = torch.cat([plain.decayed_recurrence(q[s:s + n].double() * scale, k[s:s + n].double(), v[s:s + n].double(), w[s:s + n].double())
                      for s, n in zip(starts, lengths)])
    state = torch.zeros(6, H, dv, dk, device=DEV)
    for col0 in (4, 3):
        state.zero_()
        state[1].fill_(7.0)
        got = torch.zeros(T, H * dv)
        for step in _pieces(lengths, [1, 40, 2, 7]):
            rows = [i for b, first, c in step for i in range(starts[b] + first, starts[b] + first + c)]
            cu = [0]
            for _, _, c in step:
                cu.append(cu[-1] + c)
            mat = torch.cat([torch.zeros(len(rows), col0), q[rows].reshape(len(rows), -1), k[rows].reshape(len(rows), -1),
                             v[rows].reshape(len(rows), -1)], dim=1).to(DEV).contiguous()
            dec = torch.cat([torch.zeros(len(rows), col0), w[rows].reshape(len(rows), -1)], dim=1).to(DEV).contiguous()
            out = torch.empty(len(rows), H * dv, device=DEV)
            ops.decay_scan(mat, col0, mat, col0 + H * dk, mat, col0 + 2 * H * dk, state, _i32(cu), _i32([slots[b] for b, _, _ in step]), out, H, dk,
                           dv, decay=dec, decay_col0=col0, out_scale=scale)
            got[rows] = out.cpu()
        _close(got, want.reshape(T, -1), 1e-5, "recurrence")
        assert float((state[1] - 7.0).abs().max()) == 0.0 and float(state[3].abs().max()) == 0.0, "other slots stay as they were"


def test_recurrence_keeps_a_value_for_a_thousand_tokens():
    """Decays next to one: what the first tokens wrote is still there after 1,000, to 32-bit accuracy."""
    from rocml_amd import ops
    g = _gen(1)
    T, H, dk, dv = 1000, 2, 16, 16
    q, k, v = torch.randn(T, H, dk, generator=g), torch.randn(T, H, dk, generator=g), torch.randn(T, H, dv, generator=g)
    k[5:] *= 1e-3                                # the first tokens' keys stand out
    w = 1.0 - 2.0 ** -12 * torch.rand(T, H, dk, generator=g)
    want = plain.decayed_recurrence(q.double(), k.double(), v.double(), w.double())
    mat = torch.cat([t.reshape(T, -1) for t in (q, k, v)], dim=1).to(DEV).contiguous()
    state, out = torch.zeros(1, H, dv, dk, device=DEV), torch.empty(T, H * dv, device=DEV)
    ops.decay_scan(mat, 0, mat, H * dk, mat, 2 * H * dk, state, _i32([0, T]), _i32([0]), out, H, dk, dv, decay=w.reshape(T, -1).to(DEV).contiguous())
    _close(out, want.reshape(T, -1), 5e-6)


@pytest.mark.parametrize("T,n,rank,tau", [(1, 1, 1, 1.0), (3, 70, 5, 16.0), (64, 300, 16, 8.0), (65, 513, 64, 4.0), (200, 1000, 70, 12.0), (9, 128, 200, 2.5)])
@pytest.mark.parametrize("wtype", [torch.float32, torch.bfloat16])
def test_decays_from_a_low_rank_product(T, n, rank, tau, wtype):
    from rocml_amd import ops
    g = _gen(T + n)
    low, w = torch.randn(T, rank + 3, generator=g), (torch.randn(n, rank, generator=g) * 2 / rank ** 0.5).to(wtype)
    bias = torch.randn(n, generator=g) * 4
    bias[::7] = 40.0                             # a gate that keeps all ...
    bias[3::7] = -60.0                           # ... and one that keeps next to nothing
    z = low[:, 2:2 + rank].double() @ w.double().T + bias.double()
    want = torch.exp(torch.nn.functional.logsigmoid(z) / tau)
    out = torch.empty(T, n, device=DEV)
    ops.low_rank_decay(low.to(DEV), 2, w.t().contiguous().to(DEV), bias.to(DEV), tau, out)
    err = (out.cpu().double() - want).abs()
    assert float(err.max()) < 4e-6 and float((err / want.clamp_min(1e-30))[want > 1e-20].max()) < 6e-5
    # next to one the decay itself is right to its last bits: what a thousand steps keep depends on it
    near = want > 0.99
    assert not bool(near.any()) or float(err[near].max()) < 4e-7


# ---- two maps per head --------------------------------------------------------------------------------
def _tables(T, rot):
    from rocml_amd import ops
    f, factor = plain.frequencies(rot)
    cos = torch.empty(T, rot["dims"] // 2, device=DEV)
    sin = torch.empty_like(cos)
    ops.rope_table(_i32(list(range(T))), torch.tensor(f, dtype=D64, device=DEV), cos, sin, factor)
    return cos, sin


def _in_kernel_order(q, G):
    """Query rows ``[T, H, 2, d]`` (head, map) with G key/value heads -> (key/value head, map, head of the group)."""
    T, H, _, d = q.shape
    return q.view(T, G, H // G, 2, d).transpose(2, 3).reshape(T, -1)


def _want(q, k, v, rot, scale, window, weight, diff, eps):
    T, H, _, d = q.shape
    G = k.shape[1]
    qr, kr = (plain.rotate(t.reshape(T, -1, d), rot).view(t.shape) for t in (q, k))
    seen = plain.window_seen(T, window)
    out = []
    for a in range(H):
        g = a // (H // G)
        maps = [plain.softmax_seen((qr[:, a, i] @ kr[:, g, i].T) * scale, seen) @ v[:, g] for i in (0, 1)]
        out.append(plain.combine_maps(maps[0], maps[1], weight, diff, eps))
    return torch.cat(out, dim=1)


def _attend(q, k, v, rot, dtype, scale, window, weight, diff, eps, cuts, seed, path):
    """One sequence through the library's kernels: ``cuts`` are the first positions of the steps, steps of one token by the
    single-token kernel where ``path`` is "fused".  The sequence's pages lie scattered in the pool; pages before the window are gone."""
    from rocml_amd import ops
    T, H, _, d = q.shape
    G, dv = k.shape[1], v.shape[2]
    n_pages = (T + PAGE - 1) // PAGE
    perm = torch.randperm(n_pages + 3, generator=_gen(seed))[:n_pages].tolist()
    kc = torch.zeros(n_pages + 3, 2 * G, PAGE, d, dtype=dtype, device=DEV)
    vc = torch.zeros(n_pages + 3, G, dv, PAGE, dtype=dtype, device=DEV)
    cos_all, sin_all = _tables(T, rot) if rot is not None else (None, None)
    ws = torch.empty(1 << 22, dtype=torch.uint8, device=DEV)
    out = torch.zeros(T, H * dv)
    for first, stop in zip(cuts, cuts[1:] + [T]):
        n, rows = stop - first, slice(first, stop)
        pages = [p if (i + 1) * PAGE > max(0, first - window + 1) else -1 for i, p in enumerate(perm)]
        table = torch.tensor([pages], dtype=torch.int32, device=DEV)
        qkv = torch.cat([_in_kernel_order(q[rows], G), k[rows].reshape(n, -1), v[rows].reshape(n, -1)], dim=1).float().to(DEV).contiguous()
        seq, pos = _i32([0] * n), _i32(list(range(first, stop)))
        cos, sin = (None, None) if rot is None else (cos_all[rows].contiguous(), sin_all[rows].contiguous())
        o = torch.full((n, H * dv), 9.0, dtype=dtype, device=DEV)
        if n == 1 and path == "fused":
            # (pieces of the projection, as a product cut along K leaves them, in every second step)
            src = torch.stack([0.25 * qkv, 0.5 * qkv, 0.25 * qkv]).contiguous() if first % 2 else qkv
            ops.diff_attention_decode(src, o, kc, vc, table, pos, H, G, d, dv, scale, weight, 1.0 - diff, eps, cos, sin, window=window,
                                      n_splits=1 + first % 4, workspace=ws)
        else:
            qo = torch.empty(n, 2 * H * d, dtype=dtype, device=DEV)
            ops.qk_norm_rope_append(qkv, 2 * H, 2 * G, d, None, None, 1.0, cos, sin, rot["dims"] if rot is not None else 0, qo, kc, vc, table, seq, pos,
                                    v_head_dim=dv, n_v_heads=G)
            maps = torch.empty(n, 2 * H * dv, device=DEV)
            ops.diff_attention(qo, o, kc, vc, table, seq, pos, H, G, d, dv, scale, weight, 1.0 - diff, eps, _i32([0, n]), [n], window=window, maps=maps,
                               plain=path == "plain")
        out[rows] = o.float().cpu()
    return out


SHAPES = [(torch.float32, 4, 2, 24, 20, 12, "plain"), (torch.float32, 2, 1, 64, 128, 64, "plain"), (torch.bfloat16, 4, 2, 64, 128, 64, "fused"),
          (torch.bfloat16, 4, 2, 64, 128, 32, "matrix"), (torch.bfloat16, 8, 1, 32, 64, 32, "fused"), (torch.bfloat16, 3, 3, 40, 72, 8, "fused"),
          (torch.bfloat16, 2, 1, 128, 256, 128, "fused"), (torch.bfloat16, 6, 2, 96, 60, 96, "fused"), (torch.bfloat16, 10, 1, 16, 36, 16, "matrix"),
          (torch.bfloat16, 2, 2, 128, 64, 64, "matrix"), (torch.bfloat16, 4, 4, 24, 200, None, "fused"), (torch.bfloat16, 2, 1, 20, 27, 20, "plain"),
          (torch.bfloat16, 2, 2, 64, 128, 64, "plain")]


@pytest.mark.parametrize("dtype,H,G,d,dv,dims,path", SHAPES)
@pytest.mark.parametrize("window", [1, 5, 64, 65, 130, 300])
def test_one_key_stands_out_at_every_edge(dtype, H, G, d, dv, dims, path, window):
    """In one of the maps one key wins by far over all others wherever it is seen: a window's first position, positions on both
    sides of page borders.  Every query that sees it gives its value in that map, every other nothing of it.  All queries in a prompt, in
    portions on top of a cache, and decoded ones; K pieces and splits of the keys in the decoded ones."""
    g = _gen(window * 7 + d)
    T = 200
    cuts = [0, 90, 92] + list(range(150, T))
    rot = None if dims is None else {"dims": dims, "base": 1e7}
    eps, diff, weight = 1e-5, 0.4, 0.7
    q, k = 0.3 * torch.randn(T, H, 2, d, generator=g, dtype=D64), torch.randn(T, G, 2, d, generator=g, dtype=D64)
    v = torch.randn(T, G, dv, generator=g, dtype=D64)
    # a direction that the rotation leaves alone: the slowest pair (its angle over 200 positions is next to nothing) and
    # whatever lies beyond the rotated part
    u = torch.zeros(d, dtype=D64)
    if dims is None:
        u[:] = 1.0
    else:
        u[[dims // 2 - 1, dims - 1]] = 1.0
        u[dims:] = 0.5
    u = u / u.norm() * d ** 0.5
    q = q + u
    k = k - (k @ u)[..., None] / d * u                 # nothing along u
    scale = 20.0 / d                                    # a key along u scores about 20
    for which, j in ((0, 0), (1, 63), (0, 64), (1, 100), (0, 127), (1, 128)):
        kj = k.clone()
        kj[j, :, which] = u * 1.5
        qq, kk, vv = (t.float().double() for t in (q, kj, v))
        want = _want(qq, kk, vv, rot, scale, window, weight, diff, eps)
        got = _attend(qq, kk, vv, rot, dtype, scale, window, weight, diff, eps, cuts, window + j, path)
        err = (got.double() - want).abs().amax(dim=-1) / want.abs().max()
        tol = 3e-5 if dtype == torch.float32 else 7e-2          # (a key lost or seen too long is more than 0.3)
        assert float(err.max()) < tol, f"map {which}, key {j}, worst query {int(err.argmax())}: {float(err.max()):.3g}"
        # the key shows: the last query that sees it and the next one differ by the order of its value
        last = j + window - 1
        if last + 1 < T and window > 1:
            assert float((want[last] - want[last + 1]).abs().max()) > 0.3


@pytest.mark.parametrize("H,G,d,dv,window", [(4, 2, 64, 128, 70), (8, 1, 32, 64, None), (3, 3, 128, 256, 200)])
def test_prompts_on_top_of_a_cache_and_unequal_sequences(H, G, d, dv, window):
    """Prompt steps on top of cached positions, two sequences with different first positions in one step, more rows than a block
    takes; decode steps of both sequences side by side, with splits."""
    from rocml_amd import ops
    g = _gen(d)
    lengths, cuts, eps, scale, weight, diff = [420, 330], [[0, 90, 260, 419], [0, 200, 205, 329]], 1e-5, 0.2, 0.55, 0.3
    rot = {"dims": d // 2, "base": 5000.0}
    data, want = [], []
    for n in lengths:
        q, k, v = (torch.randn(n, *s, generator=g).double() for s in ((H, 2, d), (G, 2, d), (G, dv)))
        data.append((q, k, v))
        want.append(_want(q, k, v, rot, scale, window or n, weight, diff, eps))
    table = torch.tensor([list(range(0, 14, 2)), list(range(1, 14, 2))], dtype=torch.int32, device=DEV)
    kc = torch.zeros(14, 2 * G, PAGE, d, dtype=torch.bfloat16, device=DEV)
    vc = torch.zeros(14, G, dv, PAGE, dtype=torch.bfloat16, device=DEV)
    cos_all, sin_all = _tables(max(lengths), rot)
    ws = torch.empty(1 << 24, dtype=torch.uint8, device=DEV)
    for step in range(4):
        spans = [(cuts[b][step], (cuts[b] + [lengths[b]])[step + 1]) for b in range(2)]
        counts = [e - s for s, e in spans]
        qkv = torch.cat([torch.cat([_in_kernel_order(data[b][0][s:e], G)] + [data[b][i][s:e].reshape(e - s, -1) for i in (1, 2)], dim=1)
                         for b, (s, e) in enumerate(spans)]).float().to(DEV).contiguous()
        pos = [p for s, e in spans for p in range(s, e)]
        seq = [b for b in range(2) for _ in range(counts[b])]
        cos, sin = cos_all[pos].contiguous(), sin_all[pos].contiguous()
        ref = torch.cat([want[b][s:e] for b, (s, e) in enumerate(spans)])
        if step == 3:
            for splits in (1, 2, 5, 40):
                o = torch.empty(2, H * dv, dtype=torch.bfloat16, device=DEV)
                ops.diff_attention_decode(qkv, o, kc, vc, table, _i32(pos), H, G, d, dv, scale, weight, 1.0 - diff, eps, cos, sin, window=window,
                                          n_splits=splits, workspace=ws)
                _close(o, ref, 3e-2, f"decode with {splits} splits")
            continue
        qo = torch.empty(len(pos), 2 * H * d, dtype=torch.bfloat16, device=DEV)
        ops.qk_norm_rope_append(qkv, 2 * H, 2 * G, d, None, None, 1.0, cos, sin, d // 2, qo, kc, vc, table, _i32(seq), _i32(pos), v_head_dim=dv,
                                n_v_heads=G)
        for slow in (False, True):
            o = torch.empty(len(pos), H * dv, dtype=torch.bfloat16, device=DEV)
            ops.diff_attention(qo, o, kc, vc, table, _i32(seq), _i32(pos), H, G, d, dv, scale, weight, 1.0 - diff, eps,
                               _i32([0, counts[0], sum(counts)]), counts, window=window, maps=torch.empty(len(pos), 2 * H * dv, device=DEV), plain=slow)
            _close(o, ref, 3e-2, f"step {step}, plain {slow}")


def test_maps_that_nearly_cancel_keep_their_difference():
    """Two maps that see almost the same keys and a weight next to one: the small difference is normed, so it has to be
    formed before anything is rounded to 16 bits."""
    g = _gen(3)
    T, H, G, d, dv = 150, 2, 1, 64, 128
    q, k = torch.randn(T, H, 1, d, generator=g, dtype=D64).expand(T, H, 2, d).contiguous(), torch.randn(T, G, 2, d, generator=g, dtype=D64)
    k[:, :, 1] = k[:, :, 0]
    k = k.float().bfloat16().double()
    q = q.float().bfloat16().double()
    v = torch.randn(T, G, dv, generator=g, dtype=D64).float().bfloat16().double()
    want = _want(q, k, v, None, 0.1, 50, 0.96, 0.5, 1e-9)
    for path in ("matrix", "fused", "plain"):
        got = _attend(q, k, v, None, torch.bfloat16, 0.1, 50, 0.96, 0.5, 1e-9, [0] + list(range(120, T)), 5, path)
        _close(got, want, 3e-2, path)


def test_refusals_of_the_attention():
    from rocml_amd import ops
    from rocml_amd.errors import KernelError
    q = torch.zeros(1, 2 * 64, dtype=torch.bfloat16, device=DEV)
    kc, vc = torch.zeros(1, 2, PAGE, 64, dtype=torch.bfloat16, device=DEV), torch.zeros(1, 1, 32, PAGE, dtype=torch.bfloat16, device=DEV)
    out, t = torch.empty(1, 32, dtype=torch.bfloat16, device=DEV), _i32([[0]])
    args = (t, _i32([0]), _i32([0]), 1, 1, 64, 32)
    for bad in (dict(scale=0.0), dict(eps=0.0), dict(counts=[2])):
        with pytest.raises(KernelError):
            ops.diff_attention(q, out, kc, vc, *args, bad.get("scale", 0.1), 0.5, 0.5, bad.get("eps", 1e-5), _i32([0, 1]), bad.get("counts", [1]))
    with pytest.raises(KernelError):          # a cache of one map
        ops.diff_attention(q, out, kc[:, :1].contiguous(), vc, *args, 0.1, 0.5, 0.5, 1e-5, _i32([0, 1]), [1])
    with pytest.raises(KernelError):          # the plain path without room for the maps
        ops.diff_attention(q, out, kc, vc, *args, 0.1, 0.5, 0.5, 1e-5, _i32([0, 1]), [1], plain=True)
    assert not ops.diff_attention_decode_fits(torch.bfloat16, 18, 2, 64, 128, PAGE) and not ops.diff_attention_sizes_ok(torch.bfloat16, 144, 64, PAGE)
    assert not ops.diff_attention_sizes_ok(torch.float32, 64, 128, PAGE) and ops.diff_attention_decode_fits(torch.bfloat16, 16, 2, 64, 128, PAGE)


@pytest.mark.parametrize("dtype,tol", [(torch.float32, 2e-6), (torch.bfloat16, 6e-3)])
@pytest.mark.parametrize("T", [3, 150])
@pytest.mark.parametrize("hq,hkv,hv,d,dv,rot", [(4, 4, 2, 64, 128, 64), (6, 2, 1, 40, 24, 16), (2, 2, 2, 32, 32, 8), (2, 4, 1, 24, 10, None), (2, 2, 1, 20, 7, 6)])
def test_rotation_and_append_with_shared_value_heads(hq, hkv, hv, d, dv, rot, T, dtype, tol):
    """Few rows and many (the two ways the kernels go), heads rotated whole, in part and not at all."""
    from rocml_amd import ops
    g = _gen(d + T)
    q, k, v = (torch.randn(T, *s, generator=g).double() for s in ((hq, d), (hkv, d), (hv, dv)))
    r = None if rot is None else {"dims": rot, "base": 500.0, "scaling": {"factor": 3.0, "original": 50, "fast": 8.0, "slow": 1.0}}
    qkv = torch.cat([t.reshape(T, -1) for t in (q, k, v)], dim=1).float().to(DEV).contiguous()
    cos, sin = _tables(T, r) if r is not None else (None, None)
    kc, vc = torch.full((4, hkv, PAGE, d), 5.0, dtype=dtype, device=DEV), torch.full((4, hv, dv, PAGE), 5.0, dtype=dtype, device=DEV)
    qo = torch.empty(T, hq * d, dtype=dtype, device=DEV)
    ops.qk_norm_rope_append(qkv, hq, hkv, d, None, None, 1.0, cos, sin, rot or 0, qo, kc, vc, _i32([[2, 0, 3]]), _i32([0] * T), _i32(list(range(T))),
                            v_head_dim=dv, n_v_heads=hv)
    _close(qo, plain.rotate(q, r).reshape(T, -1), tol, "queries")
    keys = torch.cat([kc[p].transpose(0, 1) for p in (2, 0, 3)])[:T]
    vals = torch.cat([vc[p].permute(2, 0, 1) for p in (2, 0, 3)])[:T]
    _close(keys, plain.rotate(k, r), tol, "keys")
    _close(vals, v, tol, "values")
    assert float((kc[1].float() - 5.0).abs().max()) == 0.0 and float((vc[1].float() - 5.0).abs().max()) == 0.0, "other pages stay as they were"


# ---- experts ----------------------------------------------------------------------------------------
@pytest.mark.parametrize("E,top", [(3, 1), (7, 3), (66, 6), (130, 12), (4, 4)])
@pytest.mark.parametrize("scale", [1.0, 2.3])
def test_choice_with_a_correction_and_a_factor(E, top, scale):
    from rocml_amd import ops
    g = _gen(E + top)
    logits, corr = torch.randn(90, E + 5, generator=g) * 1.5, torch.randn(E, generator=g) * 0.2
    want_e, want_w = plain.choose_experts(logits[:, 5:].double(), corr.double(), top, scale)
    chosen, weight = torch.empty((90, top), dtype=torch.int32, device=DEV), torch.empty((90, top), device=DEV)
    ops.moe_route(logits.to(DEV)[:, 5:], top, None, 1e-20, chosen, weight, correction=corr.to(DEV), weight_scale=scale)
    assert torch.equal(chosen.cpu().long(), want_e), "other experts (the best first)"
    _close(weight, want_w, 1e-5)
    if 1 < top < E:
        assert not torch.equal(plain.choose_experts(logits[:, 5:].double(), 0 * corr.double(), top, scale)[0], want_e), "the correction changes nothing here"


@pytest.mark.parametrize("T,w,ff,E,ident,top,limit,dtype,tol", [
    (200, 40, 24, 3, 2, 2, 0.8, torch.float32, 2e-5), (1, 72, 40, 6, 1, 3, 1.5, torch.float32, 2e-5), (200, 64, 48, 3, 1, 2, 0.7, torch.bfloat16, 2e-2),
    (5, 128, 64, 16, 4, 4, 1.0, torch.bfloat16, 2e-2), (130, 36, 20, 4, 3, 9 - 2, None, torch.bfloat16, 2e-2), (70, 64, 32, 5, 0, 5, 2.0, torch.bfloat16, 2e-2),
    (33, 256, 136, 2, 9, 11, 0.5, torch.bfloat16, 2e-2), (300, 30, 22, 1, 1, 1, 0.9, torch.bfloat16, 2e-2)])
def test_experts_with_limits_and_identities(T, w, ff, E, ident, top, limit, dtype, tol):
    """Pairs of identity experts have no place in the order; the token's own row stands for them in the weighted sum."""
    from rocml_amd import ops
    g = _gen(T + E)
    t = {"router": torch.randn(E + ident, w, generator=g), "correction": torch.randn(E + ident, generator=g) * 0.1}
    for e in range(E):
        t[f"e{e}.gate"] = (torch.randn(ff, w, generator=g) * 1.5 / w ** 0.5).to(dtype).float()
        t[f"e{e}.up"] = (torch.randn(ff, w, generator=g) * 1.5 / w ** 0.5).to(dtype).float()
        t[f"e{e}.down"] = (torch.randn(w, ff, generator=g) / ff ** 0.5).to(dtype).float()
    h = torch.randn(T, w, generator=g).to(dtype).float()
    m = {"router": {"experts": E, "identity": ident, "top": top, "scale": 1.7}, "expert": {"limit": limit}}
    want = plain.experts(h.double(), {k: v.double() for k, v in t.items()}, m)
    logits = (h.double() @ t["router"].double().T).float()
    chosen, weight = torch.empty((T, top), dtype=torch.int32, device=DEV), torch.empty((T, top), device=DEV)
    ops.moe_route(logits.to(DEV), top, None, 1e-20, chosen, weight, correction=t["correction"].to(DEV), weight_scale=1.7)
    pairs = T * top
    plan = ops.moe_plan(chosen, E, torch.empty(ops.moe_plan_words(pairs, E), dtype=torch.int32, device=DEV))
    offsets, order, place = plan[0].cpu(), plan[1].cpu(), plan[2].cpu()
    flat = chosen.cpu().reshape(-1)
    real = int((flat < E).sum())
    assert int(offsets[-1]) == real and sorted(order[:real].tolist()) == torch.nonzero(flat < E).flatten().tolist()
    assert all(int(place[int(p)]) == i for i, p in enumerate(order[:real])) and bool((place[flat >= E] == -1).all())
    if ident and T > 1:
        assert real < pairs, "no identity expert is chosen in this test"
    stack = lambda kind: torch.stack([t[f"e{e}.{kind}"] for e in range(E)]).to(dtype).to(DEV).contiguous()
    own = h.to(dtype).to(DEV)
    hid = torch.zeros((pairs, ff), dtype=dtype, device=DEV)
    act = dict(activation="sigmoid_1702", limit=limit, up_offset=1.0)
    ops.moe_gemm(own, stack("gate"), hid, plan, top, gather=True, w2=stack("up"), **act)
    y = torch.full((pairs, w), float("nan"), device=DEV)
    ops.moe_gemm(hid, stack("down"), y, plan, top, gather=False)
    out = torch.full((T, w), float("nan"), device=DEV)
    ops.moe_combine(y, plan, weight, out, own=own)
    _close(out, want, tol)
    base = torch.randn(T, w, generator=g)
    acc = base.to(DEV)
    ops.moe_combine(y, plan, weight, acc, accumulate=True, own=own)
    _close(acc, want + base.double(), tol)
    if dtype == torch.bfloat16:
        hid2 = torch.zeros_like(hid)
        ops.moe_gemm(own, stack("gate"), hid2, plan, top, gather=True, w2=stack("up"), plain=True, **act)
        _close(hid2[:real], hid[:real].double().cpu(), 2e-2, "the plain kernel")


@pytest.mark.parametrize("activation", ["silu", "relu", "gelu_tanh", "sigmoid_1702"])
def test_every_activation_in_the_experts_products(activation):
    from rocml_amd import ops
    g = _gen(4)
    x, wg, wu = torch.randn(9, 32, generator=g), torch.randn(2, 24, 32, generator=g), torch.randn(2, 24, 32, generator=g)
    chosen = torch.tensor([[i % 2] for i in range(9)], dtype=torch.int32, device=DEV)
    plan = ops.moe_plan(chosen, 2, torch.empty(ops.moe_plan_words(9, 2), dtype=torch.int32, device=DEV))
    act = {"silu": plain.silu, "relu": torch.relu, "sigmoid_1702": lambda z: z * torch.sigmoid(1.702 * z),
           "gelu_tanh": lambda z: torch.nn.functional.gelu(z, approximate="tanh")}[activation]
    gate, up = (torch.stack([x.double()[i] @ w.double()[i % 2].T for i in range(9)]) for w in (wg, wu))
    want = act(gate.clamp(max=3.0)) * (up.clamp(-3.0, 3.0) + 0.5)
    out = torch.empty(9, 24, device=DEV)
    ops.moe_gemm(x.to(DEV), wg.to(DEV), out, plan, 1, gather=True, w2=wu.to(DEV), activation=activation, limit=3.0, up_offset=0.5)
    _close(out[plan[2].long()], want, 1e-5)


def test_gated_activation_on_columns_of_a_wider_matrix():
    from rocml_amd import ops
    g = _gen(6)
    wide = torch.randn(7, 50, generator=g) * 2
    gate, up = wide[:, 3:43:2].double(), wide[:, 4:43:2].double()
    gate, up = gate.clamp(max=1.1), up.clamp(-1.1, 1.1)
    out = torch.empty(7, 20, device=DEV)
    ops.swiglu(wide.to(DEV)[:, 3:43], out, interleaved=True, activation="sigmoid_1702", limit=1.1, up_offset=1.0)
    _close(out, gate * torch.sigmoid(1.702 * gate) * (up + 1.0), 1e-6)
