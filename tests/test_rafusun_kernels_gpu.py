"""What Rafusun added to the kernels, each against plain arithmetic (float64 where the inputs are made by hand,
tests/kernel_refs.py otherwise), at sizes of their own, odd ones included, and with inputs made so that a fault
shows: one key whose score stands out at every edge of a chunk, states that are not zero, spans of one token beside
longer ones."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import kernel_refs as R
from kernel_refs import tile_cache, untile_cache
from test_nutavik_kernels_gpu import close, context
from yalis_amd.engine.batch import SeqSpan, attention_tiles, build_host_batch
from yalis_amd.ops.hip import KernelError, SplitSum
from yalis_amd.parts.base import Rotation

pytestmark = pytest.mark.gpu

_ops = {}


def ops():
    if "o" not in _ops:
        from yalis_amd.ops.hip import HipOps

        _ops["o"] = HipOps("cuda:0")
    return _ops["o"]


SPANS = [(0, 9), (30, 1), (7, 2), (12, 21), (0, 1)]
SLOTS = [2, 0, 4, 1, 5]


def step(spans_at=SPANS, slots=SLOTS):
    dev, cpu, _ = context(spans_at, 16, slots=slots)
    dev.max_qlen = cpu.max_qlen = max(n for _, n in spans_at)
    return dev, cpu, sum(n for _, n in spans_at)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [42, 320, 2048])
@pytest.mark.parametrize("buckets,mp,mc", [(61, 19, 7), (1, 3, 5), (97, 2654435761, 1), (50, 0, 1), (100003, 1000003, 7919)])
def test_rows_for_pairs_of_tokens(dtype, width, buckets, mp, mc):
    """Spans of one and of several tokens, behind a token before and as a sequence's first: the row of each pair, the scaled row of
    each token, and what the state then holds."""
    o = ops()
    dev, cpu, n = step()
    g = torch.Generator().manual_seed(width + buckets)
    vocab = 90
    table, pairs = torch.randn(vocab, width, generator=g).to(dtype), torch.randn(buckets + 1, width, generator=g).to(dtype)
    ids = torch.randint(0, vocab, (n,), generator=g, dtype=torch.int32)
    state = torch.randint(0, vocab, (6, 1), generator=g, dtype=torch.int32)
    state[2], state[5] = -1, -1  # sequences that begin with this step
    want_state = state.clone()
    want, _ = R.embed_pairs(ids, table, 3.5, pairs, buckets, mp, mc, want_state, cpu, dtype)
    sd = state.clone().cuda()
    got, rounded = o.embed_pairs(ids.cuda(), table.cuda(), 3.5, pairs.cuda(), buckets, mp, mc, sd, dev, dtype)
    close(got, want, torch.float32, "rows", f32=1e-6)
    assert torch.equal(rounded, got.to(dtype)) and torch.equal(sd.cpu(), want_state)


def unreduced(rows, slices, dtype, g):
    """``rows`` as the unreduced slices of a product."""
    parts = torch.randn(slices - 1, *rows.shape, generator=g)
    parts = torch.cat([parts, (rows.float() - parts.sum(0))[None]])
    return SplitSum(parts.cuda(), dtype), parts.sum(0).to(dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,n", [(40, 5), (42, 3), (320, 37), (1024, 4), (1500, 3), (2048, 9), (4096, 6), (5004, 2), (7000, 2)])
def test_norm_after_the_sum(dtype, width, n):
    """One branch or two, each as it is or normed with a weight of its own, as tensors and as slices (and one of each), with and
    without a weight per element; the stream is written back and its rounded copy handed on."""
    o = ops()
    g = torch.Generator().manual_seed(width + n)
    res = torch.randn(n, width, generator=g) * 2
    a, b = ((torch.randn(n, width, generator=g) * s).to(dtype) for s in (5.0, 0.2))
    mk = lambda: (torch.randn(width, generator=g) * 0.3 + 1).to(dtype)
    w, wa, wb, cw = mk(), mk(), mk(), mk()
    sa, a_sum = unreduced(a, 5, dtype, g)
    sb, b_sum = unreduced(b, 11, dtype, g)
    f = torch.randn(n, width, generator=g)  # (float32 rows beside rows of the activation dtype)
    cuda = lambda t: t.cuda() if torch.is_tensor(t) else t
    cases = [
        ([(a, None, 0.0)], 1.0, None, 3.0), ([(a, None, 0.0)], 1.0, cw, 0.5), ([(sa, None, 0.0)], 1.0, cw, 1.0), ([(a, wa, 1e-5)], 0.5, cw, 2.0),
        ([(a, wa, 1e-5), (b, wb, 1e-5)], 0.5, cw, 3.0), ([(f, None, 0.0), (sb, wb, 1e-5)], 0.5, cw, 3.0), ([(a, wa, 0.1), (sb, wb, 1e-6)], 0.25, None, 1.0),
        ([(sa, wa, 1e-5), (b, None, 0.0)], 1.0, cw, 1.5), ([(a, None, 0.0), (b, None, 0.0)], 2.0, None, 0.0),
    ]
    plain = {id(sa): a_sum, id(sb): b_sum}
    for i, (terms, scale, channel, alpha) in enumerate(cases):
        for offset in (False, True):
            v = torch.zeros(n, width, dtype=torch.float64)
            for rows, tw, e in terms:
                x = plain.get(id(rows), rows).double()
                v += x if tw is None else x / torch.sqrt((x * x).mean(-1, keepdim=True) + e) * tw.double()
            v = alpha * res.double() + scale * v * (1.0 if channel is None else channel.double())
            want = v / torch.sqrt((v * v).mean(-1, keepdim=True) + 1e-5) * (w.double() + (1.0 if offset else 0.0))
            r = res.clone().cuda()
            got = o.sum_norm(r, [(cuda(x), cuda(tw), e) for x, tw, e in terms], scale, cuda(channel), alpha, w.cuda(), 1e-5, offset, dtype)
            close(r, want, torch.float32, f"stream, case {i}", f32=3e-6)
            assert torch.equal(got, r.to(dtype)), f"case {i}: the copy is the stream, rounded"
            ref = res.clone()
            R.sum_norm(ref, [(plain.get(id(x), x), tw, e) for x, tw, e in terms], scale, channel, alpha, w, 1e-5, offset, dtype)
            close(ref, want, torch.float32, "the plain counterpart", f32=3e-6)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,mixes", [(42, 5), (64, 1), (320, 8), (2048, 5)])
def test_inputs_mixed_with_the_token_before(dtype, width, mixes):
    o = ops()
    dev, cpu, n = step()
    g = torch.Generator().manual_seed(width)
    x = torch.randn(n, width, generator=g).to(dtype)
    mu = torch.randn(mixes, width, generator=g)
    state = torch.randn(6, width, generator=g).to(dtype)
    ref, sd = state.clone(), state.clone().cuda()
    want = R.token_shift_mix(x, mu, ref, cpu)
    got = o.token_shift_mix(x.cuda(), mu.cuda(), sd, dev)
    close(got, want, dtype, "mixes", f32=1e-6, bf16=1e-2)
    assert torch.equal(sd.cpu(), ref)
    assert torch.equal(ref[3], state[3]), "a slot outside the step stays as it is"


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [1, 8, 31, 32, 33, 64, 65, 130, 700])
@pytest.mark.parametrize("groups,rows,last,k", [(5, 64, 16, 128), (5, 256, 64, 512), (4, 48, 48, 40), (3, 128, 128, 2048), (5, 21, 5, 42), (2, 192, 100, 64)])
def test_products_of_groups_with_inputs_of_their_own(dtype, n, groups, rows, last, k):
    """Few rows (one launch where the groups allow it), more, and many; groups of odd sizes; a last group with fewer rows."""
    o = ops()
    g = torch.Generator().manual_seed(n + rows)
    x = torch.randn(groups, n, k, generator=g).to(dtype)
    w = (torch.randn((groups - 1) * rows + last, k, generator=g) / k ** 0.5).to(dtype)
    want = torch.cat([x[i].double() @ w[i * rows: (i + 1) * rows].double().T for i in range(groups)], dim=1)
    for out in (dtype, torch.float32):
        got = o.grouped_linear(x.cuda(), w.cuda(), rows, out)
        assert got.dtype == out and tuple(got.shape) == tuple(want.shape)
        close(got, want, out, f"groups, {out}", f32=2e-5, bf16=1e-2)
    close(R.grouped_linear(x, w, rows, torch.float32), want, torch.float32, "the plain counterpart", f32=2e-5)
    with pytest.raises(KernelError):
        o.grouped_linear(x.cuda(), w.cuda(), rows * groups * 2, dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [1, 8, 19, 64, 65, 300])
@pytest.mark.parametrize("rank,cols,act", [(16, 128, "tanh"), (5, 21, "tanh"), (64, 2048, None), (24, 300, "tanh"), (130, 70, None)])
def test_second_products_of_low_rank_pairs(dtype, n, rank, cols, act):
    o = ops()
    g = torch.Generator().manual_seed(n + rank)
    wide = (torch.randn(n, rank + 16, generator=g) * 1.5).to(dtype)
    y = wide[:, 8: 8 + rank]  # a view with a row stride
    w = (torch.randn(cols, rank, generator=g) / rank ** 0.5).to(dtype)
    z = torch.tanh(y.double()) if act else y.double()
    got = o.low_rank(wide.cuda()[:, 8: 8 + rank], w.cuda(), act)
    assert got.dtype == torch.float32
    close(got, z @ w.double().T, dtype, "low rank", f32=1e-5, bf16=1e-2)
    close(R.low_rank(y, w, act), z @ w.double().T, torch.float32, "the plain counterpart", f32=1e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("channels", [52, 64, 1000, 1024])
@pytest.mark.parametrize("taps", [1, 2, 4, 5])
def test_convolution_moves_its_state_on(dtype, channels, taps):
    """Steps of single tokens (the state moves in the same launch) and of longer spans, with and without biases, in pieces of 16
    bytes and channel by channel; more tokens than a thread walks."""
    o = ops()
    g = torch.Generator().manual_seed(taps + channels)
    for spans, slots in ((SPANS, SLOTS), ([(3, 1), (0, 1), (70, 1)], [3, 1, 0]), ([(5, 90)], [2])):
        dev, cpu, n = step(spans, slots)
        x = torch.randn(n, channels + 8, generator=g).to(dtype)[:, :channels]
        w = (torch.randn(channels, taps, generator=g) * 0.5).to(dtype)
        bias = (torch.randn(channels, generator=g) * 0.5).to(dtype)
        for b in (None, bias):
            state = torch.randn(6, max(taps - 1, 1), channels, generator=g).to(dtype)[:, : taps - 1].contiguous()
            ref, sd = state.clone(), state.clone().cuda()
            want = R.causal_conv_act(x, w, b, ref, cpu, act="silu", move_state=True)
            wide = torch.empty(n, channels + 8, dtype=dtype, device="cuda:0")
            wide[:, :channels] = x.cuda()
            got = o.causal_conv(wide[:, :channels], w.cuda(), None if b is None else b.cuda(), sd if taps > 1 else None, dev, act="silu", move_state=True)
            close(got, want, dtype, "convolution", f32=1e-5, bf16=1e-2)
            if taps > 1:
                assert torch.equal(sd.cpu(), ref)
                assert torch.equal(o.causal_conv(wide[:, :channels], w.cuda(), None, sd, dev), o.causal_conv(wide[:, :channels], w.cuda(), None, sd, dev)), "the state moves only when asked"
                assert torch.equal(sd.cpu(), ref)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("kind", ["softplus_delta", "exp_bonus", "softplus_plain", "exp_delta_wide_beta"])
@pytest.mark.parametrize("heads,kv,dim,vdim", [(4, 2, 12, 10), (2, 2, 24, 9), (2, 2, 64, 64), (3, 1, 128, 70), (1, 1, 200, 5), (2, 1, 16, 300), (2, 2, 48, 48), (2, 1, 7, 20), (1, 1, 600, 6)])
def test_scan_with_decays_per_channel_and_the_bonus(dtype, kind, heads, kv, dim, vdim):
    """Both new decays, under the delta rule (beta in the rows' dtype or float32), plain writes, and plain writes read before they
    are made; key channels from fewer than a lane's share to many lanes a column; spans of one token and of several
    staged chunks, behind states that are not zero; and a span cut in two gives the same bits."""
    o = ops()
    if kind == "exp_bonus":
        kv = heads
    spans_at = [(0, 37), (5, 1), (9, 18)]
    dev, cpu, _ = context(spans_at, 16, slots=[1, 3, 0])
    n = sum(k for _, k in spans_at)
    g = torch.Generator().manual_seed(dim + vdim)
    kd = kv * dim
    order = (kd, 0, 2 * kd) if "plain" in kind else (0, kd, 2 * kd)  # (columns need not be q, k, v)
    qkv = torch.randn(n, 2 * kd + heads * vdim + 8 + heads, generator=g).to(dtype)
    beta_col = 2 * kd + heads * vdim + 3
    state = torch.randn(4, heads, dim, vdim, generator=g) * 0.5
    pad = 4 if dim % 4 == 0 else 3
    z = torch.randn(n, heads * dim + pad, generator=g) * 1.5
    vec, a_log = torch.randn(heads * dim, generator=g) - 1.0, torch.randn(heads, generator=g) * 0.5
    bonus = torch.randn(heads, dim, generator=g) * 2
    wide_beta = torch.randn(n, heads + 2, generator=g)

    def args(f):
        decay = ("channel_softplus", f(z), pad, f(a_log), f(vec)) if "softplus" in kind else ("channel_exp", f(z), pad, f(vec))
        beta = None
        if kind == "softplus_delta":
            beta = (f(qkv), beta_col)
        elif kind == "exp_delta_wide_beta":
            beta = (f(wide_beta), 1)
        return dict(q_scale=dim ** -0.5, unit_eps=1e-6 if "delta" in kind else None, decay=decay, beta=beta, columns=order,
                    bonus=f(bonus) if kind == "exp_bonus" else None)

    s_ref = state.clone()
    want = R.linear_state_scan(qkv, heads, kv, dim, vdim, s_ref, cpu, **args(lambda t: t))
    s_dev = state.clone().cuda()
    got = o.linear_state_scan(qkv.cuda(), heads, kv, dim, vdim, s_dev, dev, **args(lambda t: t.cuda()))
    close(got, want, torch.float32, "read-outs", f32=5e-5)
    close(s_dev, s_ref, torch.float32, "states", f32=5e-5)
    assert torch.equal(s_dev[2].cpu(), state[2]), "a slot outside the step stays as it is"
    s_two = state.clone().cuda()
    outs = []
    for p0, cnt, lo in ((0, 20, 0), (20, 17, 20)):
        d2, _, _ = context([(p0, cnt)], 16, slots=[1])
        part = lambda t, lo=lo, cnt=cnt: t[lo: lo + cnt].contiguous().cuda() if t.dim() == 2 and t.shape[0] == n else t.cuda()
        outs.append(o.linear_state_scan(part(qkv), heads, kv, dim, vdim, s_two, d2, **args(part)))
    assert torch.equal(torch.cat(outs), got[:37]) and torch.equal(s_two[1], s_dev[1])


def test_scan_refuses_what_does_not_go_together():
    o = ops()
    dev, _, n = step()
    qkv, state = torch.randn(n, 3 * 16, device="cuda:0"), torch.zeros(6, 2, 8, 8, device="cuda:0")
    z, vec = torch.randn(n, 16, device="cuda:0"), torch.randn(16, device="cuda:0")
    bonus = torch.ones(2, 8, device="cuda:0")
    with pytest.raises(KernelError, match="bonus"):
        o.linear_state_scan(qkv, 2, 2, 8, 8, state, dev, decay=("channel_exp", z, 0, vec), beta=(z, 0), bonus=bonus)
    with pytest.raises(KernelError, match="constants"):
        o.linear_state_scan(qkv, 2, 2, 8, 8, state, dev, decay=("channel_softplus", z, 0, vec, vec))
    with pytest.raises(KernelError, match="unknown kind"):
        o.linear_state_scan(qkv, 2, 2, 8, 8, state, dev, decay=("channel_tanh", z, 0, vec))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,vdim", [(4, 10), (2, 64), (3, 200)])
@pytest.mark.parametrize("gate_dtype,act", [("same", "sigmoid"), ("float32", "sigmoid"), ("float32", "silu")])
def test_read_out_norm_gated_by_the_sigmoid(dtype, heads, vdim, gate_dtype, act):
    o = ops()
    g = torch.Generator().manual_seed(vdim)
    n = 21
    x = torch.randn(n, heads * vdim, generator=g) * 4
    gate = torch.randn(n, heads * vdim + 9, generator=g).to(torch.float32 if gate_dtype == "float32" else dtype)
    for w in ((torch.randn(vdim, generator=g) * 0.3 + 1).to(dtype), (torch.randn(heads * vdim, generator=g) * 0.3 + 1).to(dtype)):
        want = R.gated_head_norm(x, w, 1e-5, gate, 9, heads, vdim, dtype, gate_act=act)
        got = o.gated_head_norm(x.cuda(), w.cuda(), 1e-5, gate.cuda(), 9, heads, vdim, dtype, gate_act=act)
        close(got, want, dtype, "head norm", bf16=1e-2)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,kv,dim,vdim,page,n", [(4, 2, 8, 8, 16, 5), (3, 3, 10, 6, 16, 40), (4, 2, 64, 64, 64, 37), (8, 2, 128, 128, 64, 20), (2, 1, 80, 96, 32, 3)])
def test_prepare_with_a_norm_without_weights(dtype, heads, kv, dim, vdim, page, n):
    """Neighbours rotate on the first elements of a head, and queries and keys are divided by their root mean square: before the
    rotation, which is the same as after it (the plain counterpart here norms after)."""
    o = ops()
    g = torch.Generator().manual_seed(heads * dim + n)
    nq, nk = heads * dim, kv * dim
    proj = (torch.randn(n, nq + nk + kv * vdim + 5, generator=g) * 3).to(dtype)
    dev, cpu, n_pages = context([(3, n)], page)
    rot = dim // 4 * 2
    angle = torch.outer(torch.arange(n + 8, dtype=torch.float32), 50.0 ** (-torch.arange(0, rot, 2, dtype=torch.float32) / rot))
    table = Rotation(torch.cos(angle), torch.sin(angle), rot, True)
    on_dev = Rotation(table.cos.cuda(), table.sin.cuda(), rot, True)
    kc, vc = torch.zeros(n_pages, kv, page, dim, dtype=dtype).cuda(), torch.zeros(n_pages, kv, vdim, page, dtype=dtype).cuda()
    got = o.qkv_prepare(proj.cuda(), heads, kv, dim, vdim, dev.arrays["positions"], dtype, qk_eps=1e-5, rotation=on_dev, k_cache=kc, v_cache=vc,
                        slots=dev.arrays["slots_g0"], page_size=page, unweighted_norm=True)
    pos, slots = cpu.arrays["positions"].long(), cpu.arrays["slots_g0"].long()

    def turned_then_normed(x):
        x = R._turn(x.double(), table.cos[pos][:, None, :].double(), table.sin[pos][:, None, :].double(), rot, True)
        return x / torch.sqrt((x * x).mean(-1, keepdim=True) + 1e-5)

    want_q = turned_then_normed(proj[:, :nq].view(n, heads, dim))
    want_k = turned_then_normed(proj[:, nq: nq + nk].view(n, kv, dim))
    close(got.view(n, heads, dim), want_q, dtype, "queries", f32=3e-6, bf16=1e-2)
    kc, vc = kc.cpu(), vc.cpu()
    if o.masked_pages_tiled(dtype, dim, vdim, page):
        kc, vc = untile_cache(kc, vc)
    close(kc[slots // page, :, slots % page], want_k, dtype, "keys in the pages", f32=3e-6, bf16=1e-2)
    close(vc[slots // page, :, :, slots % page], proj[:, nq + nk: nq + nk + kv * vdim].view(n, kv, vdim), dtype, "values in the pages", f32=1e-6, bf16=1e-6)
    kr, vr = torch.zeros(n_pages, kv, page, dim, dtype=dtype), torch.zeros(n_pages, kv, vdim, page, dtype=dtype)
    ref = R.qkv_prepare(proj, heads, kv, dim, vdim, pos, dtype, qk_eps=1e-5, rotation=table, k_cache=kr, v_cache=vr, slots=slots, page_size=page,
                        unweighted_norm=True)
    close(got, ref, dtype, "against the plain counterpart", f32=3e-6, bf16=1e-2)


def chunked_attention(q, k, v, positions, heads_per_kv, scale, softcap, chunk, sink):
    """q [N, H, d] at ``positions``; k [L, G, d], v [L, G, dv] of one sequence: float64, a dense mask."""
    j = torch.arange(k.shape[0])
    mask = (j[None, :] <= positions[:, None]) & (j[None, :] // chunk == positions[:, None] // chunk)
    out = torch.empty(q.shape[0], q.shape[1], v.shape[2], dtype=torch.float64)
    for h in range(q.shape[1]):
        g = h // heads_per_kv
        s = (q[:, h].double() @ k[:, g].double().T) * scale
        if softcap:
            s = softcap * torch.tanh(s / softcap)
        s = s.masked_fill(~mask, -float("inf"))
        if sink is not None:
            s = torch.cat([s, sink[h].double().expand(q.shape[0], 1)], dim=1)
        out[:, h] = torch.softmax(s, dim=-1)[:, : k.shape[0]] @ v[:, g].double()
    return out


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("head_dim,value_dim,heads,kv", [(64, 64, 4, 2), (128, 128, 6, 1), (32, 48, 4, 4), (64, 64, 2, 2), (128, 128, 40, 2)])
@pytest.mark.parametrize("chunk,special", [(64, 576), (64, 639), (96, 575), (96, 576), (100, 599), (100, 600), (257, 513), (257, 514), (37, 592), (300, 300),
                                           (5, 599), (1, 600), (1000, 0)])
def test_chunks_at_every_edge(dtype, head_dim, value_dim, heads, kv, chunk, special):
    """One key's score towers over the rest, the first or the last of its chunk or the one before: a prompt's portion at positions
    550..699 and single tokens in the same chunk, at its end and just beyond look for it, from pages of which those
    below the chunk have been given back.  The general kernel at every size, the matrix-core kernels (bfloat16, keys and values
    of 64 or 128 alike) whole and with their keys split; with a sink and a cap, and without."""
    o = ops()
    H, G, d, dv, page, L = heads, kv, head_dim, value_dim, 64, 700
    scale = 0.2
    gen = torch.Generator().manual_seed(special + heads)
    k = torch.randn(L, G, d, generator=gen) * 0.1
    v = torch.randn(L, G, dv, generator=gen)
    k[special, :, 0] = 40.0
    k, v = k.to(dtype).float(), v.to(dtype).float()
    end = special // chunk * chunk + chunk
    singles = sorted({p for p in (special, special + 1, end - 1, end, end + 1, 599, 600, 0) if 0 <= p < L})
    spans_at = [(550, 150), (560, 3), (595, 20)] + [(p, 1) for p in singles]
    n_pages = sum(-(-(p0 + n) // page) for p0, n in spans_at)
    perm = torch.randperm(n_pages, generator=gen).tolist()
    kc, vc = torch.full((n_pages, G, page, d), float("nan")), torch.full((n_pages, G, dv, page), float("nan"))
    kc[0], vc[0] = 7.0, 7.0  # (what a page that was given back points at)
    spans, used = [], 0
    for p0, n in spans_at:
        need = -(-(p0 + n) // page)
        table = np.array(perm[used: used + need], dtype=np.int32)
        used += need
        gone = p0 // chunk * chunk // page  # whole pages below the first token's chunk
        table[:gone] = -1
        for j in range(gone * page, p0 + n):
            kc[table[j // page], :, j % page] = k[j]
            vc[table[j // page], :, :, j % page] = v[j]
        spans.append(SeqSpan(tokens=[0] * n, first_position=p0, block_tables=[table], state_slot=len(spans), want=[]))
    kc, vc = torch.nan_to_num(kc, nan=3.0), torch.nan_to_num(vc, nan=3.0)  # (finite, and wrong wherever it is read as a key that counts)
    hb = build_host_batch(spans, 1, page)
    positions = torch.from_numpy(hb.positions).long()
    q = torch.randn(hb.n_tokens, H, d, generator=gen) * 0.1
    q[:, :, 0] = 1.0
    q = q.to(dtype).float()
    dev = "cuda:0"
    arrays = {"positions": torch.from_numpy(hb.positions).to(dev), "token_seq": torch.from_numpy(hb.token_seq).to(dev),
              "block_table_g0": torch.from_numpy(hb.block_tables[0]).to(dev)}
    ctx = SimpleNamespace(arrays=arrays, max_ctx=hb.max_ctx, host=hb)
    kc_d, vc_d = kc.to(dtype), vc.to(dtype)
    if o.masked_pages_tiled(dtype, d, dv, page):
        kc_d, vc_d = tile_cache(kc_d, vc_d)
    kc_d, vc_d = kc_d.to(dev).contiguous(), vc_d.to(dev).contiguous()
    qd = q.to(dtype).reshape(hb.n_tokens, H * d).to(dev)
    tol = 2e-4 if dtype == torch.float32 else 4e-2
    for softcap, sink in ((0.0, None), (15.0, torch.zeros(H)), (0.0, torch.full((H,), 6.0))):
        want = chunked_attention(q, k, v, positions, H // G, scale, softcap, chunk, sink)
        sink_d = None if sink is None else sink.to(dev)
        got = o.attention_masked(qd, H, G, d, dv, kc_d, vc_d, page, scale, ctx, 0, window=chunk, chunked=True, softcap=softcap, sink=sink_d)
        err = (got.float().cpu().view(-1, H, dv).double() - want).abs().max(dim=2).values.max(dim=1).values
        assert err.max() < tol, f"general kernel: position {int(positions[int(err.argmax())])} differs by {err.max():.3e}"
        if dtype == torch.bfloat16 and d == dv and d in (64, 128):
            tpt, big = o.attention_tokens_per_tile(H, G), o.attention_long_span_tile(H, G)
            tiles = torch.from_numpy(attention_tiles(hb, tpt, 1, big)).to(dev)
            for col_tiles, (plan, long_plan) in ((1, (None, None)), (2, ((4, 3), 2)), (1, ((1, 1), 1)), (2, ((1, 5), 3))):
                tile = o.attention_long_span_tile(H, G, col_tiles)
                long_tiles = torch.from_numpy(attention_tiles(hb, tile, big + 1, longest_first=True)).to(dev)
                got = o.attention(qd, H, G, d, kc_d, vc_d, page, scale, chunk, ctx, 0, tiles, long_tiles, plan=plan, long_plan=long_plan,
                                  long_col_tiles=col_tiles, softcap=softcap, sink=sink_d, chunked=True)
                err = (got.float().cpu().view(-1, H, d).double() - want).abs().max(dim=2).values.max(dim=1).values
                assert err.max() < tol, f"matrix cores, plan {plan}/{long_plan}: position {int(positions[int(err.argmax())])} differs by {err.max():.3e}"
