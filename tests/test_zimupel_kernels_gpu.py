"""What Zimupel added to the kernels, each against plain arithmetic (float64 where the inputs are made by hand,
tests/kernel_refs.py otherwise), at sizes of their own, odd ones included, and with inputs made so that a fault shows: keys
whose scores stand out in one map only, states that are not zero, spans of one token beside longer ones, ties and negative
choice scores."""
from types import SimpleNamespace

import numpy as np
import pytest
import torch

import kernel_refs as R
from kernel_refs import tile_cache, untile_cache
from test_nutavik_kernels_gpu import close, context
from yalis_amd.engine.batch import SeqSpan, attention_tiles, build_host_batch, chunk_starts, span_chunks
from yalis_amd.ops.hip import KernelError, SplitSum
from yalis_amd.parts.base import Rotation

pytestmark = pytest.mark.gpu

_ops = {}


def ops():
    if "o" not in _ops:
        from yalis_amd.ops.hip import HipOps

        _ops["o"] = HipOps("cuda:0")
    return _ops["o"]


# ------------------------------------------------------------------------------------------- a stream kept as copies
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width", [42, 64, 320, 2048, 4608])
@pytest.mark.parametrize("copies", [1, 3, 4, 6, 11])
def test_streams_norm(dtype, width, copies):
    """Nothing pending; a tensor, a product's slices, a mixture's rows (with weights and without), and both at once, mixed into
    the copies in place; picked rows, which leave the copies alone; the plain sum in place of a weighted one."""
    o = ops()
    g = torch.Generator().manual_seed(width + copies)
    n, top = 21, 3
    res = torch.randn(n, copies, width, generator=g) * 2
    y = torch.randn(n, width, generator=g).to(dtype)
    slices = torch.randn(5, n, width, generator=g)
    rows, rw = torch.randn(n * top, width, generator=g), torch.rand(n, top, generator=g)
    mix, out, read = torch.randn(copies, copies, generator=g), torch.randn(copies, generator=g), torch.randn(copies, generator=g)
    w = (torch.randn(width, generator=g) * 0.3 + 1).to(dtype)
    picked = torch.tensor([4, 0, 20, 4], dtype=torch.int32)
    d = lambda t: None if t is None else t.cuda()
    split = lambda device: SplitSum(slices.to(device), dtype)
    cases = [(None, None, False, read, None), (None, None, False, None, picked), (y, None, True, read, None), ("slices", None, True, read, None),
             (None, (rows, top, 1.0, rw), True, read, None), (y, (rows, top, 0.5, None), True, None, None), (y, (rows, top, 1.0, rw), True, None, picked),
             ("slices", None, True, None, picked)]
    for branch, experts, joins, r, pick in cases:
        want_res = res.double().clone()
        b = None if branch is None else (slices.double().sum(0).to(dtype) if branch == "slices" else branch)
        want = R.streams_norm(want_res, None if b is None else b.double(), None if experts is None else tuple(t.double() if torch.is_tensor(t) else t for t in experts),
                              mix.double() if joins else None, out.double() if joins else None, None if r is None else r.double(), pick, w.double(), 1e-5,
                              False, torch.float64)
        got_res = res.clone().cuda()
        got = o.streams_norm(got_res, split("cuda:0") if branch == "slices" else d(branch), None if experts is None else tuple(d(t) if torch.is_tensor(t) else t for t in experts),
                             d(mix) if joins else None, d(out) if joins else None, d(r), d(pick), d(w), 1e-5, False, dtype)
        assert got.dtype == dtype and tuple(got.shape) == (n if pick is None else 4, width)
        close(got, want, dtype, "norm", f32=1e-5, bf16=1e-2)
        # (slices are summed in another order than above before they are rounded: a bfloat16's last bit)
        close(got_res, want_res, torch.float32, "copies", f32=1e-5 if branch != "slices" or dtype == torch.float32 else 2e-3)
    with pytest.raises(KernelError):
        o.streams_norm(res.cuda(), None, None, d(mix)[:, :0], d(out), d(read), None, d(w), 1e-5, False, dtype)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("width,copies", [(42, 3), (64, 1), (2048, 4), (5000, 2)])
def test_embed_norm(dtype, width, copies):
    o = ops()
    g = torch.Generator().manual_seed(width)
    table, w = (torch.randn(50, width, generator=g) * 3).to(dtype), torch.randn(width, generator=g).to(dtype)
    ids = torch.randint(0, 50, (33,), generator=g, dtype=torch.int32)
    x = table[ids.long()].double()
    want = (x / torch.sqrt((x * x).mean(-1, keepdim=True) + 0.3) * w.double())[:, None, :].repeat(1, copies, 1)
    got = o.embed_norm(ids.cuda(), table.cuda(), w.cuda(), 0.3, copies)
    assert got.dtype == torch.float32
    close(got, want, torch.float32, "rows", f32=2e-6)


@pytest.mark.parametrize("cap", [0.0, 3.0])
def test_scaled_and_capped_rows(cap):
    o = ops()
    x = torch.linspace(-40, 40, 1001).repeat(3, 1).contiguous()
    want = x.double() * 0.7
    if cap:
        want = cap * torch.tanh(want / cap)
    close(o.scale_rows(x.cuda(), 0.7, softcap=cap), want, torch.float32, "rows", f32=1e-6)


# ------------------------------------------------------------------------------------------------ attention of two maps
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("n", [3, 40])
@pytest.mark.parametrize("H,G,part,dv,page", [(4, 2, 32, 64, 64), (3, 1, 64, 128, 16), (6, 2, 5, 7, 16), (2, 2, 16, 48, 32)])
def test_query_rows_per_map(dtype, n, H, G, part, dv, page):
    """Biased queries, keys and values; a row per map with zeros where the other map's elements are; the pages as ever."""
    o = ops()
    g = torch.Generator().manual_seed(H + n)
    d = 2 * part
    dev, cpu, n_pages = context([(5, n), (0, 1)], page)
    N = n + 1
    cols = H * d + G * (d + dv)
    proj = torch.randn(N, cols, generator=g).to(dtype)
    bias = torch.randn(cols, generator=g)
    kc, vc = torch.zeros(n_pages, G, page, d, dtype=dtype), torch.zeros(n_pages, G, dv, page, dtype=dtype)
    want = R.qkv_prepare(proj, H, G, d, dv, cpu.arrays["positions"], dtype, k_cache=kc, v_cache=vc, slots=cpu.arrays["slots_g0"], page_size=page, bias=bias, query_maps=2)
    kd, vd = torch.zeros_like(kc).cuda(), torch.zeros_like(vc).cuda()
    got = o.qkv_prepare(proj.cuda(), H, G, d, dv, dev.arrays["positions"], dtype, k_cache=kd, v_cache=vd, slots=dev.arrays["slots_g0"], page_size=page,
                        bias=bias.cuda(), query_maps=2)
    assert tuple(got.shape) == (N, 2 * H * d)
    close(got, want, dtype, "queries", f32=1e-6, bf16=8e-3)
    rows = got.view(N, H, 2, d)
    assert (rows[:, :, 0, part:] == 0).all() and (rows[:, :, 1, :part] == 0).all()
    kd, vd = kd.cpu(), vd.cpu()
    if o.masked_pages_tiled(dtype, d, dv, page):
        kd, vd = untile_cache(kd, vd)
    close(kd, kc, dtype, "keys", f32=1e-6, bf16=8e-3)
    close(vd, vc, dtype, "values", f32=1e-6, bf16=8e-3)


def two_map_attention(q, k, v, positions, scale, lam, eps, gain):
    """q [N, H, 2, part], k [keys, G, 2, part], v [keys, G, dv], one request's keys at hand; float64."""
    N, H = q.shape[:2]
    per = H // k.shape[1]
    out = torch.zeros(N, H, v.shape[-1], dtype=torch.float64)
    for t in range(N):
        p = int(positions[t])
        for h in range(H):
            a = [torch.softmax((k[: p + 1, h // per, m].double() @ q[t, h, m].double()) * scale, 0) @ v[: p + 1, h // per].double() for m in (0, 1)]
            o = a[0] - lam * a[1]
            out[t, h] = o / torch.sqrt((o * o).mean() + eps) * gain
    return out


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("H,G,part,dv,page", [(4, 2, 32, 64, 64), (2, 1, 64, 128, 64), (24, 2, 32, 64, 64), (6, 2, 32, 64, 16), (3, 3, 64, 128, 32),
                                              (10, 1, 64, 128, 64), (3, 1, 5, 7, 16), (4, 2, 16, 48, 32)])
def test_attention_of_two_maps(dtype, H, G, part, dv, page):
    """One key towers in the first map and another in the second, at borders of pages and of blocks of keys, among the first
    keys and far back; long and short spans and single tokens; whole and split keys."""
    o = ops()
    gen = torch.Generator().manual_seed(H * part)
    d, L = 2 * part, 330
    k, v = torch.randn(L, G, 2, part, generator=gen) * 0.3, torch.randn(L, G, dv, generator=gen)
    for m, at in ((0, [0, 15, 64, 127, 200, 319]), (1, [1, 16, 63, 128, 255])):
        for i, j in enumerate(at):
            k[j, :, m, (i + 1) % part] = 6.0
    k, v = k.to(dtype).float(), v.to(dtype).float()
    scale, lam, eps, gain = 1.7, 0.6, 1e-3, 0.7
    pages = -(-L // page)
    perm = torch.randperm(pages, generator=gen)
    kc, vc = torch.full((pages, G, page, d), 7.0), torch.full((pages, G, dv, page), 7.0)
    for j in range(L):
        kc[perm[j // page], :, j % page] = k[j].reshape(G, d)
        vc[perm[j // page], :, :, j % page] = v[j]
    table = perm.numpy().astype(np.int32)
    spans = [SeqSpan(tokens=[0] * n, first_position=p0, block_tables=[table], state_slot=i, want=[])
             for i, (p0, n) in enumerate([(0, 1), (329, 1), (200, 1), (63, 2), (120, 12), (1, 150), (180, 150)])]
    hb = build_host_batch(spans, 1, page)
    positions = torch.from_numpy(hb.positions).long()
    q = (torch.randn(hb.n_tokens, H, 2, part, generator=gen) * 0.5).to(dtype).float()
    for t in range(hb.n_tokens):
        q[t, :, 0, (t % 6 + 1) % part] = 2.0
        q[t, :, 1, (t % 5 + 1) % part] = 2.0
    want = two_map_attention(q, k, v, positions, scale, lam, eps, gain)
    assert (want - two_map_attention(q.flip(2), k, v, positions, scale, lam, eps, gain)).abs().max() > 0.5, "the maps were meant to differ"
    dev = "cuda:0"
    arrays = {"positions": torch.from_numpy(hb.positions).to(dev), "token_seq": torch.from_numpy(hb.token_seq).to(dev),
              "block_table_g0": torch.from_numpy(hb.block_tables[0]).to(dev)}
    ctx = SimpleNamespace(arrays=arrays, max_ctx=hb.max_ctx, host=hb)
    kc_d, vc_d = kc.to(dtype), vc.to(dtype)
    if o.masked_pages_tiled(dtype, d, dv, page):
        kc_d, vc_d = tile_cache(kc_d, vc_d)
    kc_d, vc_d = kc_d.to(dev).contiguous(), vc_d.to(dev).contiguous()
    tol = 2e-4 if dtype == torch.float32 else 6e-2
    maps = (lam, eps, gain)
    got = o.attention_masked(q.to(dtype).reshape(hb.n_tokens, H * d).to(dev), H, G, d, dv, kc_d, vc_d, page, scale, ctx, 0, differential=maps)
    err = (got.float().cpu().view(-1, H, dv).double() - want).abs().max(dim=2).values.max(dim=1).values
    assert err.max() < tol, f"general kernel: position {int(positions[int(err.argmax())])} differs by {err.max():.3e}"
    if dtype == torch.bfloat16 and d == dv and d in (64, 128):
        assert o.attention_takes_maps(dtype, d)
        rows = torch.zeros(hb.n_tokens, H, 2, d)
        rows[:, :, 0, :part], rows[:, :, 1, part:] = q[:, :, 0], q[:, :, 1]
        qd = rows.to(dtype).reshape(hb.n_tokens, 2 * H * d).to(dev)
        tpt, big = o.attention_tokens_per_tile(2 * H, G), o.attention_long_span_tile(2 * H, G)
        big2 = o.attention_long_span_tile(2 * H, G, 2)
        tiles = torch.from_numpy(attention_tiles(hb, tpt, 1, big)).to(dev)
        for plan, long_plan, cols in ((None, None, 1), ((4, 3), 2, 1), ((1, 1), 1, 2), ((1, 5), 3, 2)):
            long_tiles = torch.from_numpy(attention_tiles(hb, big if cols == 1 else big2, big + 1, longest_first=True)).to(dev)
            got = o.attention(qd, 2 * H, G, d, kc_d, vc_d, page, scale, 0, ctx, 0, tiles, long_tiles, plan=plan, long_plan=long_plan, long_col_tiles=cols,
                              differential=maps)
            assert tuple(got.shape) == (hb.n_tokens, H * d)
            err = (got.float().cpu().view(-1, H, d).double() - want).abs().max(dim=2).values.max(dim=1).values
            assert err.max() < tol, f"matrix cores, plan {plan}/{long_plan}/{cols}: position {int(positions[int(err.argmax())])} differs by {err.max():.3e}"


# --------------------------------------------------------------------------------------------- memories with fixed decays
def fixed_step(spans_at, slots):
    dev, cpu, _ = context(spans_at, 16, slots=slots)
    hb = build_host_batch([SeqSpan(tokens=[0] * n, first_position=p0, block_tables=[np.arange(64, dtype=np.int32)], state_slot=s, want=[])
                           for (p0, n), s in zip(spans_at, slots)], 1, 16)
    dev.max_qlen = cpu.max_qlen = max(n for _, n in spans_at)
    return dev, cpu, torch.from_numpy(span_chunks(hb, 64)).cuda(), torch.from_numpy(chunk_starts(hb, 64)).cuda(), sum(n for _, n in spans_at)


SCANS = [  # heads' decays, dim, vdim, rotated elements, interleaved, activation
    ([0.3, 0.999, 0.9], 64, 32, 64, False, None), ([0.9, 0.0], 32, 32, 0, False, "silu"), ([1.0, 0.99], 128, 48, 32, False, None),
    ([0.97], 256, 144, 128, False, None), ([0.5, 0.9995], 128, 128, 0, False, "silu"), ([0.8, 0.99], 64, 16, 24, True, None),
    ([0.9, 0.2, 0.99], 10, 6, 6, False, None), ([0.95, 0.5], 7, 5, 0, False, "silu"), ([0.9], 48, 20, 48, False, None), ([0.99], 300, 12, 0, False, "silu"),
]


def scan_inputs_for(decay, dim, vdim, rot, inter, n, gen, dtype):
    H = len(decay)
    proj = torch.randn(n, H * (2 * dim + vdim) + 8, generator=gen).to(dtype)
    rotation = None
    if rot:
        ang = torch.outer(torch.arange(700.0), 300.0 ** (-torch.arange(0, rot, 2) / rot))
        rotation = Rotation(ang.cos().contiguous(), ang.sin().contiguous(), rot, inter)
    return proj, rotation, torch.tensor(decay, dtype=torch.float32), torch.randn(6, H, dim, vdim, generator=gen)


def on_gpu(r):
    return None if r is None else Rotation(r.cos.cuda(), r.sin.cuda(), r.rotary_dim, r.interleaved)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("case", SCANS)
def test_fixed_decay_scan(dtype, case):
    """Unequal spans behind states that are not zero, in every form that takes the sizes: walked token by token, in chunks on the
    matrix cores (all at once, and in slabs of two chunks), and a step of single tokens."""
    o = ops()
    decay, dim, vdim, rot, inter, act = case
    H = len(decay)
    gen = torch.Generator().manual_seed(dim + vdim)
    slots = [5, 2, 0, 1, 4, 3]
    dev, cpu, chunks, starts, n = fixed_step([(9, 1), (0, 70), (3, 64), (100, 2), (50, 200), (0, 129)], slots)
    proj, rotation, a, state = scan_inputs_for(decay, dim, vdim, rot, inter, n, gen, dtype)
    want_state = state.double().clone()
    rows = R.scan_inputs(proj, H, dim, vdim, dim ** -0.5, rotation, cpu.arrays["positions"], act).double()
    want = torch.zeros(n, H, vdim, dtype=torch.float64)
    kd = H * dim
    for s in range(6):
        q0, ql = int(cpu.arrays["seq_qstart"][s]), int(cpu.arrays["seq_qlen"][s])
        S = want_state[slots[s]].clone()
        for t in range(q0, q0 + ql):
            q, k, v = rows[t, :kd].view(H, dim), rows[t, kd: 2 * kd].view(H, dim), rows[t, 2 * kd:].view(H, vdim)
            S = a.double()[:, None, None] * S + k[:, :, None] * v[:, None, :]
            want[t] = torch.einsum("hde,hd->he", S, q)
        want_state[slots[s]] = S
    takes_chunks = dtype == torch.bfloat16 and dim in (32, 64, 128, 256) and vdim % 16 == 0
    forms = ["walk"] + (["chunks", "slabs"] if takes_chunks else [])
    for form in forms:
        sd = state.clone().cuda()
        slab = o.DECAY_SLAB_BYTES
        if form == "slabs":
            o.DECAY_SLAB_BYTES = 2 * 4 * H * dim * vdim
        try:
            got = o.fixed_decay_scan(proj.cuda(), H, dim, vdim, sd, dev, a.cuda(), k_scale=dim ** -0.5, rotation=on_gpu(rotation), act=act, chunks=chunks,
                                     seq_chunk0=starts, form="chunks" if form == "slabs" else form)
        finally:
            o.DECAY_SLAB_BYTES = slab
        close(got.view(n, H, vdim), want, torch.float32, f"{form}: read-outs", f32=2e-5)
        close(sd, want_state, torch.float32, f"{form}: memories", f32=2e-5)
    if not takes_chunks:
        with pytest.raises(KernelError):
            o.fixed_decay_scan(proj.cuda(), H, dim, vdim, state.cuda(), dev, a.cuda(), act=act, chunks=chunks, seq_chunk0=starts, form="chunks")
    # single tokens
    dev, cpu, chunks, starts, n = fixed_step([(9, 1), (0, 1), (3, 1), (100, 1), (50, 1), (0, 1)], slots)
    sd, sw = state.clone().cuda(), state.clone()
    want = R.fixed_decay_scan(proj[:n], H, dim, vdim, sw, cpu, a, k_scale=dim ** -0.5, rotation=rotation, act=act)
    got = o.fixed_decay_scan(proj[:n].cuda(), H, dim, vdim, sd, dev, a.cuda(), k_scale=dim ** -0.5, rotation=on_gpu(rotation), act=act, chunks=chunks,
                             seq_chunk0=starts)
    close(got, want, torch.float32, "a step of single tokens", f32=2e-6)
    close(sd, sw, torch.float32, "memories after it", f32=2e-6)


def test_a_cut_leaves_the_memory_as_it_is():
    """A span whole and in two, cut inside a chunk and at its edge: the same read-outs and memory up to what is lost when float32
    numbers enter the matrix cores as two bfloat16 parts."""
    o = ops()
    gen = torch.Generator().manual_seed(7)
    decay, dim, vdim = [0.9, 0.9995], 128, 64
    proj, _, a, state = scan_inputs_for(decay, dim, vdim, 0, False, 180, gen, torch.bfloat16)
    run = lambda rows, p0, sd: o.fixed_decay_scan(rows.cuda(), 2, dim, vdim, sd, *(lambda c: (c[0], a.cuda(), 1.0, None, "silu", c[2], c[3]))(
        fixed_step([(p0, rows.shape[0])], [3])))
    whole_state = state.clone().cuda()
    whole = run(proj, 0, whole_state)
    for cut in (1, 64, 100, 179):
        sd = state.clone().cuda()
        got = torch.cat([run(proj[:cut].contiguous(), 0, sd), run(proj[cut:].contiguous(), cut, sd)])
        close(got, whole, torch.float32, f"cut at {cut}", f32=2e-5)
        close(sd, whole_state, torch.float32, f"memory, cut at {cut}", f32=2e-5)


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("heads,vdim", [(3, 7), (4, 64), (2, 256), (1, 2048), (1, 1500), (5, 1020)])
@pytest.mark.parametrize("gate_act,gate_first", [("silu", False), ("sigmoid", False), ("silu", True)])
def test_gated_head_norm_forms(dtype, heads, vdim, gate_act, gate_first):
    """No weight, a weight for all parts, a weight as wide as the row; parts of a wave and of a workgroup; columns that start anywhere."""
    o = ops()
    g = torch.Generator().manual_seed(vdim)
    n = 9
    x = torch.randn(n, heads * vdim, generator=g) * 2
    for col in (0, 8, 3):
        gate = torch.randn(n, heads * vdim + 11, generator=g).to(dtype)
        for weight in (None, torch.randn(vdim, generator=g).to(dtype), torch.randn(heads * vdim, generator=g).to(dtype)):
            gf = gate[:, col: col + heads * vdim].double().view(n, heads, vdim)
            act = torch.sigmoid(gf) * (gf if gate_act == "silu" else 1.0)
            y = x.double().view(n, heads, vdim) * (act if gate_first else 1.0)
            y = y / torch.sqrt((y * y).mean(-1, keepdim=True) + 1e-4)
            if weight is not None:
                y = y * (weight.double() if weight.numel() == vdim else weight.double().view(heads, vdim))
            want = (y if gate_first else y * act).reshape(n, -1)
            got = o.gated_head_norm(x.cuda(), None if weight is None else weight.cuda(), 1e-4, gate.cuda(), col, heads, vdim, dtype, gate_first=gate_first,
                                    gate_act=gate_act)
            close(got, want, dtype, "read-out", f32=1e-5, bf16=8e-3)


# ------------------------------------------------------------------------------------------------------- the router
@pytest.mark.parametrize("n,experts,top,padded,groups", [(1, 2, 1, 16, None), (37, 12, 4, 16, (2, 1)), (200, 8, 8, 8, (4, 4)), (64, 40, 3, 48, (10, 4)),
                                                         (9, 130, 6, 144, (13, 2)), (50, 6, 2, 16, (6, 3)), (5, 256, 8, 256, (8, 4)), (33, 9, 5, 16, None)])
def test_router_with_shares_and_groups(n, experts, top, padded, groups):
    """Corrections that make most choice scores negative (a dropped group counts as minus infinity, not zero), that decide who is
    chosen and weigh nothing; ties go to the lower number, of experts and of groups; padding columns are no experts."""
    o = ops()
    g = torch.Generator().manual_seed(n + experts)
    logits = torch.randn(n, padded, generator=g) * 1.5
    logits[:, experts:] = 50.0
    correction = torch.randn(experts, generator=g) * 0.5 - 0.8
    bias = torch.randn(experts, generator=g) * 0.5
    for b in (None, bias):
        choice, weights = o.moe_router_share(logits.cuda(), top, experts=experts, bias=None if b is None else b.cuda(), correction=correction.cuda(), groups=groups)
        want_choice, want_w = R.moe_router_share(logits, top, experts=experts, bias=b, correction=correction, groups=groups)
        # (close calls of float32 sums aside, the same experts in the same order)
        same = (choice.cpu() == want_choice).all(1)
        assert same.float().mean() > 0.97, "the choice"
        close(weights.cpu()[same], want_w[same], torch.float32, "weights", f32=3e-6)
        assert (weights.sum(1).cpu() - 1).abs().max() < 1e-5
        if groups is not None:
            size = experts // groups[0]
            assert all(len({int(e) // size for e in row}) <= groups[1] for row in choice.cpu())
    plain = R.moe_router_share(logits, top, experts=experts, correction=torch.zeros(experts), groups=groups)[0]
    assert n == 1 or top == experts or not torch.equal(torch.sort(plain, 1).values, torch.sort(R.moe_router_share(logits, top, experts=experts, correction=correction, groups=groups)[0], 1).values)
    tied = torch.zeros(2, padded)
    choice, weights = o.moe_router_share(tied.cuda(), top, experts=experts, groups=groups)
    assert choice.cpu().tolist() == [list(range(top))] * 2 and (weights.cpu() - 1 / top).abs().max() < 1e-6
    with pytest.raises(KernelError):
        o.moe_router_share(logits.cuda(), top, experts=experts, groups=(experts + 1, 1))
