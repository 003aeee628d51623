"""Rafusun in the engine against the plain implementation (tests/plain_rafusun.py): every way of cutting the work,
on the CPU with plain PyTorch ops (the host side: batching, paging, states, the order of parts) and, marked ``gpu``, with
the HIP kernels in true float32 and in bfloat16."""
import copy
import json
import os

import pytest
import torch

import plain_rafusun as P
import rafusun_cases as X
import replay_cases as C
from kernel_refs import RefOps

BACKENDS = [
    pytest.param(("cpu", "float32"), id="cpu-ref-f32"),
    pytest.param(("cuda:0", "float32"), id="hip-f32", marks=pytest.mark.gpu),
    pytest.param(("cuda:0", "bfloat16"), id="hip-bf16", marks=pytest.mark.gpu),
]
_ops = {}
_plain = {}


def ops_for(device):
    if device == "cpu":
        return RefOps()
    if device not in _ops:
        from yalis_amd.ops.hip import HipOps

        _ops[device] = HipOps(device)
    return _ops[device]


def setup(name):
    cfg = X.CONFIGS[name]
    if name not in _plain:
        weights = X.random_weights(cfg, seed=len(name), ranks=X.RANKS[name])
        reqs = X.make_requests(cfg, X.LENGTHS[name], seed=10)
        _plain[name] = (weights, reqs, X.plain_logits(cfg, weights, reqs))
    return (cfg, *_plain[name])


TRACES = {"whole": C.trace_whole, "tail": C.trace_tail, "one_by_one": lambda r: C.trace_tail(r, tail=1 << 20),
          "portions": C.trace_portions, "mixed": C.trace_mixed, "random": lambda r: C.trace_random(r, 5)}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["odd", "mix", "wide"])
@pytest.mark.parametrize("mode", list(TRACES))
def test_replay_modes(backend, name, mode):
    """Whole prompts; a prompt and then its last tokens one by one; every token one by one (prefill against
    decoding); portions down to two tokens; up to four unequal requests a step in a pool so small that pages and slots
    are used again; cuts at random."""
    device, dtype = backend
    if device == "cpu" and (name == "wide" or (name == "mix" and mode not in ("whole", "mixed", "portions"))):
        pytest.skip("the plain ops are slow at this size; the GPU runs every mode")
    cfg, weights, reqs, want = setup(name)
    steps = TRACES[mode](reqs)
    page = X.PAGE[name]
    n_pages = C.pages_needed(steps, reqs, page)
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), page, n_pages)
    got, rp = C.run_trace(runner, steps)
    X.assert_matches(got, want, dtype == "bfloat16", f"{name}/{mode}")
    runner.pages.audit()
    assert runner.pages.live_requests() == 0
    assert all(runner.pages.free_pages(g) == n_pages for g in range(len(runner.group_shapes)))
    if mode == "mixed":
        owners, reused = {}, False
        for held in rp.page_log:
            for rid, tables in held.items():
                for g, pages in enumerate(tables):
                    for p in pages:
                        if p >= 0:
                            reused |= owners.setdefault((g, p), rid) != rid
        assert reused, "the trace was meant to reuse pages"


def test_memory_plan():
    """Pages for the attention half of each "parallel" layer, chunked where it has a mask; a matrix per head (and a row of
    the token before, or a convolution's inputs) per request for every recurrence; the embedding's last token has a
    state of its own after the layers'."""
    cfg, weights, _, _ = setup("odd")
    runner = X.make_runner(cfg, weights, "float32", "cpu", RefOps(), 16, 4)
    m = runner.model
    assert [e.layer for e in m.spec.run_order] == [0, 1, 2, 3]
    assert [(s.group is not None, len(s.state_indices)) for s in m.sites] == [(True, 2), (False, 2), (False, 1), (True, 2), (False, 1)]
    assert m.embedding_site == 4 and m.sites[4].layer == -1
    shapes = [(tuple(n.shape), n.dtype) for n in m.state_needs]
    f32 = torch.float32
    assert shapes == [((3, 7, 7), f32), ((42,), f32), ((4, 6, 9), f32), ((2, 2 * 12 + 36), f32), ((3, 10, 5), f32), ((2, 10, 10), f32), ((42,), f32),
                      ((1,), torch.int32)]
    needs = [(g.need.num_kv_heads, g.need.head_dim, g.need.v_dim, g.need.window, g.need.chunked) for g in m.cache_groups]
    assert needs == [(2, 10, 6, 11, True), (3, 8, 12, 20, True)]
    no_mask = X.make_runner(X.CONFIGS["mix"], setup("mix")[1], "float32", "cpu", RefOps(), 16, 4).model
    assert [(g.need.window, g.need.chunked) for g in no_mask.cache_groups] == [(32, True), (None, False), (7, True)]
    assert runner.memory.states[-1].flatten().tolist() == [-1] * 4


@pytest.mark.parametrize("backend", BACKENDS)
def test_slots_and_pages_are_used_again(backend):
    """Two slots, six requests one after another in pairs, in a pool that holds two of them: a request that takes over
    pages and slots reads nothing of what the one before left there (matrices, convolution inputs, the token
    before, in rows and in the embedding)."""
    device, dtype = backend
    cfg, weights, reqs, want = setup("odd")
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 8, max_seqs=2)
    got, _ = C.run_trace(runner, C.trace_mixed(reqs, max_live=2))
    X.assert_matches(got, want, dtype == "bfloat16", "two slots")
    assert runner.pages.free_slots() == 2


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(backend):
    """A short prompt and 200 tokens decoded one by one: states carried far, ten and more chunks begun and left (their
    pages given back and taken again) in decoding alone."""
    device, dtype = backend
    cfg = X.CONFIGS["odd"]
    weights = X.random_weights(cfg, seed=21, ranks=X.RANKS["odd"])
    reqs = X.make_requests(cfg, [215], seed=3)
    want = X.plain_logits(cfg, weights, reqs)
    # (chunks of 11 and 20: never more than three pages of 16 held behind a single token, fifteen for the prompt alone)
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 3, max_seqs=1)
    got, rp = C.run_trace(runner, C.trace_tail(reqs, tail=200))
    X.assert_matches(got, want, dtype == "bfloat16", "long decoding")
    assert max(sum(p >= 0 for p in held["r0"][0]) for held in rp.page_log) <= 2


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["mix", "wide"])
def test_long_prompt_in_one_step(backend, name):
    """A prompt of 450 tokens whole, then a few tokens one by one; and the same prompt in portions whose edges fall inside
    pages, chunks and the blocks of keys and tokens the kernels walk."""
    device, dtype = backend
    if device == "cpu":
        pytest.skip("the plain ops are slow at this size; the GPU runs it")
    cfg = X.CONFIGS[name]
    weights = X.random_weights(cfg, seed=31, ranks=X.RANKS[name])
    reqs = X.make_requests(cfg, [456], seed=8)
    want = X.plain_logits(cfg, weights, reqs)
    for make in (lambda r: C.trace_tail(r, tail=6), lambda r: C.trace_portions(r, sizes=[70, 2, 33, 64, 5, 100, 1])):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), X.PAGE[name], 16, max_seqs=1)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", f"{name}/long prompt")


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_width_whose_products_come_in_slices(backend):
    """Width 1,024: for few tokens the products are left as slices that the next kernel sums (one half of a pair of
    mixers is normed before the other's products take the slices' workspace); more than 64 and more than 32 tokens take
    other products again."""
    device, dtype = backend
    if device == "cpu":
        pytest.skip("the plain ops have no slices; the GPU runs it")
    cfg = X.model(300, 1024, 1e-6, 2.0, [
        (X.both(X.att(8, 2, 128, 128, 1.2, 64, 30.0, (32, 10000.0)), X.mixing(8, 64)), X.dense(1024)),
        (X.delta(8, 4, 64, 128, 4), X.dense(768)),
    ], scale=32.0, bigram=(1001, 29, 3))
    weights = X.random_weights(cfg, seed=51, ranks=(72, 40, 56))
    reqs = X.make_requests(cfg, [90, 9, 48], seed=5)
    want = X.plain_logits(cfg, weights, reqs)
    for make in (C.trace_whole, lambda r: C.trace_tail(r, tail=20), C.trace_portions, C.trace_mixed):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 64, 5)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", "width 1,024")


def _one_layer(layer, ff=None, width=32, eps=1e-5, alpha=1.5, scale=2.0, bigram=None, vocab=80):
    return X.model(vocab, width, eps, alpha, [(layer, ff)], scale=scale, bigram=bigram)


_ATT, _MIX = X.att(2, 1, 8, 8, 0.5, 9), X.mixing(2, 8)
MECHANISMS = {
    "delta": _one_layer(X.delta(4, 2, 8, 8, 4)),
    "delta_one_tap_a_key_head_per_head": _one_layer(X.delta(3, 3, 6, 10, 1)),
    "delta_two_taps_one_head": _one_layer(X.delta(1, 1, 16, 4, 2)),
    "delta_wide_keys_six_taps": _one_layer(X.delta(6, 2, 20, 3, 6)),
    "parallel": _one_layer(X.both(X.att(4, 2, 8, 6, 0.5, 10, 3.0, (4, 100.0)), _MIX)),
    "parallel_no_mask_no_cap_no_rotation": _one_layer(X.both(X.att(3, 1, 6, 10, 0.7), _MIX)),
    "parallel_whole_head_rotates_chunks_of_one": _one_layer(X.both(X.att(2, 2, 8, 8, 0.4, 1, 2.0, (8, 30.0)), _MIX)),
    "parallel_chunk_longer_than_the_sequence": _one_layer(X.both(X.att(2, 1, 8, 8, 0.4, 1000, 5.0, (2, 10.0)), _MIX)),
    "parallel_mixing_of_one_head": _one_layer(X.both(_ATT, X.mixing(1, 32))),
    "parallel_mixing_of_many_small_heads": _one_layer(X.both(_ATT, X.mixing(9, 4))),
    "feed_forward": _one_layer(X.delta(1, 1, 8, 8, 2), X.dense(40)),
    "pairs": _one_layer(X.delta(1, 1, 8, 8, 2), bigram=(37, 11, 3)),
    "pairs_the_token_alone_decides": _one_layer(X.delta(1, 1, 8, 8, 2), bigram=(50, 0, 1)),
    "pairs_large_multipliers": _one_layer(X.delta(1, 1, 8, 8, 2), bigram=(64, 2654435761, 40503), scale=1.0),
    "stream_scaled_down_large_eps": _one_layer(X.delta(2, 1, 8, 8, 2), X.dense(20), alpha=0.25, eps=0.5),
}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("which", list(MECHANISMS))
def test_each_mechanism_alone(backend, which):
    """One-layer models, each with one mechanism, whole, in portions and with the last tokens one by one."""
    device, dtype = backend
    cfg = MECHANISMS[which]
    weights = X.random_weights(cfg, seed=5, ranks=(6, 4, 5))
    reqs = X.make_requests(cfg, [37, 12], seed=1)
    want = X.plain_logits(cfg, weights, reqs)
    for make in (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=9)):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 8)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", which)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["odd", "mix"])
def test_residual_stream_after_every_layer(backend, name):
    """The float32 stream after each layer equals the plain one: the pair's row, the embedding's scale, alpha and the layer
    scales show here before later norms could hide a factor.  The engine is made to stop after the first layers."""
    device, dtype = backend
    cfg, weights, reqs, _ = setup(name)
    toks = reqs["r2"]
    streams = []
    P.forward(weights, cfg, toks, streams)
    for depth in range(1, len(cfg["layers"]) + 1):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 8)
        m = runner.model
        m.spec = copy.copy(m.spec)
        object.__setattr__(m.spec, "run_order", m.spec.run_order[:depth])
        captured = {}
        original = m.final_norm.gather_add_norm

        def spy(residual, delta, rows, _original=original):
            captured["x"] = residual.float().cpu().clone()
            captured["rounded"] = delta.activations.float().cpu().clone()
            return _original(residual, delta, rows)

        m.final_norm.gather_add_norm = spy
        C.run_trace(runner, C.trace_whole({"a": toks}))
        want = streams[depth - 1]
        err = (captured["x"].double() - want).abs().max().item() / want.abs().max().item()
        assert err < (6e-2 if dtype == "bfloat16" else 1e-5), f"stream after layer {depth - 1}: relative error {err:.2e}"
        assert torch.equal(captured["rounded"], captured["x"].to(runner.rt.act_dtype).float()), "what is handed on is the stream, rounded"


def _differs(a, b):
    return X.relative_error(a.double(), b)


def _run_all(cfg, weights, reqs, want, backend, what, traces, page=16, n_pages=24, max_len=512, **kw):
    device, dtype = backend
    for make in traces:
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), page, n_pages, max_len=max_len, **kw)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", what)


def _silent_right(weights, prefix="l0.mix."):
    """The time mixing's half weighs little, so that the attention's shows."""
    weights[prefix + "right.out"] = (weights[prefix + "right.out"] * 0.02).to(torch.bfloat16).float()


def _with(name, value):
    """A context in which the plain implementation's ``name`` is replaced."""
    class _Swap:
        def __enter__(self):
            self.old = getattr(P, name)
            setattr(P, name, value)

        def __exit__(self, *a):
            setattr(P, name, self.old)
    return _Swap()


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("chunk", [300, 128, 96])
def test_sharp_attention_far_keys(backend, chunk):
    """Scores so large that most queries give most of their weight to one key, anywhere among the up to 299 before it in
    their chunk: a key lost or misplaced at a page's border, a chunk's first positions, or far back changes that query's logits
    outright."""
    device, dtype = backend
    cfg = _one_layer(X.both(X.att(2, 1, 8, 6, 6.0, chunk, 60.0, (2, 1000.0)), X.mixing(1, 4)), vocab=400)
    weights = X.random_weights(cfg, seed=13)
    _silent_right(weights)
    toks = torch.randperm(400, generator=torch.Generator().manual_seed(2))[:300].tolist()
    P.ATTENTION_PEAKS = peaks = []
    try:
        want = X.plain_logits(cfg, weights, {"a": toks})
    finally:
        P.ATTENTION_PEAKS = None
    late = [p for p in peaks if p[0] >= 100]
    assert sorted(p[3] for p in late)[len(late) // 2] > 0.5, "the test's attention was meant to be sharp"
    assert any(p[0] - p[2] > 0.7 * chunk for p in peaks), "some query was meant to pick a key far back in its chunk"
    assert all(p[2] // chunk == p[0] // chunk for p in peaks)
    _run_all(cfg, weights, {"a": toks}, want, backend, f"sharp attention, chunks of {chunk}",
             (lambda r: C.trace_tail(r, tail=60), C.trace_portions), max_len=400)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("chunk,page", [(16, 16), (13, 16), (32, 16), (5, 32), (24, 16)])
def test_chunks_begin_where_they_say(backend, chunk, page):
    """One token's key towers over every other (its queries' direction is shared), and it stands at every place around the
    chunks' edges: the queries behind it see it to their chunk's end and not a token longer, in prompts, portions cut
    anywhere and decoded tokens.  A window that slides, or chunks counted a position off, gives other logits at the edges
    (shown with the plain implementation)."""
    device, dtype = backend
    cfg = _one_layer(X.both(X.att(2, 1, 8, 8, 3.0, chunk, 40.0), X.mixing(1, 4)))
    weights = X.random_weights(cfg, seed=chunk)
    _silent_right(weights)
    # every query points along one direction (its first two dimensions), and token 7's key with it
    q, k = weights["l0.mix.left.q"], weights["l0.mix.left.k"]
    emb = weights["embed"].double() * 2.0
    u = emb.mean(0)
    weights["embed"] = (weights["embed"] + 1.5 * torch.sign(u).float() / 2.0).to(torch.bfloat16).float()
    emb = weights["embed"].double() * 2.0
    for h in range(2):
        q[8 * h] = torch.sign(u).float() * 0.5
    k[0] = ((emb[7] - emb.mean(0)).float() * 0.25)
    weights["l0.mix.left.q"], weights["l0.mix.left.k"] = q.to(torch.bfloat16).float(), k.to(torch.bfloat16).float()
    g = torch.Generator().manual_seed(3)
    n = 4 * chunk + 10
    toks = [t if t != 7 else 8 for t in torch.randint(0, 80, (n,), generator=g).tolist()]
    marked = [0, chunk - 1, chunk, 2 * chunk, 3 * chunk - 1, 3 * chunk + 1, 4 * chunk - 2]
    for i in marked:
        toks[i] = 7
    P.ATTENTION_PEAKS = peaks = []
    try:
        want = X.plain_logits(cfg, weights, {"a": toks})
    finally:
        P.ATTENTION_PEAKS = None
    picked = [p for p in peaks if p[2] in marked and p[0] != p[2]]
    assert len(picked) > 10, "the marked keys were meant to draw the queries behind them"
    slides = lambda i, mask: max(0, i - int(mask["size"]) + 1)
    late = lambda i, mask: max(0, i - 1) // int(mask["size"]) * int(mask["size"])
    early = lambda i, mask: max(0, (i + 1) // int(mask["size"]) * int(mask["size"]) - 1)
    for wrong in (slides, late, early):
        with _with("first_visible", wrong):
            d = _differs(P.forward(weights, cfg, toks), want["a"])
        assert d.max() > 0.05, "which keys a query sees was meant to show"
    _run_all(cfg, weights, {"a": toks}, want, backend, f"chunks of {chunk}, pages of {page}",
             (C.trace_whole, lambda r: C.trace_tail(r, tail=n - 20), lambda r: C.trace_portions(r, sizes=[7, 2, 30, 16, 3]),
              lambda r: C.trace_portions(r, sizes=[chunk, chunk - 1, 1, chunk + 1])), page=page, n_pages=-(-n // page) + 1, max_len=256)


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_sink_takes_its_share(backend):
    """Scores small or negative, so that the one in the denominator takes much of the weight, most at a chunk's first
    tokens, where one key stands against it: without it, or with a sink that is another number, the logits are others."""
    device, dtype = backend
    cfg = _one_layer(X.both(X.att(3, 1, 8, 6, 0.3, 6, 2.0, (8, 100.0)), X.mixing(1, 4)), alpha=0.5)
    weights = X.random_weights(cfg, seed=17)
    _silent_right(weights)
    # (the sum of the heads is normed: heads must lose unlike shares for the sink to show)
    reqs = X.make_requests(cfg, [40, 3, 1], seed=6)
    want = X.plain_logits(cfg, weights, reqs)
    plain = P.sink_softmax
    with _with("sink_softmax", lambda s: torch.softmax(s, dim=0)):
        d = _differs(X.plain_logits(cfg, weights, reqs)["r0"], want["r0"])
    assert (d > 0.02).float().mean() > 0.4, "the sink was meant to matter"
    with _with("sink_softmax", lambda s: plain(s - 2.0)):
        assert (_differs(X.plain_logits(cfg, weights, reqs)["r0"], want["r0"]) > 0.02).float().mean() > 0.3
    _run_all(cfg, weights, reqs, want, backend, "sinks", (C.trace_whole, lambda r: C.trace_tail(r, tail=30), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_rotation_pairs_neighbours_and_norms_have_no_weight(backend):
    """Sharp scores that depend on distance through the rotation: pairs taken from both halves, a rotation of the whole head,
    another base, or queries and keys left as long as they are, give other logits."""
    device, dtype = backend
    cfg = _one_layer(X.both(X.att(2, 1, 16, 8, 2.5, 70, None, (12, 40.0)), X.mixing(1, 4)))
    weights = X.random_weights(cfg, seed=41)
    _silent_right(weights)
    for n in ("q", "k"):  # (heads of unlike length)
        weights["l0.mix.left." + n] = (weights["l0.mix.left." + n] * 1.7).to(torch.bfloat16).float()
    toks = X.make_requests(cfg, [230], seed=7)["r0"]
    want = X.plain_logits(cfg, weights, {"a": toks})
    rotate, rms = P.rotate, P.rms

    def halves(x, rot):
        d = int(rot["dims"])
        order = [j for i in range(d // 2) for j in (i, i + d // 2)] + list(range(d, x.shape[-1]))
        back = [order.index(j) for j in range(x.shape[-1])]
        return rotate(x[..., order], rot)[..., back]

    for wrong in (halves, lambda x, rot: rotate(x, dict(rot, dims=16)), lambda x, rot: rotate(x, dict(rot, base=90.0))):
        with _with("rotate", wrong):
            d = _differs(P.forward(weights, cfg, toks), want["a"])
        assert (d[100:] > 0.02).float().mean() > 0.4, "the rotation was meant to show"
    with _with("rms", lambda x, eps: x if x.shape[-1] == 16 else rms(x, eps)):
        assert (_differs(P.forward(weights, cfg, toks), want["a"]) > 0.02).float().mean() > 0.5
    _run_all(cfg, weights, {"a": toks}, want, backend, "rotation", (lambda r: C.trace_tail(r, tail=80), C.trace_portions), n_pages=16)


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_order_inside_the_delta_rule(backend):
    """Strong writes and strong decays: reading before the write, writing before the decay, a decay per head in place of one
    per channel, or query and key heads dealt round the value heads give other logits."""
    device, dtype = backend
    cfg = _one_layer(X.delta(4, 2, 8, 8, 3), alpha=0.5)
    weights = X.random_weights(cfg, seed=23)
    weights["l0.mix.dt_bias"] = (weights["l0.mix.dt_bias"] + 1.0).to(torch.bfloat16).float()
    reqs = X.make_requests(cfg, [60, 5], seed=12)
    want = X.plain_logits(cfg, weights, reqs)

    def scan(order):
        def run(q, k, v, beta, g):
            n, H, d = q.shape
            S = torch.zeros(H, d, v.shape[-1], dtype=P.F)
            out = torch.zeros(n, H, v.shape[-1], dtype=P.F)
            for t in range(n):
                def write():
                    u = beta[t][:, None] * (v[t] - torch.einsum("hde,hd->he", S, k[t]))
                    return S + k[t][:, :, None] * u[:, None, :]
                for what in order:
                    if what == "decay":
                        S = g[t][:, :, None] * S
                    elif what == "write":
                        S = write()
                    else:
                        out[t] = torch.einsum("hde,hd->he", S, q[t])
            return out
        return run

    plain_decay = P.channel_decay
    wrongs = [("delta_scan", scan(("decay", "read", "write"))), ("delta_scan", scan(("write", "decay", "read"))),
              ("channel_decay", lambda *a: plain_decay(*a).mean(-1, keepdim=True).expand(-1, -1, 8))]
    for name, wrong in wrongs:
        with _with(name, wrong):
            d = _differs(X.plain_logits(cfg, weights, reqs)["r0"], want["r0"])
        assert (d > 0.03).float().mean() > 0.5, f"{name} was meant to show"
    _run_all(cfg, weights, reqs, want, backend, "delta rule", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=25), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_time_mixing_reads_before_it_writes(backend):
    """A bonus far from one, fast and slow decays, and mixes far from zero and one: a read-out of the memory after the write,
    a bonus left out, a decay before the read, or the wrong token before give other logits."""
    device, dtype = backend
    cfg = _one_layer(X.both(X.att(1, 1, 4, 4, 0.1, 3), X.mixing(3, 8)), alpha=0.5)
    weights = X.random_weights(cfg, seed=29)
    weights["l0.mix.left.out"] = (weights["l0.mix.left.out"] * 0.02).to(torch.bfloat16).float()
    weights["l0.mix.right.u"] = (weights["l0.mix.right.u"] * 3.0 + 2.0).to(torch.bfloat16).float()
    reqs = X.make_requests(cfg, [60, 5, 1], seed=12)
    want = X.plain_logits(cfg, weights, reqs)
    plain, before = P.bonus_scan, P.token_before

    def decays_first(r, k, v, w, u):
        n, H, d = r.shape
        S, out = torch.zeros(H, d, v.shape[-1], dtype=P.F), torch.zeros(n, H, v.shape[-1], dtype=P.F)
        for t in range(n):
            S = w[t][:, :, None] * S
            kv = k[t][:, :, None] * v[t][:, None, :]
            out[t] = torch.einsum("hde,hd->he", S + u[:, :, None] * kv, r[t])
            S = S + kv
        return out

    wrongs = [("bonus_scan", lambda r, k, v, w, u: plain(r, k, v, w, torch.ones_like(u))), ("bonus_scan", lambda r, k, v, w, u: plain(r, k, v, w, 0 * u)),
              ("bonus_scan", decays_first), ("token_before", lambda h: before(before(h))), ("token_before", lambda h: h)]
    for name, wrong in wrongs:
        with _with(name, wrong):
            d = _differs(X.plain_logits(cfg, weights, reqs)["r0"], want["r0"])
        assert (d > 0.03).float().mean() > 0.5, f"{name} was meant to show"
    _run_all(cfg, weights, reqs, want, backend, "time mixing", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=25), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_both_halves_are_normed_before_they_are_summed(backend):
    """Halves of very different size: summed as they are, or normed without their weights, they give other logits."""
    device, dtype = backend
    cfg = _one_layer(X.both(X.att(2, 1, 8, 8, 0.5, 12), X.mixing(2, 8)), alpha=0.5)
    weights = X.random_weights(cfg, seed=37)
    weights["l0.mix.left.o"] = (weights["l0.mix.left.o"] * 20.0).to(torch.bfloat16).float()
    reqs = X.make_requests(cfg, [40, 9], seed=5)
    want = X.plain_logits(cfg, weights, reqs)

    def unnormed(W, p, m, eps, h):
        return 0.5 * (P.chunked_attention(W, p + "left.", m["left"], eps, h) * W[p + "left.out"]
                      + P.time_mixing(W, p + "right.", m["right"], eps, h) * W[p + "right.out"])

    with _with("parallel", unnormed):
        assert (_differs(X.plain_logits(cfg, weights, reqs)["r0"], want["r0"]) > 0.05).float().mean() > 0.7
    for side in ("left", "right"):
        other = dict(weights, **{f"l0.mix.{side}.out": torch.ones(32)})
        assert (_differs(X.plain_logits(cfg, other, reqs)["r0"], want["r0"]) > 0.02).float().mean() > 0.7
    _run_all(cfg, weights, reqs, want, backend, "two halves", (C.trace_whole, C.trace_portions, C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_pairs_across_cuts_and_requests(backend):
    """Large rows for pairs: a first token that took the row of some pair, a portion's first token that forgot what came before
    it (or took another request's last token), or the two multipliers exchanged, give other logits at those tokens."""
    device, dtype = backend
    cfg = _one_layer(X.delta(1, 1, 8, 8, 1), bigram=(61, 19, 7), scale=1.0)
    weights = X.random_weights(cfg, seed=43)
    weights["bigram"] = (weights["bigram"] * 4.0).to(torch.bfloat16).float()
    reqs = X.make_requests(cfg, [45, 4, 17, 1, 30], seed=2)
    want = X.plain_logits(cfg, weights, reqs)
    row = P.bigram_row
    for wrong, where in ((lambda p, t, b: row(0 if p is None else p, t, b), 0), (lambda p, t, b: row(None if p is None else t, p or 0, b), 5)):
        with _with("bigram_row", wrong):
            assert _differs(X.plain_logits(cfg, weights, reqs)["r0"], want["r0"])[where] > 0.1
    _run_all(cfg, weights, reqs, want, backend, "pairs", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=12), C.trace_mixed,
                                                        lambda r: C.trace_random(r, 3)), n_pages=12)


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_captured_decode_step_carries_every_state(backend):
    """Single-token steps of one and of three requests, replayed many times with other steps between them: the states that a
    captured graph updates in place (matrices, convolution inputs, rows and tokens before) are those of the eager steps."""
    device, dtype = backend
    if device == "cpu":
        pytest.skip("steps are captured on the GPU only")
    cfg, weights, _, _ = setup("odd")
    reqs = X.make_requests(cfg, [40, 37, 44], seed=14)
    want = X.plain_logits(cfg, weights, reqs)
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 12)
    assert runner.use_graphs
    steps, done = [], {r: 0 for r in reqs}
    pattern = [("r0", 5), ("r1", 4), ("r2", 6)]
    steps.append({"step": 0, "entries": [{"id": r, "tokens": reqs[r][:n], "want": list(range(n))} for r, n in pattern], "end": []})
    done = dict(pattern)
    k = 0
    while any(done[r] < len(reqs[r]) for r in reqs):
        k += 1
        who = [r for r in reqs if done[r] < len(reqs[r]) and not (k % 4 == 1 and r != "r1") and not (k % 4 == 3 and r == "r1")]
        if not who:
            continue
        n = 3 if k % 7 == 0 else 1  # (an eager step now and then)
        entries = [{"id": r, "tokens": reqs[r][done[r]: done[r] + n], "want": list(range(len(reqs[r][done[r]: done[r] + n])))} for r in who]
        for r in who:
            done[r] = min(done[r] + n, len(reqs[r]))
        steps.append({"step": k, "entries": entries, "end": [r for r in who if done[r] == len(reqs[r])]})
    got, _ = C.run_trace(runner, steps)
    assert runner.graph_replays > 20
    X.assert_matches(got, want, dtype == "bfloat16", "captured steps")


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("num_pages", [24, 7])
def test_greedy_generation_through_the_engine(tmp_path, backend, num_pages):
    """``LLMEngine.generate`` with the scheduler under a token budget that cuts prompts into portions, and with so few
    pages that the youngest request is preempted and starts again: greedy tokens are the plain implementation's wherever
    its two best logits are clearly apart."""
    from yalis_amd import EngineConfig, InferenceConfig, LLMEngine, ModelConfig
    from yalis_amd.weights.safetensors_io import write_dict

    device, dtype = backend
    cfg = copy.deepcopy(X.CONFIGS["odd"])
    if num_pages == 7:  # (nothing is given back while a request lives: the pool runs out)
        for layer in cfg["layers"]:
            if layer["type"] == "parallel":
                layer["mixer"]["left"].pop("mask")
    weights = X.random_weights(cfg, seed=13, ranks=X.RANKS["odd"])  # (several greedy tokens whose best logits are clearly apart)
    folder = tmp_path / "model"
    os.makedirs(folder)
    with open(folder / "config.json", "w") as f:
        json.dump(cfg, f)
    wd = torch.float32 if dtype == "float32" else torch.bfloat16
    write_dict(str(folder / "model.safetensors"), {k: v.to(wd).contiguous() for k, v in weights.items()})
    eng = LLMEngine(
        ModelConfig(model_path=str(folder), precision="fp32" if dtype == "float32" else "bf16"),
        InferenceConfig(max_batch_size=3, max_length_of_generated_sequences=128, temperature=0.0),
        device=device, ops=RefOps() if device == "cpu" else None,
        engine_config=EngineConfig(page_size=16, num_pages=num_pages, max_num_seqs=3, max_model_len=128, max_num_batched_tokens=24,
                                   dtype=dtype, device=device),
    )
    prompts = list(X.make_requests(cfg, [30, 7, 45], seed=4).values())
    out, metrics = eng.generate(prompts, tokens_to_generate=12)
    assert out.shape == (3, 12)
    if num_pages == 7:
        assert metrics["Preemptions"] > 0, "this pool was meant to force a preemption"
    gap = 0.1 if dtype == "bfloat16" else 1e-3
    compared = 0
    for prompt, row in zip(prompts, out.tolist()):
        toks = list(prompt)
        for t in row:
            logits = P.forward(weights, cfg, toks)[-1]
            top2 = torch.topk(logits, 2).values
            if (top2[0] - top2[1]).item() < gap * logits.abs().max().item():
                break  # too close to call; what follows would compare other sequences
            assert t == int(torch.argmax(logits)), f"generated {row}, the plain implementation differs after {len(toks) - len(prompt)} tokens"
            toks.append(t)
            compared += 1
    assert compared >= 6


def test_config_reader_and_spec():
    """Sizes and constants come from config.json; what cannot run is refused with the key's name; the tensors a model asks
    for are the design's names and shapes."""
    from yalis_amd.config.reader import ConfigError
    from yalis_amd.engine.factory import spec_from_config, tensor_specs_for

    cfg = X.CONFIGS["odd"]
    _, typed, spec = spec_from_config(cfg)
    assert spec.vocab_size == 70 and spec.hidden_size == 42 and len(spec.layers) == 4 and typed.to_dict() == cfg
    assert spec.embedding.kind == "token_pair_embedding" and spec.head.params["tied_to"] is None
    e = spec.embedding.params
    assert (e["scale"], e["buckets"], e["mul_prev"], e["mul_cur"]) == (3.0, 211, 17, 5)
    assert all(layer.block == "post_norm" and layer.params["residual_scale"] == 1.7 for layer in spec.layers)
    pair = spec.layers[0].parts["mixer"]
    left, right = pair.params["left"].params, pair.params["right"].params
    assert (left["num_heads"], left["num_kv_heads"], left["head_dim"], left["value_dim"], left["window"], left["chunked"], left["softcap"],
            left["scale"], left["sink_score"]) == (6, 2, 10, 6, 11, True, 4.0, 0.6, 0.0)
    assert left["position"].params["rotary_dim"] == 6 and left["position"].params["pairing"] == "interleaved" and left["position"].params["theta"] == 50.0
    assert (right["num_heads"], right["head_dim"]) == (3, 7) and pair.params["scale"] == 0.5
    d = spec.layers[1].parts["mixer"].params
    assert (d["num_heads"], d["num_kv_heads"], d["head_dim"], d["value_dim"], d["conv_taps"], d["unit_eps"], d["out_norm_eps"]) == (4, 2, 6, 9, 3, 1e-6, 1e-5)
    assert "feed_forward" not in spec.layers[1].parts and "feed_forward_norm" not in spec.layers[1].parts
    assert spec.layers[2].parts["feed_forward"].params["activation"] == "gelu_tanh"
    assert spec.layers[2].parts["feed_forward_norm"].params["branch_weight"] == "l2.ls2"
    specs = tensor_specs_for(cfg)
    assert specs["embed"].shape == (70, 42) and specs["head"].shape == (70, 42) and specs["bigram"].shape == (212, 42)
    assert specs["l0.mix.left.q"].shape == (60, 42) and specs["l0.mix.left.v"].shape == (12, 42) and specs["l0.mix.left.o"].shape == (42, 36)
    assert not any(n.startswith("l0.mix.left") and "norm" in n for n in specs) and "l0.mix.left.sink" not in specs
    assert specs["l0.mix.right.u"].shape == (3, 7) and specs["l0.mix.right.norm"].shape == (21,) and specs["l0.mix.right.mu.w"].shape == (42,)
    assert specs["l0.mix.right.w1"].free_axes == (0,) and specs["l0.mix.right.w2"].shape[0] == 21
    assert specs["l0.mix.left.out"].shape == (42,) and specs["l0.mix.right.out"].shape == (42,)
    assert specs["l1.mix.q"].shape == (12, 42) and specs["l1.mix.v"].shape == (36, 42) and specs["l1.mix.v.conv"].shape == (36, 3)
    assert specs["l1.mix.A_log"].shape == (4,) and specs["l1.mix.dt_bias"].shape == (24,) and specs["l1.mix.norm"].shape == (9,)
    assert specs["l1.mix.a2"].shape[0] == 24 and specs["l1.mix.g2"].shape[0] == 36 and "l1.mix.a" not in specs and "l1.mix.g" not in specs
    assert "l1.norm2" not in specs and "l1.ls2" not in specs and specs["l1.ls1"].shape == (42,)
    for path, value, what in [
        (("layers", 0, "mixer", "left", "kv_heads"), 4, "multiple"), (("layers", 1, "mixer", "kv_heads"), 3, "multiple"),
        (("layers", 0, "type"), "delta", "not one of"), (("layers", 0, "mixer", "left", "rot", "dims"), 12, "dims"),
        (("layers", 0, "mixer", "left", "rot", "dims"), 5, "dims"), (("layers", 0, "mixer", "left", "mask", "size"), 0, "size"),
        (("layers", 1, "mixer", "conv"), 0, "conv"), (("layers", 0, "mlp", "kind"), "moe", "kind"),
        (("embedding", "bigram", "buckets"), 0, "buckets"), (("layers",), [], "layers"),
    ]:
        bad = copy.deepcopy(cfg)
        node = bad
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        with pytest.raises(ConfigError, match=what):
            spec_from_config(bad)
    for path in (("postln_alpha",), ("layers", 0, "mixer", "left", "scale"), ("norm", "eps"), ("layers", 0, "mixer", "right")):
        missing = copy.deepcopy(cfg)
        node = missing
        for key in path[:-1]:
            node = node[key]
        del node[path[-1]]
        with pytest.raises(ConfigError, match=path[-1]):
            spec_from_config(missing)
    plain = copy.deepcopy(cfg)
    del plain["embedding"]
    assert spec_from_config(plain)[2].embedding.kind == "token_embedding"


def test_a_design_without_pairs_runs():
    """config.json may leave the pairs' table (and the scale) out: the rows as they are."""
    cfg = copy.deepcopy(X.CONFIGS["odd"])
    cfg["embedding"] = {"scale": 1.0}
    weights = X.random_weights(cfg, seed=3, ranks=X.RANKS["odd"])
    assert "bigram" not in weights
    reqs = X.make_requests(cfg, [20, 5], seed=3)
    runner = X.make_runner(cfg, weights, "float32", "cpu", RefOps(), 16, 8)
    got, _ = C.run_trace(runner, C.trace_mixed(reqs))
    X.assert_matches(got, X.plain_logits(cfg, weights, reqs), False, "no pairs")
