"""Zimupel in the engine against the plain implementation (tests/plain_zimupel.py): every way of cutting the work, on the
CPU with plain PyTorch ops (the host side: batching, paging, states, the order of parts) and, marked ``gpu``, with the HIP
kernels in true float32 and in bfloat16."""
import copy
import json
import os

import pytest
import torch

import plain_zimupel as P
import replay_cases as C
import zimupel_cases as X
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
        weights = X.random_weights(cfg, seed=X.SEEDS[name])
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
    """Pages for every attention layer with keys of its own (both maps of a head side by side), none for one that reads another's;
    a float32 matrix per head and request for every recurrence."""
    cfg, weights, _, _ = setup("odd")
    runner = X.make_runner(cfg, weights, "float32", "cpu", RefOps(), 16, 4)
    m = runner.model
    assert [(e.layer, e.cache_from) for e in m.spec.run_order] == [(0, None), (1, None), (2, 0), (3, None), (4, None)]
    assert [(s.group, s.index_in_group, s.owns_cache, len(s.state_indices)) for s in m.sites] == [
        (0, 0, True, 0), (None, None, False, 1), (0, 0, False, 0), (None, None, False, 1), (None, None, False, 1)]
    needs = [(g.need.num_kv_heads, g.need.head_dim, g.need.v_dim, g.need.window) for g in m.cache_groups]
    assert needs == [(2, 10, 7, None)]
    assert [(tuple(n.shape), n.dtype) for n in m.state_needs] == [((3, 7, 5), torch.float32), ((2, 10, 6), torch.float32), ((3, 6, 9), torch.float32)]
    two = X.make_runner(X.CONFIGS["mix"], setup("mix")[1], "float32", "cpu", RefOps(), 16, 4).model
    assert [(g.need.num_kv_heads, g.need.head_dim, g.need.v_dim, g.entries) for g in two.cache_groups] == [(1, 16, 16, (1,)), (3, 24, 8, (3,))]


@pytest.mark.parametrize("backend", BACKENDS)
def test_slots_and_pages_are_used_again(backend):
    """Two slots, six requests one after another in pairs, in a pool that holds two of them: a request that takes over pages
    and slots reads nothing of what the one before left there."""
    device, dtype = backend
    cfg, weights, reqs, want = setup("odd")
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 8, max_seqs=2)
    got, _ = C.run_trace(runner, C.trace_mixed(reqs, max_live=2))
    X.assert_matches(got, want, dtype == "bfloat16", "two slots")
    assert runner.pages.free_slots() == 2


@pytest.mark.parametrize("backend", BACKENDS)
def test_long_decoding(backend):
    """A short prompt and 200 tokens decoded one by one: matrices carried far, pages taken in decoding alone."""
    device, dtype = backend
    cfg = X.CONFIGS["odd"]
    weights = X.random_weights(cfg, seed=X.SEEDS["odd"])
    reqs = X.make_requests(cfg, [215], seed=3)
    want = X.plain_logits(cfg, weights, reqs)
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 14, max_seqs=1)
    got, _ = C.run_trace(runner, C.trace_tail(reqs, tail=200))
    X.assert_matches(got, want, dtype == "bfloat16", "long decoding")


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["mix", "wide"])
def test_long_prompt_in_one_step(backend, name):
    """A prompt of 450 tokens whole, then a few tokens one by one; and the same prompt in portions whose edges fall inside
    pages, the scan's chunks and the blocks of keys the kernels walk."""
    device, dtype = backend
    if device == "cpu":
        pytest.skip("the plain ops are slow at this size; the GPU runs it")
    cfg, weights, _, _ = setup(name)
    reqs = X.make_requests(cfg, [456], seed=8)
    want = X.plain_logits(cfg, weights, reqs)
    for make in (lambda r: C.trace_tail(r, tail=6), lambda r: C.trace_portions(r, sizes=[70, 2, 33, 64, 5, 128, 1, 63])):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), X.PAGE[name], 16, max_seqs=1)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", f"{name}/long prompt")


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_width_whose_products_come_in_slices(backend):
    """Width 1,024: for few tokens the products are left as slices that the pass over the copies of the stream sums; more than 64
    and more than 32 tokens take other products again."""
    device, dtype = backend
    if device == "cpu":
        pytest.skip("the plain ops have no slices; the GPU runs it")
    cfg = X.model(300, 1024, 1e-6, 4, [
        (X.att(8, 2, 64, 128, 0.1, 0.4), X.dense(1024)),
        (X.lightning(128, 128, [0.9, 0.99, 0.5]), X.moe(6, 2, 256, (3, 2))),
        (X.retention(256, 128, [0.95, 0.999], (128, 10000.0)), X.dense(768)),
    ], cap=20.0)
    weights = X.random_weights(cfg, seed=51)
    reqs = X.make_requests(cfg, [90, 9, 48], seed=5)
    want = X.plain_logits(cfg, weights, reqs)
    for make in (C.trace_whole, lambda r: C.trace_tail(r, tail=20), C.trace_portions, C.trace_mixed):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 64, 5)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", "width 1,024")


def _layers(*layers, width=32, eps=1e-5, streams=2, vocab=80, **kw):
    return X.model(vocab, width, eps, streams, list(layers), **kw)


_LIGHT = X.lightning(8, 8, [0.9, 0.97])
MECHANISMS = {
    "attention": _layers((X.att(4, 2, 4, 8, 0.5, 0.3), None)),
    "attention_of_one_head": _layers((X.att(1, 1, 8, 4, 0.5, 0.2), None)),
    "attention_a_key_head_per_head": _layers((X.att(3, 3, 5, 6, 0.7, 0.0), None)),
    "attention_wide_maps_narrow_values": _layers((X.att(4, 1, 16, 3, 0.3, 0.6), None)),
    "attention_whose_share_is_negative": _layers((X.att(2, 1, 4, 8, 0.5, -0.4), None)),
    "attention_on_another_layers_keys": _layers((X.att(4, 2, 4, 8, 0.5, 0.3), None), (X.att(4, 2, 4, 8, 0.8, 0.6, kv_from=0), None)),
    "retention": _layers((X.retention(8, 8, [0.9, 0.99], (8, 100.0)), None)),
    "retention_part_of_the_head_rotates": _layers((X.retention(12, 5, [0.95], (6, 30.0)), None)),
    "retention_nothing_rotates": _layers((X.retention(6, 10, [0.9, 0.8, 0.99]), None)),
    "retention_that_forgets_nothing": _layers((X.retention(8, 8, [1.0, 1.0], (2, 10.0)), None)),
    "lightning": _layers((_LIGHT, None)),
    "lightning_wide_keys_one_head": _layers((X.lightning(24, 4, [0.95]), None)),
    "dense": _layers((_LIGHT, X.dense(40))),
    "experts": _layers((_LIGHT, X.moe(6, 2, 16))),
    "experts_in_groups": _layers((_LIGHT, X.moe(8, 3, 16, (4, 2)))),
    "experts_groups_of_one": _layers((_LIGHT, X.moe(4, 2, 16, (4, 3)))),
    "experts_one_group_holds_all": _layers((_LIGHT, X.moe(4, 1, 16, (1, 1)))),
    "experts_all_chosen": _layers((_LIGHT, X.moe(3, 3, 12))),
    "one_expert": _layers((_LIGHT, X.moe(1, 1, 12))),
    "one_copy_of_the_stream": _layers((_LIGHT, X.dense(24)), streams=1),
    "seven_copies": _layers((_LIGHT, X.dense(24)), streams=7),
    "twelve_copies": _layers((_LIGHT, X.dense(24)), streams=12),
    "capped_logits": _layers((_LIGHT, None), scale=2.5, cap=1.5),
    "scaled_logits": _layers((_LIGHT, None), scale=0.2),
    "large_eps": _layers((X.retention(8, 8, [0.9, 0.99]), X.dense(20)), eps=0.5),
}


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("which", list(MECHANISMS))
def test_each_mechanism_alone(backend, which):
    """Models of one layer or two, each with one mechanism, whole, in portions and with the last tokens one by one."""
    device, dtype = backend
    cfg = MECHANISMS[which]
    weights = X.random_weights(cfg, seed=6)
    reqs = X.make_requests(cfg, [37, 12], seed=1)
    want = X.plain_logits(cfg, weights, reqs)
    for make in (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=9)):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 8)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", which)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("name", ["odd", "mix"])
def test_residual_stream_after_every_layer(backend, name):
    """The sum of the float32 copies after each layer, with what the layer left pending, equals the plain one.  The engine is made
    to stop after the first layers; the final norm's input is seen through a norm that does nothing but scale."""
    device, dtype = backend
    cfg, weights, reqs, _ = setup(name)
    toks = reqs["r2"]
    streams = []
    P.forward(weights, cfg, toks, streams)
    for depth in range(1, len(cfg["layers"]) + 1):
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 32, 8)
        m = runner.model
        m.spec = copy.copy(m.spec)
        object.__setattr__(m.spec, "run_order", m.spec.run_order[:depth])
        captured = {}
        original = m.final_norm.gather_add_norm

        def spy(residual, delta, rows, _original=original):
            # the pass every block begins with, on a copy: what is pending joins the copies
            x = residual.clone()
            m.final_norm.streams_norm(x, delta, None)
            captured["x"] = x.sum(1).double().cpu()
            return _original(residual, delta, rows)

        m.final_norm.gather_add_norm = spy
        C.run_trace(runner, C.trace_whole({"a": toks}))
        want = streams[depth - 1]
        err = (captured["x"] - want).pow(2).mean(1).sqrt() / want.pow(2).mean(1).sqrt()
        bound = 2e-2 * depth if dtype == "bfloat16" else 1e-5
        assert err.median() < bound and (dtype == "bfloat16" or err.max() < 2e-3), f"stream after layer {depth - 1}: relative error {err.max():.2e}"


def _differs(a, b):
    return X.relative_error(a.double(), b)


def _run_all(cfg, weights, reqs, want, backend, what, traces, page=16, n_pages=24, max_len=512, **kw):
    device, dtype = backend
    for make in traces:
        runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), page, n_pages, max_len=max_len, **kw)
        got, _ = C.run_trace(runner, make(reqs))
        X.assert_matches(got, want, dtype == "bfloat16", what)


def _with(name, value):
    """A context in which the plain implementation's ``name`` is replaced."""
    class _Swap:
        def __enter__(self):
            self.old = getattr(P, name)
            setattr(P, name, value)

        def __exit__(self, *a):
            setattr(P, name, self.old)
    return _Swap()


def _shows(cfg, weights, reqs, want, name, wrong, what, share=0.3, by=0.02):
    """The plain implementation with one function replaced gives other logits (so that the test would notice)."""
    with _with(name, wrong):
        d = torch.cat([_differs(P.forward(weights, cfg, toks), want[rid]) for rid, toks in reqs.items()])
    assert (d > by).float().mean() > share, f"{what} was meant to show"


def _rounded(weights, name, value):
    weights[name] = value.to(torch.bfloat16).float()


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("dim,vdim,page", [(4, 6, 16), (32, 64, 64)])
def test_sharp_attention_far_keys(backend, dim, vdim, page):
    """Scores so large that in both maps most queries give most of their weight to one key, anywhere among the up to 299 before
    it: a key lost or misplaced at a page's border, among the first tokens or far back changes that query's logits outright.  Every
    token stands once, since a mixer without positions gives equal tokens equal keys."""
    device, dtype = backend
    cfg = _layers((X.att(2, 1, dim, vdim, 4.0 * dim ** -0.5, 0.2), None), vocab=400)
    weights = X.random_weights(cfg, seed=13)
    for n in ("q", "k"):
        _rounded(weights, f"l0.mix.{n}", weights[f"l0.mix.{n}"] * 2.0)
    toks = torch.randperm(400, generator=torch.Generator().manual_seed(2))[:300].tolist()
    P.ATTENTION_PEAKS = peaks = []
    try:
        want = X.plain_logits(cfg, weights, {"a": toks})
    finally:
        P.ATTENTION_PEAKS = None
    for which in (0, 1):
        late = [p for p in peaks if p[0] >= 100 and p[2] == which]
        assert sorted(p[4] for p in late)[len(late) // 2] > 0.5, "the test's attention was meant to be sharp"
        assert any(p[0] - p[3] > 230 for p in late) and any(p[3] < 16 for p in late), "some query was meant to pick a key far back"
    _run_all(cfg, weights, {"a": toks}, want, backend, "sharp attention", (C.trace_whole, lambda r: C.trace_tail(r, tail=60), C.trace_portions),
             page=page, n_pages=-(-300 // page), max_len=400)


@pytest.mark.parametrize("backend", BACKENDS)
def test_how_two_maps_become_one(backend):
    """A lambda far from its offset, and values that both maps weigh: maps exchanged, lambda without its exponentials, no norm, a
    norm before the difference, or the share left out of the output give other logits."""
    device, dtype = backend
    cfg = _layers((X.att(4, 2, 6, 10, 0.6, 0.3), None))
    weights = X.random_weights(cfg, seed=17)
    for n, s in (("lq1", 0.5), ("lk1", 0.4), ("lq2", 0.3), ("lk2", -0.5)):
        _rounded(weights, f"l0.mix.{n}", torch.full((6,), s) + 0.05 * torch.arange(6))
    reqs = X.make_requests(cfg, [40, 3, 1], seed=6)
    want = X.plain_logits(cfg, weights, reqs)
    combine, lam = P.combine_maps, P.map_weight
    assert abs(lam({k: v.double() for k, v in weights.items()}, "l0.mix.", cfg["layers"][0]["mixer"]) - 0.3) > 0.5
    for what, name, wrong in [
        ("the maps' order", "combine_maps", lambda a, b, l, d, e: combine(b, a, l, d, e)),
        ("lambda", "map_weight", lambda W, p, m: float(m["diff"])),
        ("the norm", "combine_maps", lambda a, b, l, d, e: (a - l * b) * (1.0 - d)),
        ("a norm per map", "combine_maps", lambda a, b, l, d, e: (P.rms(a, e) - l * P.rms(b, e)) * (1.0 - d)),
        ("the output's share", "combine_maps", lambda a, b, l, d, e: combine(a, b, l, 0.0, e)),
    ]:
        _shows(cfg, weights, reqs, want, name, wrong, what)
    _run_all(cfg, weights, reqs, want, backend, "two maps", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=30), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_layer_reads_an_earlier_layers_keys(backend):
    """Three attention layers, the last one on the first one's keys and values: those of the second, or an own projection's, are
    other logits; biases of keys and values that are large enough to show."""
    device, dtype = backend
    cfg = _layers((X.att(4, 2, 4, 8, 0.7, 0.2), None), (X.att(4, 2, 4, 8, 0.7, 0.2), None), (X.att(4, 2, 4, 8, 1.1, 0.5, kv_from=0), None))
    weights = X.random_weights(cfg, seed=19)
    for i in (0, 1):
        for n in ("q.b", "k.b", "v.b"):
            _rounded(weights, f"l{i}.mix.{n}", weights[f"l{i}.mix.{n}"] * 2.0)
    assert "l2.mix.k" not in weights and "l2.mix.v.b" not in weights and "l2.mix.q.b" in weights
    reqs = X.make_requests(cfg, [50, 20, 2], seed=3)
    want = X.plain_logits(cfg, weights, reqs)
    other = copy.deepcopy(cfg)
    other["layers"][2]["mixer"]["kv_from"] = 1
    for c, w, what in ((other, weights, "another layer's keys"),
                       (cfg, dict(weights, **{"l0.mix.v.b": 0 * weights["l0.mix.v.b"]}), "the values' bias"),
                       (cfg, dict(weights, **{"l2.mix.q.b": 0 * weights["l2.mix.q.b"]}), "the queries' bias")):
        d = _differs(P.forward(w, c, reqs["r0"]), want["r0"])
        assert (d > 0.02).float().mean() > 0.5, f"{what} was meant to show"
    _run_all(cfg, weights, reqs, want, backend, "borrowed keys", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=20), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_the_order_inside_the_recurrences(backend):
    """Reading before the write, decaying after it, decays dealt to the heads the other way round, a rotation of neighbours or of
    other elements, values rotated too, and keys left unscaled give other logits."""
    device, dtype = backend
    cfg = _layers((X.retention(8, 6, [0.3, 0.99, 0.8], (6, 40.0)), None), eps=1.0)
    weights = X.random_weights(cfg, seed=23)
    reqs = X.make_requests(cfg, [60, 5], seed=12)
    want = X.plain_logits(cfg, weights, reqs)
    scan, rotate = P.fixed_decay_scan, P.rotate

    def ordered(order):
        def run(q, k, v, decay):
            n, H, d = q.shape
            a = torch.tensor(decay, dtype=P.F)[:, None, None]
            S, out = torch.zeros(H, d, v.shape[-1], dtype=P.F), torch.zeros(n, H, v.shape[-1], dtype=P.F)
            for t in range(n):
                for what in order:
                    if what == "decay":
                        S = a * S
                    elif what == "write":
                        S = S + k[t][:, :, None] * v[t][:, None, :]
                    else:
                        out[t] = torch.einsum("hde,hd->he", S, q[t])
            return out
        return run

    def neighbours(x, rot):
        d = int(rot["dims"])
        order = [j for i in range(d // 2) for j in (2 * i, 2 * i + 1)]
        order = order[0::2] + order[1::2] + list(range(d, x.shape[-1]))
        return rotate(x[..., order], rot)[..., [order.index(j) for j in range(x.shape[-1])]]

    for what, name, wrong in [
        ("reading first", "fixed_decay_scan", ordered(("decay", "read", "write"))),
        ("decaying last", "fixed_decay_scan", ordered(("write", "decay", "read"))),
        ("the heads' decays", "fixed_decay_scan", lambda q, k, v, a: scan(q, k, v, a[::-1])),
        ("the keys' scale", "fixed_decay_scan", lambda q, k, v, a: scan(q, k * 8 ** 0.5, v, a)),
        ("pairs of neighbours", "rotate", neighbours),
        ("how much rotates", "rotate", lambda x, rot: rotate(x, dict(rot, dims=8))),
        ("the base", "rotate", lambda x, rot: rotate(x, dict(rot, base=400.0))),
    ]:
        _shows(cfg, weights, reqs, want, name, wrong, what)
    _run_all(cfg, weights, reqs, want, backend, "retention", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=25), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
@pytest.mark.parametrize("layer", [X.retention(32, 32, [0.9995, 0.999], (32, 10000.0)), X.lightning(32, 32, [0.9995, 0.999]), X.lightning(6, 5, [1.0, 0.9995])])
def test_a_memory_that_lasts(backend, layer):
    """Decays so slow that what was written 200 tokens ago decides: a state lost between two steps changes the last logits, in
    prompts cut anywhere (inside the scan's chunks and at their edges), and in decoding."""
    device, dtype = backend
    if device == "cpu" and layer["mixer"]["dim"] == 32:
        pytest.skip("the plain ops are slow at this size; the GPU runs it")
    cfg = _layers((layer, None), eps=1e-3)
    weights = X.random_weights(cfg, seed=29)
    toks = X.make_requests(cfg, [300], seed=4)["r0"]
    want = X.plain_logits(cfg, weights, {"a": toks})
    forgot = P.forward(weights, cfg, toks[100:])[100:]  # (other positions too, which retention's distances do not see)
    assert (_differs(forgot, want["a"][200:]) > 0.02).float().mean() > 0.5, "the first hundred tokens were meant to matter"
    for sizes in ([64], [63, 65, 1, 2], [7, 100, 64, 5], [128, 3]):
        _run_all(cfg, weights, {"a": toks}, want, backend, f"portions of {sizes}", (lambda r: C.trace_portions(r, sizes=sizes),), max_len=400)
    _run_all(cfg, weights, {"a": toks}, want, backend, "decoding", (lambda r: C.trace_tail(r, tail=100),), max_len=400)


@pytest.mark.parametrize("backend", BACKENDS)
def test_lightning_norms_and_gates(backend):
    """Heads of very different size: a norm per head, a gate by silu, projections without their activation give other logits."""
    device, dtype = backend
    cfg = _layers((X.lightning(8, 6, [0.5, 0.99, 0.9]), None), eps=1e-3)
    weights = X.random_weights(cfg, seed=31)
    v = weights["l0.mix.v"].clone()
    v[:6] *= 4.0
    _rounded(weights, "l0.mix.v", v)
    reqs = X.make_requests(cfg, [60, 5], seed=12)
    want = X.plain_logits(cfg, weights, reqs)
    rms = P.rms
    _shows(cfg, weights, reqs, want, "rms", lambda x, e: rms(x.view(-1, 3, 6), e).reshape(-1, 18) if x.shape[-1] == 18 else rms(x, e), "a norm per head")
    _shows(cfg, weights, reqs, want, "silu", lambda z: z, "the projections' activation")
    _shows(cfg, dict(weights, **{"l0.mix.norm": torch.ones(18)}), reqs, want, "rms", rms, "the norm's weight")
    _run_all(cfg, weights, reqs, want, backend, "lightning", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=25), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_how_the_streams_mix(backend):
    """Mixes far from symmetric, copies read and written unevenly: the mix the other way round, new copies made of copies already
    new, a branch that every copy gets in full, or one copy read alone give other logits; so does a second branch that hangs
    on the stream like the first."""
    device, dtype = backend
    cfg = _layers((_LIGHT, X.dense(24)), (X.lightning(6, 10, [0.8]), X.dense(30)), streams=4)
    weights = X.random_weights(cfg, seed=37)
    g = torch.Generator().manual_seed(1)
    for i in (0, 1):
        for q in (1, 2):
            _rounded(weights, f"l{i}.hc{q}.mix", 0.6 * torch.eye(4) + 0.5 * torch.triu(torch.rand(4, 4, generator=g), 1))
            _rounded(weights, f"l{i}.hc{q}.in", torch.tensor([0.9, 0.2, -0.4, 0.6]).roll(i + q))
            _rounded(weights, f"l{i}.hc{q}.out", torch.tensor([1.2, -0.5, 0.3, 0.8]).roll(2 * i + q))
    reqs = X.make_requests(cfg, [40, 9], seed=5)
    want = X.plain_logits(cfg, weights, reqs)
    write = P.write_streams

    def in_turn(Xs, mix, out, y):
        Xs = Xs.clone()
        for t in range(Xs.shape[1]):
            Xs[:, t] = torch.einsum("s,nsc->nc", mix[:, t], Xs) + out[t] * y
        return Xs

    for what, name, wrong in [
        ("the mix's direction", "write_streams", lambda Xs, mix, out, y: write(Xs, mix.T, out, y)),
        ("all copies at once", "write_streams", in_turn),
        ("how much a copy gets", "write_streams", lambda Xs, mix, out, y: write(Xs, mix, torch.ones_like(out), y)),
        ("what is read", "read_streams", lambda Xs, w: Xs[:, 0]),
    ]:
        _shows(cfg, weights, reqs, want, name, wrong, what, share=0.7)
    same = dict(weights, **{f"l1.hc2.{n}": weights[f"l1.hc1.{n}"] for n in ("in", "out", "mix")})
    assert (_differs(P.forward(same, cfg, reqs["r0"]), want["r0"]) > 0.02).float().mean() > 0.7
    _run_all(cfg, weights, reqs, want, backend, "streams", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=12), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_who_is_chosen_and_how_they_weigh(backend):
    """Corrections of about the scores' size, many below minus one, so that choice scores are negative: dropped groups that count
    as zero, groups scored by their best or by all their experts, corrections that weigh too, weights that are not shares, or a
    choice without groups give other logits."""
    device, dtype = backend
    cfg = _layers((_LIGHT, X.moe(9, 2, 16, (3, 1))), streams=2)
    weights = X.random_weights(cfg, seed=41)
    # group 0 holds the best expert and two bad ones, group 1 two good ones, group 2 three middling ones
    _rounded(weights, "l0.mlp.correction", torch.tensor([-0.9, -2.4, -2.6, -1.2, -1.25, -2.8, -1.6, -1.65, -1.6]))
    for e in range(9):
        _rounded(weights, f"l0.mlp.e{e}.down", weights[f"l0.mlp.e{e}.down"] * 3.0)
    reqs = X.make_requests(cfg, [60, 9], seed=5)
    want = X.plain_logits(cfg, weights, reqs)
    route = P.route

    def other(choice_of=None, weight_of=None, kept=None):
        def run(W, p, f, x):
            s = torch.sigmoid(W[p + "router"] @ x)
            c = s + W[p + "correction"]
            allowed = (kept or P.kept_experts)(c, f["router"].get("groups"))
            masked = torch.zeros_like(c) if choice_of == "zero" else torch.full_like(c, -1e9)
            masked[allowed] = c[allowed]
            top = torch.topk(masked, int(f["router"]["top"])).indices.tolist()
            if weight_of == "correction":
                w = c[top] / c[top].sum()
            elif weight_of == "scores":
                w = s[top]
            else:
                w = s[top] / s[top].sum()
            return [(e, float(v)) for e, v in zip(top, w)]
        return run

    def by(score):
        def kept(c, groups):
            per = c.view(groups["count"], -1)
            best = torch.topk(score(per), groups["keep"]).indices.tolist()
            return [g * per.shape[1] + i for g in best for i in range(per.shape[1])]
        return kept

    for what, wrong in [
        ("dropped groups at zero", other(choice_of="zero")),
        ("groups by their best", other(kept=by(lambda per: per.max(1).values))),
        ("groups by all", other(kept=by(lambda per: per.sum(1)))),
        ("no groups", other(kept=lambda c, groups: list(range(9)))),
        ("corrected weights", other(weight_of="correction")),
        ("weights that are no shares", other(weight_of="scores")),
    ]:
        _shows(cfg, weights, reqs, want, "route", wrong, what, share=0.05)
    _shows(cfg, dict(weights, **{"l0.mlp.correction": torch.zeros(9)}), reqs, want, "route", route, "the correction")
    _run_all(cfg, weights, reqs, want, backend, "router", (C.trace_whole, C.trace_portions, lambda r: C.trace_tail(r, tail=25), C.trace_mixed), n_pages=8)


@pytest.mark.parametrize("backend", BACKENDS)
def test_a_captured_decode_step_carries_every_state(backend):
    """Single-token steps of one and of three requests, replayed many times with other steps between them: the states and copies
    that a captured graph updates in place are those of the eager steps."""
    device, dtype = backend
    if device == "cpu":
        pytest.skip("steps are captured on the GPU only")
    cfg, weights, _, _ = setup("odd")
    reqs = X.make_requests(cfg, [40, 37, 44], seed=14)
    want = X.plain_logits(cfg, weights, reqs)
    runner = X.make_runner(cfg, weights, dtype, device, ops_for(device), 16, 12)
    assert runner.use_graphs
    steps = []
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
    cfg = X.CONFIGS["odd"]
    weights = X.random_weights(cfg, seed=X.SEEDS["odd"])
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
    prompts = list(X.make_requests(cfg, [30, 7, 45], seed=9).values())  # (several greedy tokens whose best logits are clearly apart)
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
            if dtype == "bfloat16" and not X.steady(X.plain_logits(cfg, weights, {"a": toks}))["a"][-1]:
                break  # (nor where a rounding decides, see ``steady``)
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
    assert spec.vocab_size == 70 and spec.hidden_size == 42 and len(spec.layers) == 5 and typed.to_dict() == cfg
    assert spec.embedding.kind == "normed_token_embedding" and spec.embedding.params["streams"] == 3 and spec.head.params["tied_to"] is None
    assert (spec.head.params["scale"], spec.head.params["softcap"]) == (0.7, 6.0)
    assert all(layer.block == "mixed_streams" for layer in spec.layers)
    a = spec.layers[2].parts["mixer"].params
    assert (a["num_heads"], a["num_kv_heads"], a["head_dim"], a["value_dim"], a["scale"], a["differential"]["offset"]) == (6, 2, 5, 7, 0.9, 0.1)
    r = spec.layers[3].parts["mixer"]
    assert r.kind == "retention" and r.params["decay"] == [0.9, 0.995] and r.params["position"].params["rotary_dim"] == 6
    assert r.params["position"].params["pairing"] == "half" and r.params["position"].params["theta"] == 50.0
    assert spec.layers[4].parts["mixer"].params["position"] is None and spec.layers[1].parts["mixer"].kind == "lightning_attention"
    f = spec.layers[0].parts["feed_forward"].params
    assert (f["experts"], f["top"], f["groups"], f["choice_correction"]) == (6, 2, {"count": 3, "keep": 2}, "correction")
    assert spec.layers[3].parts["feed_forward"].params["groups"] is None and "feed_forward" not in spec.layers[2].parts
    specs = tensor_specs_for(cfg)
    assert specs["embed"].shape == (70, 42) and specs["embed.norm"].shape == (42,) and specs["head"].shape == (70, 42)
    assert specs["l0.mix.q"].shape == (60, 42) and specs["l0.mix.k"].shape == (20, 42) and specs["l0.mix.v"].shape == (14, 42)
    assert specs["l0.mix.o"].shape == (42, 42) and specs["l0.mix.v.b"].shape == (14,) and specs["l0.mix.lq2"].shape == (5,)
    assert "l2.mix.k" not in specs and "l2.mix.k.b" not in specs and "l2.mix.v" not in specs and specs["l2.mix.q.b"].shape == (60,)
    assert specs["l1.mix.norm"].shape == (15,) and "l3.mix.norm" not in specs and specs["l3.mix.g"].shape == (12, 42)
    assert specs["l0.hc1.mix"].shape == (3, 3) and specs["l1.hc2.in"].shape == (3,) and "l2.hc2.mix" not in specs and "l2.norm2" not in specs
    assert specs["l0.mlp.correction"].shape == (6,) and specs["l0.mlp.e5.gate"].shape == (10, 42) and "l0.mlp.e6.up" not in specs
    for path, value, what in [
        (("layers", 0, "mixer", "kv_heads"), 4, "multiple"), (("layers", 2, "mixer", "kv_from"), 1, "kv_from"),
        (("layers", 2, "mixer", "kv_from"), 2, "kv_from"), (("layers", 2, "mixer", "vdim"), 8, "vdim"),
        (("layers", 0, "type"), "gla", "not one of"), (("layers", 3, "mixer", "rot", "dims"), 12, "dims"),
        (("layers", 3, "mixer", "rot", "dims"), 5, "dims"), (("layers", 1, "mixer", "decay"), [0.5], "decay"),
        (("layers", 1, "mixer", "decay"), [0.5, 0.5, 1.5], "decay"), (("layers", 0, "mlp", "kind"), "table", "kind"),
        (("layers", 0, "mlp", "router", "groups", "count"), 4, "groups"), (("layers", 0, "mlp", "router", "groups", "keep"), 4, "groups"),
        (("layers", 0, "mlp", "router", "top"), 5, "top"), (("layers", 3, "mlp", "router", "top"), 6, "top"),
        (("streams",), 0, "streams"), (("streams",), 17, "streams"), (("layers",), [], "layers"), (("logit_softcap",), -1.0, "logit_softcap"),
    ]:
        bad = copy.deepcopy(cfg)
        node = bad
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        with pytest.raises(ConfigError, match=what):
            spec_from_config(bad)
    for path in (("streams",), ("layers", 0, "mixer", "diff"), ("norm", "eps"), ("layers", 1, "mixer", "decay"), ("layers", 0, "mlp", "expert")):
        missing = copy.deepcopy(cfg)
        node = missing
        for key in path[:-1]:
            node = node[key]
        del node[path[-1]]
        with pytest.raises(ConfigError, match=path[-1]):
            spec_from_config(missing)
    plain = copy.deepcopy(cfg)
    del plain["logit_scale"], plain["logit_softcap"]
    assert spec_from_config(plain)[2].head.params["scale"] == 1.0 and spec_from_config(plain)[2].head.params["softcap"] is None
