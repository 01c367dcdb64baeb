"""Nolatar on the GPU: every new or extended mechanism's kernel against the plain implementation, then whole models
through the trace replay (the engine's step function, cache manager and kernels) under every schedule, keys at the edges of
chunks, long decoding, and greedy generation through the entry point with and without captured steps."""
import json
import os
import subprocess
import sys

import pytest
import torch

from tests import nolatar_cases as nc
from tests import replay_cases as rc
from tests.gpu_util import close, require_gpu
from tests.plain import nolatar_plain as plain
from tests.test_gpu_sodedra import DT, TOL, i32, rnd, two_steps

pytestmark = pytest.mark.gpu
DTYPES = ["float32", "bfloat16"]


def compare(got, ref, dtype, what, median=0.04, decile=0.12):
    """float32: every logit within a small tolerance.  bfloat16: a row's error, root mean square over the vocabulary,
    against the row's own root mean square, in the median and for nine rows in ten (a router's close call may pick another
    expert for a row, in every layer anew; float32 holds every row)."""
    if dtype == "float32":
        return rc.compare(got, ref, what=what, **TOL["float32"])
    assert got, "the replay wrote no logits"
    rel = []
    for (rid, pos), row in sorted(got.items(), key=lambda kv: (str(kv[0][0]), kv[0][1])):
        want = ref[rid][pos].double()
        err = torch.from_numpy(row).double() - want
        assert bool(torch.isfinite(err).all()), "%s: request %r position %d is not finite" % (what, rid, pos)
        rel.append(float(err.pow(2).mean().sqrt() / want.pow(2).mean().sqrt()))
    rel = torch.tensor(rel)
    assert float(rel.median()) < median and float(rel.quantile(0.9)) < decile, \
        "%s: rows are off by %.3f of their size in the median, %.3f at the ninth decile" % (what, float(rel.median()), float(rel.quantile(0.9)))


# ---- norms of results ---------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H", [(13, 50), (5, 2048), (70, 1100), (9, 42), (3, 8192), (2, 9000), (40, 320), (2, 20000), (17, 4096)])
def test_layer_normed_results_into_the_stream(dtype, T, H):
    """Rows, a weighted pair and experts' unsummed rows; rows with a mean far from zero (deviations are squared behind the
    mean)."""
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    g = torch.Generator().manual_seed(H + T)
    base, y, z = rnd(g, T, H).float(), (rnd(g, T, H, std=0.3) + 3.0).to(DT[dtype]), rnd(g, T, H).to(DT[dtype])
    w, b = (1 + 0.3 * rnd(g, H)).to(DT[dtype]), rnd(g, H, std=0.5).to(DT[dtype])
    ref = lambda r: base.double() + plain.layer_norm(r, w.double(), b.double(), 1e-3)
    out, copy = ops.layer_norm_residual(base.to(dev), y.to(dev), w.to(dev), b.to(dev), 1e-3, None, DT[dtype])
    close(out, ref(y.double()), torch.float32, scale=2.0, what="rows")
    assert (copy is None) == (dtype == "float32")
    if copy is not None:
        close(copy, ref(y.double()), torch.bfloat16, what="copy")
    r = base.to(dev)
    pair = ops.WeightedPair(y.to(dev), z.to(dev), 0.7, -1.3)
    out, _ = ops.layer_norm_residual(r, pair, w.to(dev), b.to(dev), 1e-3, r)
    close(r, ref(0.7 * y.double() - 1.3 * z.double()), torch.float32, scale=2.0, what="pair, in place")
    close(pair.resolve(), 0.7 * y.double() - 1.3 * z.double(), DT[dtype], scale=2.0, what="resolved pair")
    top, n = 3, T * 3 + 5
    rows = torch.randperm(n, generator=g)[:T * top].to(torch.int32)
    ey, wt = rnd(g, n, H).float(), torch.rand((T, top), generator=g)
    for weights, add in ((wt, None), (None, z)):
        summed = 0.37 * (ey.double()[rows.long()].view(T, top, H) * (weights.double()[:, :, None] if weights is not None else 1.0)).sum(1)
        summed = summed + (add.double() if add is not None else 0.0)
        to = lambda t: None if t is None else t.to(dev)
        ex = ops.ExpertRows(ey.to(dev), rows.to(dev), to(weights), to(add), top, 0.37, T, DT[dtype])
        out, _ = ops.layer_norm_residual(base.to(dev), ex, w.to(dev), b.to(dev), 1e-3)
        close(out, ref(summed), torch.float32, scale=2.0, what="experts")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,H", [(9, 50), (3, 4096), (5, 1100), (4, 1026), (3, 20000), (2, 320), (2, 9000), (3, 14336)])
def test_layer_norm_of_the_stream_at_picked_rows(dtype, T, H):
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    g = torch.Generator().manual_seed(H)
    x, w, b = (rnd(g, T, H) + 2.0).float(), (1 + 0.3 * rnd(g, H)).to(DT[dtype]), rnd(g, H, std=0.5).to(DT[dtype])
    ref = plain.layer_norm(x.double(), w.double(), b.double(), 1e-4)
    close(ops.layer_norm(x.to(dev), w.to(dev), b.to(dev), 1e-4, DT[dtype]), ref, DT[dtype], scale=2.0, what="all rows")
    close(ops.layer_norm(x.to(dev), w.to(dev), b.to(dev), 1e-4, DT[dtype], i32([T - 1, 0, T - 1], dev)), ref[[T - 1, 0, T - 1]], DT[dtype], scale=2.0, what="picked rows")


# ---- feed-forwards ------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,K,I", [(1, 128, 96), (7, 40, 22), (16, 256, 1024), (33, 128, 64), (64, 384, 48), (65, 128, 80), (200, 72, 40), (48, 128, 6160), (3, 24, 20)])
def test_ungated_feed_forward_with_the_exact_gelu(dtype, T, K, I):
    from spyinfer_amd.parts import DenseMLP
    from tests.test_gpu_parts import bind
    dev = require_gpu()
    part = DenseMLP(K, I, "gelu")
    w = bind(part, "m", DT[dtype], dev, 40, 0.3)
    assert set(w) == {"m.up", "m.down"}
    x = rnd(torch.Generator().manual_seed(T), T, K).to(DT[dtype])
    ref = plain.ungated_ff(x.double(), w["m.up"].double(), w["m.down"].double())
    close(part.forward(x.to(dev), None), ref, DT[dtype], scale=4.0, what="gelu feed-forward")


def test_gelu_at_the_ends_of_its_range():
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    z = torch.tensor([0.0, -0.0, 1e-6, -1e-6, 0.5, -0.5, 3.0, -3.0, 5.0, -5.0, 8.0, -8.0, 40.0, -40.0, 1e4, -1e4, 2.0])
    close(ops.gelu(z.clone().to(dev)), plain.gelu(z.double()), torch.float32, what="gelu")
    close(ops.gelu(z[:16].clone().to(dev)), plain.gelu(z[:16].double()), torch.float32, what="gelu, four at a time")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [1, 6, 40, 150])
@pytest.mark.parametrize("W,F,E,top,shared", [(40, 12, 6, 2, 18), (128, 64, 8, 3, 256), (32, 32, 1, 1, None), (256, 96, 5, 5, 40), (64, 40, 33, 4, None)])
def test_mixture_of_ungated_experts(dtype, T, W, F, E, top, shared):
    """Every row: the inputs are drawn so that no choice is a close call."""
    from spyinfer_amd.parts import DenseMLP, MoEMLP
    from tests.test_gpu_parts import bind
    dev = require_gpu()
    part = MoEMLP(W, F, E, top, correction=False, activation="gelu", shared=DenseMLP(W, shared, "gelu") if shared else None)
    w = bind(part, "m", DT[dtype], dev, 60, 0.15)
    g = torch.Generator().manual_seed(T + E)
    x = rnd(g, 4 * T + 200, W).to(DT[dtype])
    z = (x.double() @ w["m.router"].double().T).sort(dim=1, descending=True).values
    clear = (z[:, top - 1] - z[:, top] > 1e-3) if top < E else torch.ones(x.shape[0], dtype=torch.bool)
    x = x[clear][:T].contiguous()
    assert x.shape[0] == T
    mlp = dict(router=dict(top=top), shared=shared and dict(ff=shared))
    ref = plain.mixture(x.double(), {k[2:]: v.double() for k, v in w.items()}, mlp)
    close(part.forward(x.to(dev), None), ref, DT[dtype], scale=4.0, what="mixture")
    close(part.forward_unsummed(x.to(dev), None).combine(), ref, DT[dtype], scale=4.0, what="unsummed rows")


# ---- attention ----------------------------------------------------------------------------------
def _bind(part, dtype, dev, seed, std, tweak=None):
    """Random weights; returns them in float64 under their names behind the prefix."""
    from tests.test_gpu_parts import bind
    seen = {}
    orig = part.bind

    def tweaked(prefix, weights):
        if tweak is not None:
            tweak(weights)
        seen.update({k[2:]: v.double().cpu() for k, v in weights.items()})
        orig(prefix, weights)
    part.bind = tweaked
    bind(part, "a", DT[dtype], dev, seed, std)
    return seen


def _run_parts(parts, layers, manager, dtype, dev, x, spans):
    """One step: every part of ``parts`` in turn on the same rows ``x``; ``layers``: (cache, store) of each."""
    from tests.test_gpu_parts import make_batch
    batch, entries = make_batch(manager, DT[dtype], dev, spans)
    for p in parts:
        p.plan(batch)
    batch.upload()
    outs = [p.forward(x.to(dev), batch, cache, store) for p, (cache, store) in zip(parts, layers)]
    for e in entries:
        manager.commit(e.cache, len(e.tokens))
    return outs


def _whole_then_cut(parts, layers, manager, dtype, dev, x, other, refs, tol, whats):
    """A whole sequence; then the same in portions and single tokens beside another request, in pages used again."""
    T = x.shape[0]

    def run(spans, xs):
        return _run_parts(parts, layers, manager, dtype, dev, torch.cat(xs), spans)
    a = manager.admit("a")
    for y, ref, what in zip(run([(a, T)], [x]), refs, whats):
        close(y, ref, DT[dtype], scale=tol, what=what + ": whole")
    manager.release(a)
    b, a = manager.admit("b"), manager.admit("a")
    cut = T - 7
    rows = [[y[5:] for y in run([(b, 5), (a, 11)], [other[:5], x[:11]])], [y[:cut - 11] for y in run([(a, cut - 11), (b, 1)], [x[11:cut], other[5:6]])]]
    for t in range(cut, T):
        ys = run([(b, 1), (a, 1)] if t % 2 else [(a, 1)], [other[6:7], x[t:t + 1]] if t % 2 else [x[t:t + 1]])
        rows.append([y[-1:] for y in ys])
    for i, (ref, what) in enumerate(zip(refs, whats)):
        close(torch.cat([r[i] for r in rows]), ref, DT[dtype], scale=tol, what=what + ": portions and single tokens")
    manager.check()


# heads, kv heads, map size, value size, rotated dims, tokens
DIFF_CASES = [(4, 2, 32, 64, 16, 150), (3, 1, 12, 10, 8, 70), (2, 2, 64, 128, 64, 300), (6, 3, 48, 96, 48, 330), (4, 1, 32, 48, 30, 1100), (16, 2, 16, 32, 16, 200),
              (2, 1, 96, 64, 96, 140), (1, 1, 128, 256, 128, 90), (2, 2, 5, 40, 4, 60), (12, 1, 32, 40, 8, 100)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,d,dv,dims,T", DIFF_CASES)
def test_differential_attention_and_a_layer_that_reads_its_cache(dtype, H, G, d, dv, dims, T):
    from spyinfer_amd.cache import CacheManager
    from spyinfer_amd.cache.storage import CacheStorage
    from spyinfer_amd.models.nolatar import ATTENTION_NAMES
    from spyinfer_amd.parts import DifferentialAttention, RotaryEmbedding
    dev = require_gpu()
    W, eps, base = 72, 1e-4, 3000.0
    cfgs = [dict(heads=h, kv_heads=G, dim=d, vdim=dv, scale=s, diff=lam, rot=dict(base=base, dims=dims)) for h, s, lam in ((H, 1.2 * d ** -0.5, 0.3), (3 * G, 0.8 * d ** -0.5, 0.55))]
    parts = [DifferentialAttention(W, m["heads"], G, d, dv, RotaryEmbedding(d, base, dims, interleaved=True), m["scale"], eps, m["diff"], own_kv=i == 0, names=ATTENTION_NAMES)
             for i, m in enumerate(cfgs)]

    def tweak(weights):
        for n, v in (("lq1", 0.6), ("lk1", 0.7), ("lq2", 0.4), ("lk2", -0.9)):
            weights["a." + n] = torch.full_like(weights["a." + n], v / d ** 0.5)
    ws = [_bind(p, dtype, dev, 10 + 30 * i, 0.15, tweak) for i, p in enumerate(parts)]
    g = torch.Generator().manual_seed(20)
    x, other = rnd(g, T, W).to(DT[dtype]), rnd(g, 9, W).to(DT[dtype])
    first, kv = plain.differential_attention(x.double(), ws[0], cfgs[0], eps)
    second, _ = plain.differential_attention(x.double(), ws[1], cfgs[1], eps, kv)
    manager = CacheManager([parts[0].cache_spec()], page_size=16, num_pages=2 * (T // 16 + 2), max_num_seqs=3)
    storage = CacheStorage(manager, DT[dtype], dev)
    storage.fill(float("nan"))
    # (the difference of two nearly equal maps, normed, carries their rounding many times over; an angle in float32 is off
    # by up to 1e-7 of itself, which at position 1000 shows)
    _whole_then_cut(parts, [(storage.layer(0), True), (storage.layer(0), False)], manager, dtype, dev, x, other, (first, second),
                    (6.0 if T < 1000 else 24.0) if dtype == "float32" else 8.0, ("own cache", "another's cache"))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("nq,nkv,d,dv,chunk,dims,T", [(6, 2, 32, 32, 24, 16, 150), (4, 4, 64, 80, 50, 30, 300), (8, 1, 16, 48, 1, 2, 60), (3, 1, 12, 10, 16, 8, 70),
                                                      (2, 2, 128, 128, 130, 64, 300), (6, 3, 96, 96, 48, 96, 330), (4, 2, 64, 64, 700, 48, 1100), (20, 1, 64, 48, 200, 32, 420)])
def test_attention_in_chunks_with_normed_heads(dtype, nq, nkv, d, dv, chunk, dims, T):
    from spyinfer_amd.cache import CacheManager
    from spyinfer_amd.cache.storage import CacheStorage
    from spyinfer_amd.models.nolatar import ATTENTION_NAMES
    from spyinfer_amd.parts import PagedAttention, RotaryEmbedding
    dev = require_gpu()
    W, eps, scale = 72, 1e-4, 1.3 * d ** -0.5
    cfg = dict(heads=nq, kv_heads=nkv, dim=d, vdim=dv, scale=scale, mask=dict(size=chunk), rot=dict(base=3000.0, dims=dims))
    part = PagedAttention(W, nq, nkv, d, RotaryEmbedding(d, 3000.0, dims), qk_norm_eps=eps, scale=scale, value_dim=dv, names=ATTENTION_NAMES, chunk=chunk, formed_angles=True)
    w = _bind(part, dtype, dev, 10, 0.15)
    g = torch.Generator().manual_seed(20)
    x, other = rnd(g, T, W).to(DT[dtype]), rnd(g, 9, W).to(DT[dtype])
    ref = plain.chunked_attention(x.double(), w, cfg, eps)
    manager = CacheManager([part.cache_spec()], page_size=16, num_pages=2 * (T // 16 + 2), max_num_seqs=3)
    storage = CacheStorage(manager, DT[dtype], dev)
    storage.fill(float("nan"))
    _whole_then_cut([part], [(storage.layer(0), True)], manager, dtype, dev, x, other, (ref,), (3.0 if T < 1000 else 24.0) if dtype == "float32" else 6.0, ("chunks",))


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("d,dv,chunk,page", [(64, 64, 100, 16), (64, 48, 64, 8), (32, 32, 45, 32), (128, 128, 256, 16), (40, 40, 30, 16)])
def test_keys_just_inside_and_just_outside_a_chunk(dtype, d, dv, chunk, page):
    """Keys that stand out by far lie at the last position of every chunk and at the first: each decides the result of the
    queries that see it, and a chunk that is one position off changes those rows by much more than the tolerance (shown with
    the mistake in the oracle).  In a prompt, and decoded token by token over the edges."""
    from spyinfer_amd.cache import CacheManager
    from spyinfer_amd.cache.storage import CacheStorage
    from spyinfer_amd.models.nolatar import ATTENTION_NAMES
    from spyinfer_amd.parts import PagedAttention
    dev = require_gpu()
    W, nq, nkv, T, eps = 64, 4, 2, 2 * chunk + 9, 1e-6
    cfg = dict(heads=nq, kv_heads=nkv, dim=d, vdim=dv, scale=14.0 / d, mask=dict(size=chunk), rot=dict(base=10.0, dims=0))

    def beacons(weights):
        # coordinate 0 of the input is one everywhere and makes all of a query's values but the last; coordinate 1 marks the
        # keys that point the queries' way, coordinate 2 those that point elsewhere
        for n, rows in (("q", nq), ("k", nkv)):
            m = torch.zeros((rows, d, W))
            if n == "q":
                m[:, :, 0] = 1.0
            else:
                m[:, :, 1] = 1.0
                m[:, ::2, 2], m[:, 1::2, 2] = 1.0, -1.0
            weights["a." + n] = m.view(rows * d, W).to(weights["a." + n])
            weights["a.%s.norm" % n] = torch.ones_like(weights["a.%s.norm" % n])
    part = PagedAttention(W, nq, nkv, d, None, qk_norm_eps=eps, scale=cfg["scale"], value_dim=dv, names=ATTENTION_NAMES, chunk=chunk, formed_angles=True)
    w = _bind(part, dtype, dev, 3, 0.2, beacons)
    g = torch.Generator().manual_seed(chunk)
    x = rnd(g, T, W, std=0.5)
    x[:, 0], x[:, 1], x[:, 2] = 1.0, 0.0, 1.0
    for p in (0, chunk - 1, chunk, 2 * chunk - 1, 2 * chunk):
        x[p, 1], x[p, 2] = 1.0, 0.0
    x = x.to(DT[dtype])
    ref = plain.chunked_attention(x.double(), w, cfg, eps)
    tol = 3.0 if dtype == "float32" else 6.0
    for off in (-1, 1):
        wrong = plain.chunked_attention(x.double(), w, dict(cfg, mask=dict(size=chunk + off)), eps)
        with pytest.raises(AssertionError):
            close(wrong, ref, DT[dtype], scale=4 * tol)
    manager = CacheManager([part.cache_spec()], page_size=page, num_pages=2 * (T // page + 2), max_num_seqs=2)
    storage = CacheStorage(manager, DT[dtype], dev)
    storage.fill(float("nan"))
    layers = [(storage.layer(0), True)]
    a = manager.admit("a")
    close(_run_parts([part], layers, manager, dtype, dev, x, [(a, T)])[0], ref, DT[dtype], scale=tol, what="prompt")
    manager.release(a)
    a = manager.admit("a")
    at, rows = 0, []
    for n in [chunk - 3] + [1] * 6 + [chunk - 6] + [1] * 6 + [2, 4]:
        rows.append(_run_parts([part], layers, manager, dtype, dev, x[at:at + n], [(a, n)])[0])
        at += n
    assert at == T
    close(torch.cat(rows), ref, DT[dtype], scale=tol, what="decoded over the edges")


# ---- recurrences --------------------------------------------------------------------------------
def rows_close(got, ref, dtype, what):
    """Row by row, root mean square against root mean square: a norm over a few values that happen to be small carries the
    rounding of its inputs many times over, so single elements say little.  bfloat16: nine rows in ten."""
    got, ref = got.detach().double().cpu(), ref.double()
    rel = (got - ref).pow(2).mean(dim=1).sqrt() / ref.pow(2).mean(dim=1).sqrt()
    assert bool(torch.isfinite(rel).all()), "%s: row %d is not finite" % (what, int(torch.nonzero(~torch.isfinite(rel))[0]))
    worst = float(rel.max() if dtype == "float32" else rel.quantile(0.9))
    assert worst < (1e-4 if dtype == "float32" else 0.05) and float(rel.median()) < (1e-5 if dtype == "float32" else 0.012), \
        "%s: rows are off by %.2g of their size in the median, %.2g in the worst (row %d)" % (what, float(rel.median()), worst, int(rel.argmax()))


def _run_mixer(part, manager, storage, dtype, dev, x, spans):
    return _run_parts([part], [(storage.layer(0), True)], manager, dtype, dev, x, spans)[0]


def _recurrence_in_cuts(part, dtype, dev, xs, refs):
    """Three requests at once, cut into portions of every kind beside each other (single tokens alone, single tokens beside
    portions, two tokens, many pieces), in slots that are used a second time."""
    from spyinfer_amd.cache import CacheManager
    from spyinfer_amd.cache.storage import CacheStorage
    manager = CacheManager([part.cache_spec()], page_size=16, num_pages=8, max_num_seqs=3)
    storage = CacheStorage(manager, DT[dtype], dev)
    storage.fill(float("nan"))

    def start(name):
        rc_ = manager.admit(name)
        part_state = storage.layer(0)
        manager.state_groups[0].spec.reset(part_state, torch.tensor([rc_.slot], device=dev))
        return rc_
    for turn in range(2):
        held = [start("r%d" % i) for i in range(len(xs))]
        at, got, k = [0] * len(xs), [[] for _ in xs], turn
        cuts = [[300, 1, 1, 64, 2, 130, 1, 5], [1, 1, 65, 1, 63, 3, 200, 1], [2, 1, 128, 1, 1, 1, 40, 9]]
        while any(a < x.shape[0] for a, x in zip(at, xs)):
            spans, rows, order = [], [], []
            for i in (range(len(xs)) if k % 2 else reversed(range(len(xs)))):
                n = min(cuts[(i + turn) % 3][k % 8], xs[i].shape[0] - at[i])
                if n and not (k % 5 == 4 and i == 1):
                    spans.append((held[i], n))
                    rows.append(xs[i][at[i]:at[i] + n])
                    order.append((i, n))
                    at[i] += n
            k += 1
            if not spans:
                continue
            y, r = _run_mixer(part, manager, storage, dtype, dev, torch.cat(rows), spans), 0
            for i, n in order:
                got[i].append(y[r:r + n])
                r += n
        for i, (ref, rc_) in enumerate(zip(refs, held)):
            rows_close(torch.cat(got[i]), ref, dtype, "request %d, turn %d" % (i, turn))
            manager.release(rc_)
    manager.check()


LENGTHS = [331, 70, 9]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,d,dv,dims", [(3, 10, 6, 8), (2, 64, 64, 64), (4, 128, 128, 64), (1, 8, 8, 8), (2, 16, 33, 2), (2, 40, 200, 40), (1, 256, 256, 256), (5, 33, 12, 30), (3, 96, 80, 96)])
def test_retention(dtype, H, d, dv, dims):
    from spyinfer_amd.parts import Retention, RotaryEmbedding
    dev = require_gpu()
    W, eps = 56, 1e-4
    decay = [1.0, 0.999, 0.97, 0.5, 0.03][:H] if H > 1 else [0.995]
    cfg = dict(heads=H, dim=d, vdim=dv, decay=decay, rot=dict(base=500.0, dims=dims))
    part = Retention(W, H, d, dv, decay, RotaryEmbedding(d, 500.0, dims), eps)
    w = _bind(part, dtype, dev, 30, 0.2)
    g = torch.Generator().manual_seed(d)
    xs = [rnd(g, n, W).to(DT[dtype]) for n in LENGTHS]
    _recurrence_in_cuts(part, dtype, dev, xs, [plain.retention(x.double(), w, cfg, eps) for x in xs])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,dv,N,G,conv,ng", [(6, 5, 7, 3, 4, 2), (4, 64, 128, 1, 4, 4), (8, 32, 64, 2, 3, 1), (1, 8, 8, 1, 1, 1), (2, 80, 16, 2, 8, 2), (4, 12, 40, 2, 2, 8),
                                              (2, 160, 256, 1, 4, 2), (3, 7, 5, 1, 5, 3)])
def test_state_space(dtype, H, dv, N, G, conv, ng):
    from spyinfer_amd.parts import StateSpace
    dev = require_gpu()
    W, eps = 56, 1e-4
    cfg = dict(heads=H, vdim=dv, state=N, groups=G, conv=conv, norm_groups=ng)
    part = StateSpace(W, H, dv, N, G, conv, ng, eps)

    def tweak(weights):
        # (decays from slow to fast, step sizes of every size)
        weights["a.A_log"] = torch.linspace(-4.0, 1.5, H).to(weights["a.A_log"])
        weights["a.dt_bias"] = torch.linspace(-3.0, 2.0, H).to(weights["a.dt_bias"])
        weights["a.conv"] = weights["a.conv"] * 3
        weights["a.conv.b"] = weights["a.conv.b"] * 3
    w = _bind(part, dtype, dev, 30, 0.2, tweak)
    g = torch.Generator().manual_seed(N)
    xs = [rnd(g, n, W).to(DT[dtype]) for n in LENGTHS]
    _recurrence_in_cuts(part, dtype, dev, xs, [plain.state_space(x.double(), w, cfg, eps) for x in xs])


def test_a_token_that_forgets_everything_leaves_the_others_their_decays():
    """Steps of every size beside each other: decays of e^-3000 and of 1 - 1e-3 in one piece."""
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    g = torch.Generator().manual_seed(4)
    T, H, d, dv = 150, 2, 16, 8
    q, k, v = (rnd(g, T, H * n).float() for n in (d, d, dv))
    raw = torch.full((T, H), -7.0)
    raw[torch.rand((T, H), generator=g) < 0.1] = 300.0
    bias, rate = torch.zeros(H), torch.tensor([1.0, 10.0])
    dt = torch.nn.functional.softplus(raw.double())

    def walk(q, k, v):
        S, ref = torch.zeros((H, d, dv), dtype=torch.float64), torch.zeros((T, H, dv), dtype=torch.float64)
        for t in range(T):
            S = torch.exp(-rate.double() * dt[t])[:, None, None] * S + (dt[t][:, None] * k[t].double().view(H, d))[:, :, None] * v[t].double().view(H, 1, dv)
            ref[t] = torch.einsum("hij,hi->hj", S, q[t].double().view(H, d))
        return ref, S
    ref, S = walk(q, k, v)
    size, _ = walk(q.abs(), k.abs(), v.abs())          # what a sum's rounding is in proportion to
    state = torch.zeros((1, H * d * dv), device=dev)
    pieces = i32([0, 0, 0, 0, 64, 128, 64, 128, 150, 0, 0, 0], dev)
    out = ops.decay_memory(*(t.to(dev) for t in (q, k, v)), H, H, d, dv, state, i32([0, T], dev), i32([0], dev), (pieces, 3, True), steps=(raw.to(dev), bias.to(dev), rate.to(dev)))
    err = (out.double().cpu().view(T, H, dv) - ref).abs() / size
    assert float(err.max()) < 2e-6, "decays are off by %.2g" % float(err.max())
    assert float((state.double().cpu().view(H, d, dv) - S).abs().max()) < 2e-6 * float(S.abs().max())


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("C,n", [(48, 4), (512, 2), (2056, 3), (50, 4), (64, 1), (24, 7), (4096, 4)])
@pytest.mark.parametrize("with_bias", [True, False])
def test_short_convolution_of_many_tokens(dtype, C, n, with_bias):
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    g = torch.Generator().manual_seed(C + n)
    lengths, cut = [150, 3, 41, 90], [77, 1, 41, 2]
    wide = rnd(g, sum(lengths), C + 16).to(DT[dtype])
    taps, bias = rnd(g, C, n).to(DT[dtype]), rnd(g, C).to(DT[dtype])
    ref, first = [], 0
    for m in lengths:
        ref.append(plain.silu(plain.causal_conv(wide[first:first + m, 8:8 + C].double(), taps.double(), bias.double() if with_bias else 0.0)))
        first += m
    ref = torch.cat(ref)
    state = torch.zeros((4, 5 + (n - 1) * C), device=dev)
    for rows, cu, sl, ent in two_steps(lengths, cut):
        x = wide[rows].to(dev)
        y = ops.causal_conv_silu(x[:, 8:8 + C], taps.to(dev), state, 5, i32(ent, dev), i32(cu, dev), i32(sl, dev), bias=bias.to(dev) if with_bias else None)
        close(y, ref[rows], DT[dtype], scale=2.0, what="convolution")
    last = [first for first in (149, 152, 193, 283)]
    slots = [2, 0, 3, 1]
    x1 = rnd(g, 4, C + 16).to(DT[dtype])
    # one more token each: the kernel for single tokens, from what the portions left
    hist = [torch.cat([wide[max(0, e + 1 - m):e + 1, 8:8 + C], x1[i:i + 1, 8:8 + C]]).double() for i, (e, m) in enumerate(zip(last, lengths))]
    want = torch.stack([plain.silu(plain.causal_conv(h, taps.double(), bias.double() if with_bias else 0.0))[-1] for h in hist])
    y = ops.causal_conv_silu(x1.to(dev)[:, 8:8 + C], taps.to(dev), state, 5, i32([0, 1, 2, 3], dev), i32([0, 1, 2, 3, 4], dev), i32(slots, dev),
                             bias=bias.to(dev) if with_bias else None)
    close(y, want, DT[dtype], scale=2.0, what="single tokens")


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,groups", [(60, 4), (4096, 1), (4096, 8), (1100, 2), (33, 33), (20000, 1), (8192, 1), (1024, 8), (1000, 8)])
def test_norm_in_groups_with_a_gate(dtype, N, groups):
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    g = torch.Generator().manual_seed(N)
    y, w, gate = rnd(g, 5, N).float(), (1 + 0.3 * rnd(g, N)).to(DT[dtype]), rnd(g, 5, N + 7).to(DT[dtype])
    ref = plain.over_rms(y.double().view(5, groups, -1), 1e-3).reshape(5, N)
    close(ops.group_norm(y.to(dev), w.to(dev), 1e-3, groups, DT[dtype]), ref * w.double(), DT[dtype], what="weighted")
    close(ops.group_norm(y.to(dev), None, 1e-3, groups, DT[dtype], gate.to(dev)[:, 7:]), ref * plain.silu(gate[:, 7:].double()), DT[dtype], what="gated")


def test_what_the_kernels_assume_is_checked():
    from spyinfer_amd.kernels import ops
    dev = require_gpu()
    z = lambda *s: torch.zeros(s, device=dev)
    q, st, cu, sl = z(2, 8), z(2, 64), i32([0, 1, 2], dev), i32([0, 1], dev)
    good = dict(H=1, G=1, d=8, dv=8, state=st, cu_q=cu, slot_ids=sl, pieces=None, log_decay=z(1))
    ops.decay_memory(q, q, q, **good)
    for bad in (dict(log_decay=None), dict(log_decay=z(2)), dict(d=16), dict(state=z(2, 60)), dict(norm_eps=1e-5), dict(gate=q), dict(steps=(z(2, 1), z(1), z(1))),
                dict(angles=z(2, 5, 2)), dict(slot_ids=i32([0], dev)), dict(d=300)):
        with pytest.raises(ops.KernelError):
            ops.decay_memory(q, q, q, **dict(good, **bad))
    x, pos, one = z(3, 40), i32([0, 1, 2], dev), z(4)
    ops.norm_rope_store(x, 2, 1, 4, 6, 16, one, None, 1e-5, None, 0, pos, None, None, 8, None, maps=2)
    for bad in (dict(d=6), dict(rotary_dim=2), dict(rotary_dim=3, freq=z(1)), dict(n_q=6), dict(slots=pos), dict(positions=i32([0], dev))):
        kw = dict(n_q=2, n_kv=1, dim=4, value_dim=6, d=16, q_norm_w=one, k_norm_w=None, eps=1e-5, freq=None, rotary_dim=0, positions=pos, k_cache=None, v_cache=None,
                  page_size=8, slots=None, maps=2)
        kw.update(bad)
        with pytest.raises(ops.KernelError):
            ops.norm_rope_store(x, **kw)
    with pytest.raises(ops.KernelError):
        ops.map_difference(z(2, 30), 2, 4, 8, 0.3, 1e-5, 0.7)
    with pytest.raises(ops.KernelError):
        ops.layer_norm_residual(z(3, 4), z(2, 4), one, one, 1e-5)


# ---- whole models ------------------------------------------------------------------------------
MODELS = {"a": (nc.NOL_A, 3, None), "b": (nc.NOL_B, 4, None), "c": (nc.NOL_C, 6, nc.slow_decays()), "state": (nc.NOL_STATE, 2, nc.slow_decays()),
          "diff": (nc.NOL_DIFF, 8, nc.uneven_maps()),
          "a_sharp": (nc.NOL_A, 5, nc.both(nc.sharpen(), nc.uneven_maps(), nc.slow_decays(), nc.unread(nc.NOL_A))),
          "c_sharp": (nc.NOL_C, 12, nc.both(nc.sharpen(3.0), nc.slow_decays())), "far_sharp": (nc.NOL_FAR, 8, nc.both(nc.sharpen(6.0), nc.uneven_maps(), nc.slow_decays(-6.0)))}


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: nc.write_model(str(tmp_path_factory.mktemp("gnol_" + name)), cfg, seed, tweak) for name, (cfg, seed, tweak) in MODELS.items()}


# (sharpened scores carry several times the rounding of a bfloat16 key: those models are held in float32 only)
@pytest.mark.parametrize("name,dtype", [(n, d) for n in ("a", "b", "c", "state", "diff", "a_sharp") for d in DTYPES if not (n.endswith("sharp") and d == "bfloat16")])
@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions", "mixed"])
def test_schedules_equal_the_plain_implementation(folders, name, mode, dtype, tmp_path):
    require_gpu()
    folder = folders[name]
    requests = rc.random_requests(nc.vocab_of(folder), [41, 1, 2, 130, 23, 30, 52, 38, 75], 7)
    steps = {"whole": rc.whole, "bulk_tail": lambda r: rc.bulk_tail(r, 40), "portions": rc.portions, "mixed": rc.mixed}[mode](requests)
    rc.run_replay_inprocess(folder, dtype, str(tmp_path), steps, rc.max_live_tokens(steps),
                            ["--kvcache-block-size", "8" if not name.startswith("c") else "16", "--poison-cache"])
    compare(rc.collect(str(tmp_path), steps, nc.vocab_of(folder)), nc.plain_logits(folder, requests), dtype, "%s/%s/%s" % (name, mode, dtype))


@pytest.mark.parametrize("name", ["far_sharp", "c_sharp"])
@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions", "mixed"])
def test_far_keys_and_chunk_edges_among_hundreds_of_tokens(folders, name, mode, tmp_path):
    """Sharp scores and slow decays: what decides a row's result lies anywhere in 600 tokens, across many pages and pieces."""
    require_gpu()
    folder = folders[name]
    requests = rc.random_requests(nc.vocab_of(folder), [600, 333, 2, 150], 12)
    steps = {"whole": rc.whole, "bulk_tail": lambda r: rc.bulk_tail(r, 50), "portions": lambda r: rc.portions(r, (100, 3, 2, 257, 64, 1)),
             "mixed": lambda r: rc.mixed(r, seed=3)}[mode](requests)
    rc.run_replay_inprocess(folder, "float32", str(tmp_path), steps, rc.max_live_tokens(steps), ["--poison-cache"])
    rc.compare(rc.collect(str(tmp_path), steps, nc.vocab_of(folder)), nc.plain_logits(folder, requests), what="far/" + mode, **TOL["float32"])


@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions"])
def test_long_requests_in_bfloat16_on_the_matrix_cores(folders, mode, tmp_path):
    """Portions of hundreds of tokens take the attention's large tiles and the recurrences' pieces, single tokens over hundreds
    of keys the small ones with the keys cut into parts; the experts' products take their kernels for many rows."""
    require_gpu()
    folder = folders["c"]
    requests = rc.random_requests(400, [700, 260], 21)
    steps = {"whole": rc.whole, "bulk_tail": lambda r: rc.bulk_tail(r, 60), "portions": lambda r: rc.portions(r, (300, 2, 129, 64, 5, 411, 33))}[mode](requests)
    rc.run_replay_inprocess(folder, "bfloat16", str(tmp_path), steps, rc.max_live_tokens(steps), ["--poison-cache"])
    compare(rc.collect(str(tmp_path), steps, 400), nc.plain_logits(folder, requests), "bfloat16", "long/%s" % mode)


@pytest.mark.parametrize("name,dtype", [("a_sharp", "float32"), ("c", "bfloat16")])
def test_long_decoding(folders, name, dtype, tmp_path):
    """250 tokens one by one over the edges of every layer's chunks, in a pool that holds no more than the request."""
    require_gpu()
    folder = folders[name]
    requests = rc.random_requests(nc.vocab_of(folder), [260], 13)
    steps = rc.bulk_tail(requests, 250)
    rc.run_replay_inprocess(folder, dtype, str(tmp_path), steps, rc.max_live_tokens(steps), ["--kvcache-block-size", "8", "--poison-cache"])
    compare(rc.collect(str(tmp_path), steps, nc.vocab_of(folder)), nc.plain_logits(folder, requests), dtype, "long decoding")


def test_a_batch_of_unequal_requests_equals_each_alone(folders, tmp_path):
    """One step over single tokens and portions of requests of very different lengths, against the same steps alone."""
    require_gpu()
    folder = folders["c"]
    requests = rc.random_requests(400, [310, 5, 101, 64], 17)
    first = {"r0": 290, "r1": 4, "r2": 60, "r3": 63}
    together = [dict(step=0, entries=[dict(id=r, tokens=t[:first[r]], want=[]) for r, t in requests.items()], end=[]),
                dict(step=1, entries=[dict(id=r, tokens=t[first[r]:], want=list(range(len(t) - first[r]))) for r, t in requests.items()], end=list(requests))]
    alone = []
    for r, t in requests.items():
        alone += [dict(step=len(alone), entries=[dict(id=r, tokens=t[:first[r]], want=[])], end=[]),
                  dict(step=len(alone) + 1, entries=[dict(id=r, tokens=t[first[r]:], want=list(range(len(t) - first[r])))], end=[r])]
    for dtype, lim in (("float32", 1e-4), ("bfloat16", 0.05)):
        got = {}
        for name, steps in (("together", together), ("alone", alone)):
            out = str(tmp_path / (dtype + name))
            rc.run_replay_inprocess(folder, dtype, out, steps, rc.max_live_tokens(steps), ["--poison-cache"])
            got[name] = rc.collect(out, steps, 400)
        assert set(got["together"]) == set(got["alone"])
        off = []
        for key, row in got["together"].items():
            a, b = torch.from_numpy(row).double(), torch.from_numpy(got["alone"][key]).double()
            off.append(float((a - b).pow(2).mean().sqrt() / b.pow(2).mean().sqrt()))
        # (in bfloat16 a router's close call may pick another expert for a row)
        off = torch.tensor(off)
        assert float(off.max() if dtype == "float32" else off.quantile(0.9)) < lim, "%s: rows depend on their batch (%.3g)" % (dtype, float(off.max()))


# ---- the entry point ---------------------------------------------------------------------------
@pytest.mark.parametrize("eager", [True, False])
def test_greedy_generation_equals_plain(folders, eager):
    from spyinfer_amd.engine.llm_engine import LLMEngine
    from spyinfer_amd.sampling import SamplingParams
    require_gpu()
    folder = folders["a"]
    model = plain.PlainNolatar.from_folder(folder)
    prompts = list(rc.random_requests(89, [5, 17, 2, 30, 9], 9).values())
    want = [model.greedy(p, 24) for p in prompts]
    for opts in (dict(), dict(max_num_batched_tokens=12, prefill_chunk=7, max_num_seqs=2)):
        kw = dict(dtype="float32", max_model_len=64, num_kvcache_blocks=24, max_num_seqs=4, kvcache_block_size=8, enforce_eager=eager)
        kw.update(opts)
        eng = LLMEngine(folder, **kw)
        assert eng.generate(prompts, SamplingParams(max_new_tokens=24, ignore_eos=True)) == want
        if not eager:
            assert eng.runner.graph_replays > 0
        eng.runner.manager.check()


def test_bfloat16_generation_follows_the_plain_logits(folders):
    from spyinfer_amd.engine.llm_engine import LLMEngine
    from spyinfer_amd.sampling import SamplingParams
    require_gpu()
    folder = folders["c"]
    model = plain.PlainNolatar.from_folder(folder)
    prompts = list(rc.random_requests(400, [33, 90, 8], 10).values())
    eng = LLMEngine(folder, dtype="bfloat16", max_model_len=128, num_kvcache_blocks=40, max_num_seqs=4, enforce_eager=False)
    outs = eng.generate(prompts, SamplingParams(max_new_tokens=24, ignore_eos=True))
    assert eng.runner.graph_replays > 0
    clear = total = 0
    for p, out in zip(prompts, outs):
        toks = list(p)
        for t in out:
            logits = model.forward(toks)[-1]
            best = int(torch.argmax(logits))
            clear += t == best or float(logits[best] - logits[t]) < 0.25 * float(logits.pow(2).mean().sqrt())
            total += 1
            toks.append(t)
    # (a router's close call may pick another expert for a token)
    assert clear >= 0.9 * total, "%d of %d tokens are ones that the plain logits do not prefer" % (total - clear, total)


def test_trace_run_as_a_program(folders, tmp_path):
    require_gpu()
    folder = folders["b"]
    requests = rc.random_requests(61, [19, 40], 14)
    steps = rc.portions(requests)
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, os.path.join(root, "bin", "trace_run"), "--model", folder, "--dtype", "float32", "--out", str(tmp_path),
                        "--max-tokens", str(rc.max_live_tokens(steps))], input="".join(json.dumps(s) + "\n" for s in steps),
                       capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    rc.compare(rc.collect(str(tmp_path), steps, 61), nc.plain_logits(folder, requests), what="trace_run", **TOL["float32"])


def test_command_line_generates(folders):
    require_gpu()
    root = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))
    r = subprocess.run([sys.executable, "-m", "spyinfer_amd", "-m", folders["a"], "--dtype", "float32", "--random-prompts", "5,9",
                        "--max-new-tokens", "6", "--max-model-len", "64", "--num-kvcache-blocks", "16", "--max-num-seqs", "4"],
                       cwd=root, capture_output=True, text=True, timeout=600)
    assert r.returncode == 0, r.stderr[-2000:]
    assert r.stdout.strip(), "the command line printed no tokens"
