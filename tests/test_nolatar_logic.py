"""Nolatar through the engine's own step function, cache manager, scheduler and entry point, with the CPU stand-in
for the kernels: what is tested here is the logic around them (which layer's cache is read, what state a request has, which
norm sums what, where keys and values go), against the plain implementation."""
import copy
import math

import pytest
import torch

from tests import nolatar_cases as nc
from tests import replay_cases as rc
from tests.plain import nolatar_plain as plain
from tests.plain.nolatar_plain import PlainNolatar

CPU = ["--device", "cpu"]
TOL = dict(atol=3e-4, rtol=3e-4)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    return {name: nc.write_model(str(tmp_path_factory.mktemp("nol_" + name)), cfg, seed, tweak, torch.float32)
            for name, cfg, seed, tweak in (("a", nc.NOL_A, 3, None), ("b", nc.NOL_B, 4, None), ("state", nc.NOL_STATE, 2, nc.slow_decays()),
                                           ("diff", nc.NOL_DIFF, 8, nc.uneven_maps()),
                                           ("a_sharp", nc.NOL_A, 5, nc.both(nc.sharpen(), nc.uneven_maps(), nc.slow_decays(), nc.unread(nc.NOL_A))))}


def test_configuration_is_read_by_name_and_checked():
    from spyinfer_amd.config import ConfigError, NolatarConfig
    from spyinfer_amd.config.registry import architecture_of
    assert architecture_of(nc.NOL_A).name == "Nolatar"
    cfg = NolatarConfig.from_dict(copy.deepcopy(nc.NOL_A))
    assert (cfg.vocab, cfg.width, cfg.norm_eps, len(cfg.layers)) == (89, 40, 2e-6, 7)
    assert cfg.layers[0]["mixer"]["left"]["chunk"] == 13 and cfg.layers[0]["mixer"]["right"]["decay"] == [0.9, 0.97, 0.5]
    assert (cfg.layers[0]["mixer"]["left_scale"], cfg.layers[0]["mixer"]["right_scale"]) == (0.7, -0.4)
    assert [l["mixer"].get("kv_from") for l in cfg.layers] == [None, None, None, 1, None, 1, None]
    assert cfg.layers[1]["mlp"]["shared_ff"] is None and cfg.layers[3]["mlp"] is None and cfg.layers[0]["mlp"]["shared_ff"] == 18
    some = copy.deepcopy(nc.NOL_B)
    for key in ("groups", "norm_groups"):
        del some["layers"][0]["mixer"][key]
    for key in ("kv_heads", "vdim"):
        del some["layers"][2]["mixer"][key]
    del some["layers"][2]["mixer"]["rot"]["dims"]
    read = NolatarConfig.from_dict(some).layers
    assert (read[0]["mixer"]["groups"], read[0]["mixer"]["norm_groups"], read[2]["mixer"]["kv_heads"], read[2]["mixer"]["vdim"]) == (1, 1, 1, 8)
    assert read[2]["mixer"]["rot"]["dims"] == 8
    for path, value in ((("layers", 0, "type"), "conv"), (("layers", 0, "mixer", "left", "kv_heads"), 4), (("layers", 0, "mixer", "left", "rot", "dims"), 5),
                        (("layers", 0, "mixer", "right", "rot", "dims"), 12), (("layers", 0, "mixer", "right", "decay"), [0.9, 0.97]),
                        (("layers", 0, "mixer", "right", "decay"), [0.9, 0.97, 0.0]), (("layers", 0, "mixer", "right", "decay"), [0.9, 0.97, "x"]),
                        (("layers", 0, "mixer", "left_scale"), None), (("layers", 0, "mixer", "left", "mask", "size"), 0),
                        (("layers", 1, "mixer", "diff"), None), (("layers", 3, "mixer", "kv_from"), 0), (("layers", 3, "mixer", "kv_from"), 3),
                        (("layers", 5, "mixer", "kv_from"), 3), (("layers", 3, "mixer", "vdim"), 8), (("layers", 3, "mixer", "rot", "base"), 201.0),
                        (("layers", 2, "mixer", "groups"), 4), (("layers", 2, "mixer", "norm_groups"), 4), (("layers", 2, "mixer", "conv"), 9),
                        (("layers", 2, "mixer", "state"), 0), (("width",), None), (("layers", 1, "mlp", "kind"), "dense"),
                        (("layers", 0, "mlp", "router", "top"), 7), (("layers", 0, "mlp", "shared", "ff"), 0), (("norm", "eps"), 0.0), (("layers",), [])):
        bad = copy.deepcopy(nc.NOL_A)
        node = bad
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        with pytest.raises(ConfigError):
            NolatarConfig.from_dict(bad)


def test_the_model_in_parts():
    from spyinfer_amd.cache.spec import FixedState, PagedKV
    from spyinfer_amd.config import NolatarConfig
    from spyinfer_amd.models.nolatar import build_nolatar
    model = build_nolatar(NolatarConfig.from_dict(copy.deepcopy(nc.NOL_A)))
    # two maps of a key head lie in one row; layers that read another's cache have none of their own; a state is rounded up
    # to whole 16-byte pieces; the retention beside the chunked attention has the cache id behind the layers'
    assert model.cache_specs() == [PagedKV(2, 16, None, 13), PagedKV(2, 16), FixedState((6 * 7 * 5 + 3 * (30 + 42) + 2,)), None,
                                   FixedState((4 * 12 * 8 + 2 * (32 + 24),)), None, PagedKV(1, 32), FixedState((3 * 10 * 6,))]
    assert build_nolatar(NolatarConfig.from_dict(dict(nc.NOL_B, layers=[nc._layer(nc._mamba(3, 2, 5, 1, 1, 1))]))).cache_specs() == [FixedState((3 * 5 * 2 + 2,))]
    assert [(c.layer, c.cache, c.store) for c in model.schedule][3:6] == [(3, 1, False), (4, 4, True), (5, 1, False)]
    names = {s.name: s for s in model.weight_specs() if not s.optional}
    assert names["l1.mix.q"].shape == (48, 40) and names["l1.mix.k"].shape == (24, 40) and names["l5.mix.q"].shape == (72, 40) and names["l5.mix.o"].shape == (40, 54)
    assert not {"l3.mix.k", "l3.mix.v", "l3.mix.k.norm", "l3.norm2", "l3.norm2.b", "l1.mlp.shared.up", "l0.mlp.e0.gate"} & set(names)
    assert names["l2.mix.in"].shape == (30 + 72 + 6, 40) and names["l2.mix.conv"].shape == (72, 4) and names["l2.mix.conv.b"].shape == (72,)
    assert names["l0.mix.left.q.norm"].shape == (12,) and names["l0.mix.right.g"].shape == (18, 40) and names["final.norm.b"].shape == (40,)


@pytest.mark.parametrize("name", ["a", "b", "state", "diff", "a_sharp"])
@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions", "mixed"])
def test_schedules_equal_the_plain_implementation(folders, name, mode, tmp_path, emu_ops):
    folder = folders[name]
    requests = rc.random_requests(nc.vocab_of(folder), [41, 1, 2, 67, 23, 30, 52, 38, 45], 7)
    steps = {"whole": rc.whole, "bulk_tail": lambda r: rc.bulk_tail(r, 12), "portions": rc.portions, "mixed": rc.mixed}[mode](requests)
    if mode == "mixed":
        rc.assert_mixed(steps, name)
    rc.run_replay_inprocess(folder, "float32", str(tmp_path), steps, rc.max_live_tokens(steps), CPU + ["--kvcache-block-size", "8"])
    rc.compare(rc.collect(str(tmp_path), steps, nc.vocab_of(folder)), nc.plain_logits(folder, requests), what="%s/%s" % (name, mode), **TOL)


def test_pages_and_slots_go_back_and_are_used_again(folders, emu_ops):
    from spyinfer_amd.engine.batch import StepEntry
    from spyinfer_amd.engine.runner import ModelRunner, load_model
    folder = folders["a_sharp"]
    model = load_model(folder, "float32", "cpu")
    runner = ModelRunner(model, "float32", "cpu", 4, 26, 2, max_num_batched_tokens=1 << 20)
    plain_model = PlainNolatar.from_folder(folder)
    m = runner.manager
    chunked = next(g for g in m.page_groups if g.spec.chunk == 13)
    for turn in range(3):                          # the same two slots and the same pages serve three pairs of requests
        reqs = rc.random_requests(89, [57, 33], 20 + turn)
        held = {rid: m.admit(rid) for rid in reqs}
        got = {rid: [] for rid in reqs}
        fed = {rid: 0 for rid in reqs}
        while any(fed[r] < len(reqs[r]) for r in reqs):
            entries = []
            for rid, toks in reqs.items():
                n = min(5 if rid == "r0" else 1, len(toks) - fed[rid])
                if n:
                    m.reserve(held[rid], n)
                    entries.append((rid, StepEntry(held[rid], toks[fed[rid]:fed[rid] + n], list(range(n)))))
                    fed[rid] += n
            logits = runner.step([e for _, e in entries])
            r = 0
            for rid, e in entries:
                got[rid].append(logits[r:r + len(e.tokens)].clone())
                r += len(e.tokens)
            m.check()
            assert all(len(held[rid].pages_held(chunked.index)) <= 4 for rid in reqs)      # what lies before the chunk has gone back
        for rid, toks in reqs.items():
            torch.testing.assert_close(torch.cat(got[rid]), plain_model.forward(toks).float(), **TOL)
            m.release(held[rid])
        assert m.num_free_pages() == [g.pool.num_pages for g in m.page_groups] and m.slots.num_free == 2


def test_greedy_generation_through_the_entry_point(folders, emu_ops):
    from spyinfer_amd.engine.llm_engine import LLMEngine
    from spyinfer_amd.sampling import SamplingParams
    folder = folders["a"]
    plain_model = PlainNolatar.from_folder(folder)
    prompts = list(rc.random_requests(89, [5, 17, 2, 30, 9], 9).values())
    want = [plain_model.greedy(p, 10) for p in prompts]
    for opts in (dict(), dict(max_num_batched_tokens=12, prefill_chunk=7, max_num_seqs=2), dict(num_kvcache_blocks=None)):
        kw = dict(dtype="float32", max_model_len=64, num_kvcache_blocks=24, max_num_seqs=4, kvcache_block_size=8, device="cpu")
        kw.update(opts)
        eng = LLMEngine(folder, **kw)
        assert eng.generate(prompts, SamplingParams(max_new_tokens=10, ignore_eos=True)) == want
        eng.runner.manager.check()
    # a pool too small for all requests at once: the request admitted last is preempted, gives its pages and slot back and
    # later runs again from its first token
    eng = LLMEngine(folder, dtype="float32", max_model_len=64, num_kvcache_blocks=9, max_num_seqs=4, kvcache_block_size=8, device="cpu")
    assert eng.generate(prompts, SamplingParams(max_new_tokens=10, ignore_eos=True)) == want
    assert eng.scheduler.num_preemptions > 0
    eng.runner.manager.check()


def test_a_layer_norm_takes_whatever_a_block_leaves_pending(emu_ops):
    from spyinfer_amd.kernels import ops
    from spyinfer_amd.parts import LayerNorm
    g = torch.Generator().manual_seed(3)
    part = LayerNorm(11, 1e-5)
    w, b, x, d = (torch.randn((n, 11) if n > 1 else (11,), generator=g) for n in (1, 1, 4, 4))
    part.bind("n", {"n": w, "n.b": b})
    ref = lambda s: plain.layer_norm(s.double(), w.double(), b.double(), 1e-5).float()
    torch.testing.assert_close(part.add_norm(x.clone(), None, torch.float32), ref(x))
    r = x.clone()
    torch.testing.assert_close(part.add_norm(r, d, torch.float32), ref(x + d))
    torch.testing.assert_close(r, x + d)
    r = x.clone()
    torch.testing.assert_close(part.add_norm(r, (d, ops.WeightedPair(d, x, 2.0, -1.0)), torch.float32, torch.tensor([2, 0], dtype=torch.int32)), ref(3 * d)[[2, 0]])
    torch.testing.assert_close(r, x)
    with pytest.raises(ValueError):
        part.add_normed(x, d, mix=(None, 1, None))


def test_the_plain_pieces():
    """The oracle's own mechanisms by hand."""
    f = torch.float64
    # a rotation of a quarter turn per position and pair, the two layouts of pairs, the rest passing
    x = torch.tensor([[[1.0, 2.0, 3.0, 4.0, 5.0]]], dtype=f).repeat(2, 1, 1)
    pos = torch.tensor([0, 1])
    half, pairs = plain.rotate_half(x, pos, 1.0, 4), plain.rotate_pairs(x, pos, 1.0, 4)
    c, s = math.cos(1.0), math.sin(1.0)
    torch.testing.assert_close(half[1, 0], torch.tensor([c - 3 * s, 2 * c - 4 * s, 3 * c + s, 4 * c + 2 * s, 5.0], dtype=f))
    torch.testing.assert_close(pairs[1, 0], torch.tensor([c - 2 * s, 2 * c + s, 3 * c - 4 * s, 4 * c + 3 * s, 5.0], dtype=f))
    assert torch.equal(half[0], x[0]) and torch.equal(pairs[0], x[0])
    # a convolution: the last tap is the current token's
    y = plain.causal_conv(torch.tensor([[1.0], [10.0], [100.0]], dtype=f), torch.tensor([[1.0, 2.0, 3.0]], dtype=f), torch.tensor([0.5], dtype=f))
    assert y[:, 0].tolist() == [3.5, 32.5, 321.5]
    # retention with one head and one channel: a decaying sum
    w = {n: torch.ones((1, 1), dtype=f) for n in "qkvgo"}
    m = dict(heads=1, dim=1, vdim=1, decay=[0.5], rot=dict(base=10.0, dims=0))
    h = torch.tensor([[1.0], [2.0], [3.0]], dtype=f)
    out = plain.retention(h, w, m, 1e-12)
    torch.testing.assert_close(out[:, 0], plain.silu(h[:, 0]))              # (one value over its own size is one)
    # a state space with one channel: dt = ln 2, so that exp(-1 dt) halves the state
    w = {"in": torch.tensor([[0.0], [1.0], [0.0], [0.0], [0.0]], dtype=f), "conv": torch.tensor([[1.0], [0.0], [0.0]], dtype=f), "conv.b": torch.tensor([0.0, 1.0, 1.0], dtype=f),
         "dt_bias": torch.zeros(1, dtype=f), "A_log": torch.zeros(1, dtype=f), "D": torch.zeros(1, dtype=f), "norm": torch.ones(1, dtype=f), "o": torch.ones((1, 1), dtype=f)}
    m = dict(heads=1, vdim=1, state=1, groups=1, norm_groups=1)
    assert torch.equal(plain.state_space(h, w, m, 1e-6), torch.zeros((3, 1), dtype=f))          # silu(z) = 0 shuts the gate ahead of the norm
    # lambda, and the exact gelu
    lam = plain.lambda_of({"lq1": torch.tensor([1.0, 2.0], dtype=f), "lk1": torch.tensor([0.5, -0.25], dtype=f), "lq2": torch.zeros(2, dtype=f), "lk2": torch.ones(2, dtype=f)}, 0.3)
    assert abs(float(lam) - 0.3) < 1e-12
    torch.testing.assert_close(plain.gelu(torch.tensor([1.0], dtype=f)), torch.tensor([0.8413447460685429], dtype=f))
    # experts: the softmax over the chosen logits alone
    w = {"router": torch.tensor([[1.0], [2.0], [3.0]], dtype=f)}
    for e in range(3):
        w["e%d.up" % e], w["e%d.down" % e] = torch.full((1, 1), 10.0, dtype=f), torch.full((1, 1), float(e + 1), dtype=f)
    out = plain.mixture(torch.ones((1, 1), dtype=f), w, dict(router=dict(top=2)))
    p = 1.0 / (1.0 + math.exp(-1.0))
    torch.testing.assert_close(out[0], torch.tensor([10.0 * (3 * p + 2 * (1 - p))], dtype=f))
    # keys of the query's own chunk only
    assert plain.seen(5, 2).int().tolist() == [[1, 0, 0, 0, 0], [1, 1, 0, 0, 0], [0, 0, 1, 0, 0], [0, 0, 1, 1, 0], [0, 0, 0, 0, 1]]
