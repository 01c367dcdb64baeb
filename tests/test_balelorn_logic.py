"""Balelorn through the engine's own step function, cache manager, scheduler and entry point, with the CPU stand-in
for the kernels: what is tested here is the logic around them (which pages a chunk needs and gives back, whose values are
blended in, which norm feeds what, which experts a token has), against the plain implementation."""
import copy

import pytest
import torch

from tests import balelorn_cases as bc
from tests import replay_cases as rc
from tests.plain.balelorn_plain import PlainBalelorn, chunked_attention, seen, softmax_with_sink

CPU = ["--device", "cpu"]
TOL = dict(atol=3e-4, rtol=3e-4)


@pytest.fixture(scope="module")
def folders(tmp_path_factory):
    tweaks = bc.both(bc.strong_blend(), bc.heavy_sink())
    return {name: bc.write_model(str(tmp_path_factory.mktemp("bal_" + name)), cfg, seed, tweak, torch.float32)
            for name, cfg, seed, tweak in (("a", bc.BAL_A, 3, None), ("b", bc.BAL_B, 4, bc.strong_blend()), ("plain", bc.BAL_PLAIN, 2, None),
                                        ("a_sharp", bc.BAL_A, 5, bc.both(bc.sharpen(), bc.strong_blend())),
                                        ("a_sink", bc.BAL_A, 6, bc.both(tweaks, bc.unread(bc.BAL_A))))}


def test_configuration_is_read_by_name_and_checked():
    from spyinfer_amd.config import BalelornConfig, ConfigError
    from spyinfer_amd.config.registry import architecture_of
    assert architecture_of(bc.BAL_A).name == "Balelorn"
    cfg = BalelornConfig.from_dict(copy.deepcopy(bc.BAL_A))
    assert (cfg.vocab, cfg.width, cfg.norm_eps, len(cfg.layers)) == (89, 40, 2e-6, 5)
    assert [l["mixer"]["chunk"] for l in cfg.layers] == [13, 8, None, 21, 13] and [l["mixer"]["v_mix"] for l in cfg.layers] == [False, True, True, False, True]
    assert cfg.layers[3]["mixer"]["rot"] is None and cfg.layers[1]["mixer"]["rot"] == dict(base=10000.0, dims=4)
    assert cfg.layers[1]["mlp"] == dict(kind="dense", ff=22) and cfg.layers[3]["mlp"] is None
    assert cfg.layers[2]["mlp"] == dict(kind="moe", ff=20, limit=1.5, experts=5, top=3)
    assert BalelornConfig.from_dict(copy.deepcopy(bc.BAL_B)).layers[1]["mixer"]["kv_heads"] == 1
    for path, value in ((("layers", 1, "mixer", "kv_heads"), 3), (("layers", 0, "type"), "conv"), (("layers", 0, "mixer", "rot", "dims"), 3),
                        (("layers", 0, "mixer", "rot", "dims"), 14), (("width",), None), (("layers", 1, "mlp", "kind"), "sparse"),
                        (("layers", 0, "mlp", "router", "top"), 7), (("layers", 0, "mlp", "expert", "limit"), 0.0), (("norm", "eps"), 0.0),
                        (("layers", 0, "mixer", "mask", "size"), 0), (("layers", 2, "mixer", "vdim"), 9), (("layers", 4, "mixer", "kv_heads"), 1),
                        (("layers", 0, "mixer", "v_mix"), 1), (("layers",), [])):
        bad = copy.deepcopy(bc.BAL_A)
        node = bad
        for key in path[:-1]:
            node = node[key]
        node[path[-1]] = value
        with pytest.raises(ConfigError):
            BalelornConfig.from_dict(bad)


def test_the_model_in_parts():
    from spyinfer_amd.cache.spec import PagedKV
    from spyinfer_amd.config import BalelornConfig
    from spyinfer_amd.models.balelorn import build_balelorn
    model = build_balelorn(BalelornConfig.from_dict(copy.deepcopy(bc.BAL_A)))
    specs = model.cache_specs()
    # key and value heads of different sizes share one padded head size; layers of one chunk length share pages only with their like
    assert specs == [PagedKV(1, 16, None, 13), PagedKV(2, 16, None, 8), PagedKV(2, 16), PagedKV(2, 4, None, 21), PagedKV(2, 16, None, 13)]
    assert [l.mixer.value_mix for l in model.layers] == [None, "first", "blend", None, "blend"]
    names = {s.name: s for s in model.weight_specs() if not s.optional}
    assert "l1.mix.vmix" not in names and names["l2.mix.vmix"].shape == () and "l0.mix.vmix" not in names
    assert names["embed.norm"].shape == (40,) and names["l0.ls1"].shape == (40,) and names["l0.norm2b"].shape == (40,)
    assert "l3.norm1b" in names and not {"l3.norm2", "l3.norm2b", "l3.ls2"} & set(names)
    assert names["l2.mlp.table"].shape == (89, 3) and names["l2.mlp.e4.down"].shape == (40, 20) and names["l1.mlp.down"].shape == (40, 22)


def test_a_table_that_names_an_expert_too_many_is_refused(tmp_path, emu_ops):
    from spyinfer_amd.engine.runner import load_model

    def tweak(tensors):
        tensors["l0.mlp.table"][17, 1] = 6
    folder = bc.write_model(str(tmp_path), bc.BAL_A, 3, tweak)
    with pytest.raises(ValueError, match="l0.mlp.table"):
        load_model(folder, "float32", "cpu")


@pytest.mark.parametrize("chunk,page", [(13, 4), (8, 8), (1, 4), (20, 16), (64, 8)])
def test_chunk_pages_are_held_while_they_are_read(chunk, page):
    """Token by token and in portions: a request holds the pages of the chunk that the next token lies in, and no more once
    it has left a chunk's last page."""
    from spyinfer_amd.cache import CacheManager
    from spyinfer_amd.cache.spec import PagedKV
    from spyinfer_amd.cache.manager import window_pages
    m = CacheManager([PagedKV(1, 8, None, chunk), PagedKV(1, 8)], page_size=page, num_pages=80, max_num_seqs=2, max_step_tokens=7)
    assert m.page_groups[0].pool.num_pages == min(80, 2 * window_pages(chunk, page, 7)) and m.page_groups[1].pool.num_pages == 80
    rc_, n = m.admit("x"), 0
    for step in [1, 1, 7, 2, 5, 1, 1, 3, 7, 7, 1, 6, 7, 7, 7, 2, 1, 7, 7, 7, 7, 4, 1, 1, 1]:
        start = n // chunk * chunk                        # the first key that the step's first query reads
        assert all(rc_.tables[0][p] >= 0 for p in range(start // page, -(-n // page)))
        m.reserve(rc_, step)
        assert len(rc_.pages_held(0)) <= window_pages(chunk, page, 7)
        m.commit(rc_, step)
        n += step
        assert all(rc_.tables[0][p] < 0 for p in range(n // chunk * chunk // page))
        m.check()
    assert m.max_tokens_per_request() == 80 * page        # the chunk's group sets no limit
    m.release(rc_)
    assert m.num_free_pages() == [g.pool.num_pages for g in m.page_groups]


def test_a_chunk_cannot_be_rewound_behind_its_pages():
    from spyinfer_amd.cache import CacheManager
    from spyinfer_amd.cache.spec import PagedKV
    m = CacheManager([PagedKV(1, 8, None, 8)], page_size=4, num_pages=8, max_num_seqs=1)
    rc_ = m.admit("x")
    m.reserve(rc_, 15)
    m.commit(rc_, 15)
    assert rc_.tables[0][:2] == [-1, -1] and m.rewind(rc_, 14)
    m.commit(rc_, 1)
    m.reserve(rc_, 1)
    m.commit(rc_, 1)                                       # 16 tokens: the second chunk's pages are gone
    assert not m.rewind(rc_, 15) and m.rewind(rc_, 16)


@pytest.mark.parametrize("name", ["a", "b", "plain", "a_sharp", "a_sink"])
@pytest.mark.parametrize("mode", ["whole", "bulk_tail", "portions", "mixed"])
def test_schedules_equal_the_plain_implementation(folders, name, mode, tmp_path, emu_ops):
    folder = folders[name]
    requests = rc.random_requests(bc.vocab_of(folder), [41, 1, 2, 67, 23, 30, 52, 38, 45], 7)
    steps = {"whole": rc.whole, "bulk_tail": lambda r: rc.bulk_tail(r, 12), "portions": rc.portions, "mixed": rc.mixed}[mode](requests)
    if mode == "mixed":
        rc.assert_mixed(steps, name)
    rc.run_replay_inprocess(folder, "float32", str(tmp_path), steps, rc.max_live_tokens(steps), CPU + ["--kvcache-block-size", "8"])
    rc.compare(rc.collect(str(tmp_path), steps, bc.vocab_of(folder)), bc.plain_logits(folder, requests), what="%s/%s" % (name, mode), **TOL)


def test_pages_go_back_and_are_used_again(folders, emu_ops):
    from spyinfer_amd.engine.batch import StepEntry
    from spyinfer_amd.engine.runner import ModelRunner, load_model
    folder = folders["a_sharp"]
    model = load_model(folder, "float32", "cpu")
    runner = ModelRunner(model, "float32", "cpu", 4, 26, 2, max_num_batched_tokens=1 << 20)
    plain = PlainBalelorn.from_folder(folder)
    m = runner.manager
    chunked = next(g for g in m.page_groups if g.spec.chunk == 8)
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
            assert all(len(held[rid].pages_held(chunked.index)) <= 2 for rid in reqs)      # what lies before the chunk has gone back
        for rid, toks in reqs.items():
            torch.testing.assert_close(torch.cat(got[rid]), plain.forward(toks).float(), **TOL)
            m.release(held[rid])
        assert m.num_free_pages() == [g.pool.num_pages for g in m.page_groups] and m.slots.num_free == 2


def test_greedy_generation_through_the_entry_point(folders, emu_ops):
    from spyinfer_amd.engine.llm_engine import LLMEngine
    from spyinfer_amd.sampling import SamplingParams
    folder = folders["a"]
    plain = PlainBalelorn.from_folder(folder)
    prompts = list(rc.random_requests(89, [5, 17, 2, 30, 9], 9).values())
    want = [plain.greedy(p, 10) for p in prompts]
    for opts in (dict(), dict(max_num_batched_tokens=12, prefill_chunk=7, max_num_seqs=2), dict(num_kvcache_blocks=None)):
        kw = dict(dtype="float32", max_model_len=64, num_kvcache_blocks=24, max_num_seqs=4, kvcache_block_size=8, device="cpu")
        kw.update(opts)
        eng = LLMEngine(folder, **kw)
        assert eng.generate(prompts, SamplingParams(max_new_tokens=10, ignore_eos=True)) == want
        eng.runner.manager.check()
    # a pool too small for all requests at once: the request admitted last is preempted, gives its pages back and later
    # runs again from its first token
    eng = LLMEngine(folder, dtype="float32", max_model_len=64, num_kvcache_blocks=9, max_num_seqs=4, kvcache_block_size=8, device="cpu")
    assert eng.generate(prompts, SamplingParams(max_new_tokens=10, ignore_eos=True)) == want
    assert eng.scheduler.num_preemptions > 0
    eng.runner.manager.check()


def test_the_plain_pieces():
    """The oracle's own mechanisms by hand: who sees whom at a chunk's edges, and what a sink takes."""
    ok = seen(7, 3)
    assert ok.int().tolist() == [[1, 0, 0, 0, 0, 0, 0], [1, 1, 0, 0, 0, 0, 0], [1, 1, 1, 0, 0, 0, 0], [0, 0, 0, 1, 0, 0, 0], [0, 0, 0, 1, 1, 0, 0],
                                 [0, 0, 0, 1, 1, 1, 0], [0, 0, 0, 0, 0, 0, 1]]
    p = softmax_with_sink(torch.zeros((1, 1, 3), dtype=torch.float64), torch.log(torch.tensor([5.0], dtype=torch.float64)))
    torch.testing.assert_close(p[0, 0], torch.full((3,), 0.125, dtype=torch.float64))
    g = torch.Generator().manual_seed(1)
    m = dict(heads=2, kv_heads=1, dim=4, vdim=3, scale=0.5, mask=dict(size=4), rot=dict(base=100.0, dims=2))
    w = {n: torch.randn(s, generator=g, dtype=torch.float64) for n, s in (("q", (8, 6)), ("k", (4, 6)), ("v", (3, 6)), ("g", (6, 6)), ("o", (6, 6)), ("sink", (2,)))}
    h = torch.randn((9, 6), generator=g, dtype=torch.float64)
    whole, _ = chunked_attention(h, w, m, None)
    # a change before the chunk of a position does not reach it; one inside does
    other = h.clone()
    other[3] += 1.0
    changed = (chunked_attention(other, w, m, None)[0] - whole).abs().sum(dim=1) > 1e-9
    assert changed.tolist() == [False, False, False, True, False, False, False, False, False]
