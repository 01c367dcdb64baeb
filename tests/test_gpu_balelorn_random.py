"""Balelorn configurations drawn at random, each replayed whole, in portions and mixed against the plain implementation:
any order of layers, chunks from one position to more than a request has, with and without rotation and blending, head
sizes that are and are not whole MFMA tiles, value heads larger and smaller than key heads, widths that are and are not
multiples of 128, feed-forwards dense, mixed or absent, pages of 8 to 32 tokens."""
import random

import pytest
import torch

from tests import balelorn_cases as bc
from tests import replay_cases as rc
from tests.gpu_util import require_gpu
from tests.test_gpu_balelorn import compare

pytestmark = pytest.mark.gpu


def draw_config(seed):
    rng = random.Random(9000 + seed)
    width = rng.choice([128, 256, 384]) if seed % 3 == 0 else rng.choice([8 * rng.randint(5, 40), 4 * rng.randint(9, 70) + 2 * (seed % 2)])
    mix_kv, mix_vdim = rng.choice([1, 2, 3]), rng.choice([8, 16, 40, 64, 96])
    layers = []
    for _ in range(rng.randint(1, 6)):
        blends = rng.random() < 0.6
        kv = mix_kv if blends else rng.choice([1, 2, 3])
        dim = rng.choice([6, 8, 16, 24, 32, 48, 64, 80, 96, 128])
        vdim = mix_vdim if blends else (dim if rng.random() < 0.5 else rng.choice([5, 8, 16, 40, 64, 112]))
        rot = None if rng.random() < 0.15 else dict(base=rng.choice([50.0, 1e4, 5e6]), dims=dim if rng.random() < 0.3 else 2 * rng.randint(1, dim // 2))
        mixer = dict(heads=kv * rng.choice([1, 2, 3, 5]), kv_heads=kv, dim=dim, vdim=vdim, scale=dim ** -0.5 * rng.choice([0.5, 1.0, 1.5]), v_mix=blends,
                     mask=None if rng.random() < 0.2 else dict(size=rng.choice([1, 7, 16, 33, 50, 64, 100, 128, 300])), rot=rot)
        kind = rng.random()
        mlp = None
        if kind < 0.4:
            mlp = dict(kind="dense", ff=rng.choice([8 * rng.randint(1, 30), 16 * rng.randint(1, 20), 2 * rng.randint(3, 40)]))
        elif kind < 0.9:
            experts = rng.choice([1, 2, 4, 6, 8, 16])
            mlp = dict(kind="moe", expert=dict(ff=rng.choice([8, 4]) * rng.randint(1, 20), limit=rng.choice([0.3, 1.0, 4.0])),
                       router=dict(experts=experts, top=rng.randint(1, min(experts, 4))))
        layers.append(dict(type="attention", mixer=mixer, mlp=mlp))
    return dict(architecture="Balelorn", vocab=rng.randint(90, 700), width=width, norm=dict(eps=rng.choice([1e-6, 1e-5, 3e-6])), layers=layers), rng.choice([8, 16, 32])


@pytest.mark.parametrize("seed", range(18))
def test_random_configuration(seed, tmp_path):
    require_gpu()
    cfg, page = draw_config(seed)
    print("seed %d: width %d, page %d, layers %s" % (seed, cfg["width"], page, [(l["mixer"], l["mlp"]) for l in cfg["layers"]]), flush=True)
    folder = bc.write_model(str(tmp_path / "m"), cfg, 300 + seed, bc.both(bc.strong_blend(), bc.heavy_sink()) if seed % 2 else None)
    rng = random.Random(seed)
    reqs = rc.random_requests(cfg["vocab"], [rng.randint(1, 150) for _ in range(5)] + [70, 140], seed=seed)
    ref = bc.plain_logits(folder, reqs)
    for dtype in ("float32", "bfloat16"):
        for name, steps in (("whole", rc.whole(reqs)), ("portions", rc.portions(reqs)), ("mixed", rc.mixed(reqs, seed=seed))):
            out = str(tmp_path / (dtype + name))
            rc.run_replay_inprocess(folder, dtype, out, steps, rc.max_live_tokens(steps), ["--kvcache-block-size", str(page), "--poison-cache"])
            compare(rc.collect(out, steps, cfg["vocab"]), ref, dtype, "seed %d/%s/%s" % (seed, name, dtype), 0.35, 0.06)
