"""Nolatar configurations drawn at random, each replayed whole, in portions and mixed against the plain implementation: any
order of layers, layers that read an earlier layer's cache, chunks from one position to more than a request has, head and
state sizes that are and are not whole tiles, values larger and smaller than keys, widths that are and are not multiples of
128, mixtures with and without an expert for everyone, pages of 8 to 32 tokens."""
import random

import pytest
import torch

from tests import nolatar_cases as nc
from tests import replay_cases as rc
from tests.gpu_util import require_gpu
from tests.test_gpu_nolatar import compare

pytestmark = pytest.mark.gpu


def _dims(rng, dim):
    return dim // 2 * 2 if rng.random() < 0.3 else 2 * rng.randint(1, max(1, dim // 2))


def draw_config(seed):
    rng = random.Random(5000 + seed)
    width = rng.choice([128, 256, 384]) if seed % 3 == 0 else rng.choice([8 * rng.randint(5, 40), 4 * rng.randint(9, 70) + 2 * (seed % 2)])
    layers, owners = [], []
    for i in range(rng.randint(1, 6)):
        kind = rng.choice(["mamba2", "attention", "attention", "parallel"])
        if kind == "mamba2":
            groups, per = rng.choice([1, 2, 3]), rng.choice([1, 2, 4])
            heads, vdim = groups * per, rng.choice([3, 8, 16, 20, 48, 64])
            mixer = nc._mamba(heads, vdim, rng.choice([5, 8, 16, 33, 64, 128]), groups, rng.choice([1, 2, 3, 4, 4, 6]), rng.choice([1, heads, vdim if vdim % 2 else 2]) if heads * vdim % 2 == 0 else 1)
        elif kind == "attention":
            if owners and rng.random() < 0.5:
                src = rng.choice(owners)
                own = layers[src]["mixer"]
                mixer = nc._attention(own["kv_heads"] * rng.choice([1, 2, 3]), own["kv_heads"], own["dim"], own["vdim"], own["dim"] ** -0.5 * rng.choice([0.7, 1.4]),
                                      rng.choice([0.1, 0.5, 0.8]), own["rot"]["base"], own["rot"]["dims"], src)
            else:
                kv, dim = rng.choice([1, 2, 3]), rng.choice([6, 8, 15, 16, 24, 32, 48, 64, 80])
                mixer = nc._attention(kv * rng.choice([1, 2, 4]), kv, dim, rng.choice([5, 8, 2 * dim, dim, 40, 96]), dim ** -0.5 * rng.choice([0.7, 1.0, 1.4]), rng.choice([0.1, 0.3, 0.6]),
                                      rng.choice([50.0, 1e4, 5e6]), _dims(rng, dim))
                owners.append(i)
        else:
            kv, dim, rdim, rheads = rng.choice([1, 2, 3]), rng.choice([6, 8, 16, 24, 32, 48, 64, 96]), rng.choice([6, 8, 16, 32, 48, 64, 128]), rng.choice([1, 2, 3, 4])
            mixer = nc._parallel((kv * rng.choice([1, 2, 5]), kv, dim, rng.choice([5, 8, dim, 40, 64]), dim ** -0.5 * rng.choice([0.7, 1.4]), rng.choice([1, 7, 16, 33, 64, 100, 128, 300]),
                                  rng.choice([50.0, 1e4]), _dims(rng, dim)),
                                 (rheads, rdim, rng.choice([5, 8, 16, 32, 64, 80]), [rng.choice([0.4, 0.9, 0.99, 0.9995, 1.0]) for _ in range(rheads)], rng.choice([50.0, 1e6]), _dims(rng, rdim)),
                                 (rng.choice([0.3, 1.0]), rng.choice([-0.5, 0.8])))
        mlp = None
        if rng.random() < 0.8:
            experts = rng.choice([1, 2, 4, 6, 8, 16])
            mlp = nc._moe(rng.choice([8, 4]) * rng.randint(1, 20), experts, rng.randint(1, min(experts, 4)), rng.choice([None, 8 * rng.randint(1, 24), 2 * rng.randint(3, 40)]))
        layers.append(nc._layer(mixer, mlp))
    return dict(architecture="Nolatar", vocab=rng.randint(90, 700), width=width, norm=dict(eps=rng.choice([1e-6, 1e-5, 3e-6])), layers=layers), rng.choice([8, 16, 32])


@pytest.mark.parametrize("seed", range(18))
def test_random_configuration(seed, tmp_path):
    require_gpu()
    cfg, page = draw_config(seed)
    print("seed %d: width %d, page %d, layers %s" % (seed, cfg["width"], page, [(l["type"], l["mixer"], l["mlp"]) for l in cfg["layers"]]), flush=True)
    folder = nc.write_model(str(tmp_path / "m"), cfg, 300 + seed, nc.both(nc.uneven_maps(), nc.slow_decays(-3.0)) if seed % 2 else None)
    rng = random.Random(seed)
    reqs = rc.random_requests(cfg["vocab"], [rng.randint(1, 150) for _ in range(5)] + [70, 140], seed=seed)
    ref = nc.plain_logits(folder, reqs)
    for dtype in ("float32", "bfloat16"):
        for name, steps in (("whole", rc.whole(reqs)), ("portions", rc.portions(reqs)), ("mixed", rc.mixed(reqs, seed=seed))):
            out = str(tmp_path / (dtype + name))
            rc.run_replay_inprocess(folder, dtype, out, steps, rc.max_live_tokens(steps), ["--kvcache-block-size", str(page), "--poison-cache"])
            compare(rc.collect(out, steps, cfg["vocab"]), ref, dtype, "seed %d/%s/%s" % (seed, name, dtype), 0.06, 0.2)
