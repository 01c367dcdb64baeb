"""Small Balelorn configurations and helpers shared by the CPU and GPU tests of that design."""
import copy
import json
import os

import torch
from safetensors.torch import load_file, save_file

from tests.plain.balelorn_plain import PlainBalelorn


def _attention(heads, kv_heads, dim, vdim, scale, chunk, v_mix, base=10000.0, dims=None):
    m = dict(heads=heads, dim=dim, vdim=vdim, scale=scale, v_mix=v_mix)
    if kv_heads is not None:
        m["kv_heads"] = kv_heads
    m["mask"] = dict(size=chunk) if chunk else None
    m["rot"] = dict(base=base, dims=dim if dims is None else dims) if base else None
    return m


def _layer(mixer, mlp=None):
    return dict(type="attention", mixer=mixer, mlp=mlp)


def _dense(ff):
    return dict(kind="dense", ff=ff)


def _moe(ff, experts, top, limit):
    return dict(kind="moe", expert=dict(ff=ff, limit=limit), router=dict(experts=experts, top=top))


#: every size differs from every other: value heads larger and smaller than key heads, fewer kv heads than heads, chunks
#: that are and are not whole pages, a layer that reads everything, one without rotation, one without a feed-forward,
#: blending that starts in the second layer and leaves out the fourth
BAL_A = dict(architecture="Balelorn", vocab=89, width=40, norm=dict(eps=2e-6),
             layers=[_layer(_attention(3, 1, 12, 7, 0.3, 13, False, base=500.0, dims=6), _moe(12, 6, 2, 0.8)),
                     _layer(_attention(4, 2, 6, 10, 0.35, 8, True, dims=4), _dense(22)),
                     _layer(_attention(6, 2, 8, 10, 0.25, None, True, base=100.0, dims=2), _moe(20, 5, 3, 1.5)),
                     _layer(_attention(2, 2, 4, 4, 0.5, 21, False, base=None), None),
                     _layer(_attention(2, 2, 14, 10, 0.2, 13, True, dims=10), _moe(8, 3, 1, 0.5))])

#: values that may happen to be equal or 1 elsewhere: one head, one expert of one, chunks of one position and of one page,
#: kv heads not named, every layer blending, the whole head rotated
BAL_B = dict(architecture="Balelorn", vocab=61, width=32, norm=dict(eps=1e-5),
             layers=[_layer(_attention(1, 1, 8, 8, 1.0, 1, True), _moe(32, 1, 1, 1.0)),
                     _layer(_attention(1, None, 8, 8, 0.35, 8, True), _moe(8, 4, 4, 2.0)),
                     _layer(_attention(1, 1, 8, 8, 0.35, 8, True), _dense(32))])

#: no blending at all, the mixture first and last, a chunk longer than any request
BAL_PLAIN = dict(architecture="Balelorn", vocab=53, width=24, norm=dict(eps=1e-6),
                 layers=[_layer(_attention(2, 1, 6, 8, 0.4, 1000, False, dims=2), _moe(9, 3, 2, 1.2)),
                         _layer(_attention(4, 4, 4, 4, 0.5, 5, False)),
                         _layer(_attention(2, 2, 10, 6, 0.3, 17, False, base=1000.0, dims=8), _moe(7, 4, 3, 0.7))])

#: sizes that the products' tiled kernels and the MFMA attention and expert kernels take in bfloat16
BAL_C = dict(architecture="Balelorn", vocab=400, width=128, norm=dict(eps=4e-6),
             layers=[_layer(_attention(4, 2, 64, 32, 0.125, 100, True, dims=32), _dense(256)),
                     _layer(_attention(8, 2, 32, 32, 0.18, 64, True, dims=16), _moe(64, 8, 2, 1.0)),
                     _layer(_attention(4, 1, 128, 128, 0.09, None, False, dims=64), _moe(96, 16, 4, 2.0)),
                     _layer(_attention(6, 2, 48, 32, 0.14, 33, True, dims=48), _moe(128, 4, 1, 0.7))])

#: chunks of hundreds of positions: far keys inside a chunk, and chunk edges among hundreds
BAL_FAR = dict(architecture="Balelorn", vocab=83, width=48, norm=dict(eps=1e-6),
               layers=[_layer(_attention(3, 1, 16, 16, 0.25, 290, True, base=100000.0, dims=8), _moe(24, 4, 2, 1.0)),
                       _layer(_attention(4, 2, 24, 16, 0.2, 77, False, base=300000.0, dims=12), _dense(40)),
                       _layer(_attention(2, 1, 16, 16, 0.25, None, True, base=1000000.0, dims=6), _moe(16, 3, 1, 1.1))])

INIT = dict(matrix_std=0.12, norm_std=0.2, bias_std=0.3)


def write_model(folder, config, seed, tweak=None, dtype=torch.bfloat16):
    """A model folder with random weights; ``tweak(tensors)`` may change them before they are written."""
    from spyinfer_amd.weights import write_random_model
    write_random_model(folder, copy.deepcopy(config), seed, dtype, **INIT)
    path = os.path.join(folder, "model.safetensors")
    tensors = load_file(path)
    (tweak or (lambda t: None))(tensors)
    save_file({k: v.contiguous() for k, v in tensors.items()}, path)
    return folder


def sharpen(factor=6.0):
    """Queries scaled so that a softmax has few large terms: a key that is missed or wrongly seen changes the result by
    much more than rounding, also among hundreds of keys."""
    def tweak(tensors):
        for name in tensors:
            if name.endswith(".mix.q"):
                tensors[name] = (tensors[name].float() * factor).to(tensors[name].dtype)
    return tweak


def heavy_sink(values=(2.5, -1.0, 4.0)):
    """Sinks that take a large share of every softmax and differ from head to head: one that is left out, counted twice,
    scaled or taken from another head shows."""
    def tweak(tensors):
        for name in tensors:
            if name.endswith(".mix.sink"):
                t = tensors[name]
                tensors[name] = torch.tensor([values[i % len(values)] for i in range(t.shape[0])], dtype=t.dtype)
    return tweak


def strong_blend(values=(0.7, -0.4, 0.9)):
    """Blending numbers far from 0 and 1, and one in the layer that does not use its own (a checkpoint may hold it)."""
    def tweak(tensors):
        stored = sorted((n for n in tensors if n.endswith(".mix.vmix")), key=lambda n: int(n[1:n.index(".")]))
        for i, name in enumerate(stored):
            tensors[name] = torch.tensor(values[i % len(values)], dtype=tensors[name].dtype)
    return tweak


def unread(config):
    """Tensors that a checkpoint may hold and nothing reads: the first blending layer's number, and the norms and scale of
    a feed-forward that a layer does not have."""
    def tweak(tensors):
        some = next(iter(tensors.values()))
        firsts = [i for i, l in enumerate(config["layers"]) if l["mixer"].get("v_mix")]
        if firsts:
            tensors["l%d.mix.vmix" % firsts[0]] = torch.tensor(0.6, dtype=some.dtype)
        for i, layer in enumerate(config["layers"]):
            if not layer["mlp"]:
                for n in ("norm2", "norm2b", "ls2"):
                    tensors["l%d.%s" % (i, n)] = torch.full((config["width"],), 2.0, dtype=some.dtype)
    return tweak


def both(*tweaks):
    def tweak(tensors):
        for t in tweaks:
            t(tensors)
    return tweak


def plain_logits(folder, requests):
    plain = PlainBalelorn.from_folder(folder)
    return {rid: plain.forward(toks) for rid, toks in requests.items()}


def vocab_of(folder):
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)["vocab"]
