"""Small Nolatar configurations and helpers shared by the CPU and GPU tests of that design."""
import copy
import json
import os

import torch
from safetensors.torch import load_file, save_file

from tests.plain.nolatar_plain import PlainNolatar


def _rot(base, dims):
    return dict(base=base, dims=dims)


def _attention(heads, kv_heads, dim, vdim, scale, diff, base=10000.0, dims=None, kv_from=None):
    m = dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, diff=diff, rot=_rot(base, dim if dims is None else dims))
    if kv_from is not None:
        m["kv_from"] = kv_from
    return "attention", m


def _mamba(heads, vdim, state, groups, conv, norm_groups):
    return "mamba2", dict(heads=heads, vdim=vdim, state=state, groups=groups, conv=conv, norm_groups=norm_groups)


def _parallel(left, right, scales):
    heads, kv_heads, dim, vdim, scale, chunk, base, dims = left
    rheads, rdim, rvdim, decay, rbase, rdims = right
    return "parallel", dict(left=dict(heads=heads, kv_heads=kv_heads, dim=dim, vdim=vdim, scale=scale, mask=dict(size=chunk), rot=_rot(base, dims)),
                            right=dict(heads=rheads, dim=rdim, vdim=rvdim, decay=decay, rot=_rot(rbase, rdims)),
                            left_scale=scales[0], right_scale=scales[1])


def _layer(mixer, mlp=None):
    return dict(type=mixer[0], mixer=mixer[1], mlp=mlp)


def _moe(ff, experts, top, shared=None):
    m = dict(kind="moe", expert=dict(ff=ff), router=dict(experts=experts, top=top))
    if shared:
        m["shared"] = dict(ff=shared)
    return m


#: every size differs from every other: rotations of part of a head, values larger and smaller than keys, groups that heads
#: share, norm groups that are not those groups, two layers that read the same earlier layer's cache with more and fewer
#: query heads than it has, a layer without a feed-forward, a mixture without an expert for everyone
NOL_A = dict(architecture="Nolatar", vocab=89, width=40, norm=dict(eps=2e-6),
             layers=[_layer(_parallel((6, 2, 12, 7, 0.3, 13, 500.0, 6), (3, 10, 6, [0.9, 0.97, 0.5], 300.0, 8), (0.7, -0.4)), _moe(12, 6, 2, 18)),
                     _layer(_attention(4, 2, 6, 9, 0.4, 0.25, 200.0, 4), _moe(14, 5, 3)),
                     _layer(_mamba(6, 5, 7, 3, 4, 2), _moe(9, 3, 1, 11)),
                     _layer(_attention(2, 2, 6, 9, 0.5, 0.6, 200.0, 4, kv_from=1)),
                     _layer(_mamba(4, 8, 12, 1, 3, 4), _moe(20, 4, 4, 6)),
                     _layer(_attention(6, 2, 6, 9, 0.3, 0.1, 200.0, 4, kv_from=1), _moe(12, 7, 2, 30)),
                     _layer(_attention(3, 1, 10, 4, 0.35, 0.45, 50.0, 10), _moe(8, 2, 2, 5))])

#: values that may happen to be equal or 1 elsewhere: one head, one group, one tap, one expert of one, chunks of one position
#: and of one page, no decay at all, equal scales
NOL_B = dict(architecture="Nolatar", vocab=61, width=32, norm=dict(eps=1e-5),
             layers=[_layer(_mamba(1, 8, 8, 1, 1, 1), _moe(32, 1, 1, 32)),
                     _layer(_parallel((1, 1, 8, 8, 1.0, 1, 10000.0, 8), (1, 8, 8, [1.0], 10000.0, 8), (1.0, 1.0)), _moe(8, 4, 4, 8)),
                     _layer(_attention(1, 1, 8, 8, 0.35, 0.5), _moe(16, 2, 1)),
                     _layer(_parallel((2, 2, 8, 8, 0.35, 8, 100.0, 2), (2, 8, 8, [0.25, 0.999], 100.0, 2), (0.5, 0.5)))])

#: only the recurrent mixers (no pages), and only the attention
NOL_STATE = dict(architecture="Nolatar", vocab=53, width=24, norm=dict(eps=1e-6),
                 layers=[_layer(_mamba(3, 6, 5, 3, 2, 3), _moe(9, 3, 2, 7)), _layer(_mamba(2, 10, 9, 2, 8, 1))])
NOL_DIFF = dict(architecture="Nolatar", vocab=57, width=36, norm=dict(eps=1e-6),
                layers=[_layer(_attention(2, 1, 8, 16, 0.4, 0.2), _moe(10, 3, 2, 9)), _layer(_attention(4, 1, 8, 16, 0.3, 0.7, kv_from=0), _moe(6, 2, 1))])

#: sizes that the products' tiled kernels, the MFMA attention and expert kernels and whole tiles of the recurrences take
NOL_C = dict(architecture="Nolatar", vocab=400, width=128, norm=dict(eps=4e-6),
             layers=[_layer(_attention(4, 2, 32, 64, 0.18, 0.3, 10000.0, 16), _moe(64, 8, 2, 128)),
                     _layer(_mamba(8, 32, 64, 2, 4, 4), _moe(96, 16, 4, 64)),
                     _layer(_parallel((8, 2, 64, 48, 0.125, 100, 10000.0, 32), (4, 64, 64, [0.96, 0.99, 0.995, 0.999], 10000.0, 64), (0.55, 0.6)), _moe(128, 4, 1, 96)),
                     _layer(_attention(8, 2, 32, 64, 0.18, 0.5, 10000.0, 16, kv_from=0), _moe(64, 4, 2, 256)),
                     _layer(_attention(4, 1, 64, 128, 0.125, 0.2), _moe(32, 8, 3, 64)),
                     _layer(_mamba(4, 80, 48, 1, 3, 2), _moe(40, 4, 2, 128))])

#: far keys among hundreds, chunks of hundreds of positions, slow decays
NOL_FAR = dict(architecture="Nolatar", vocab=83, width=48, norm=dict(eps=1e-6),
               layers=[_layer(_attention(3, 1, 16, 24, 0.25, 0.3, 100000.0, 8), _moe(24, 4, 2, 16)),
                       _layer(_parallel((4, 2, 16, 16, 0.25, 290, 300000.0, 12), (2, 16, 12, [0.998, 0.9999], 1000000.0, 16), (0.6, 0.5)), _moe(16, 3, 1, 20)),
                       _layer(_attention(3, 1, 16, 24, 0.3, 0.4, 100000.0, 8, kv_from=0)),
                       _layer(_mamba(4, 12, 16, 2, 4, 2), _moe(12, 3, 2, 8))])

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


def sharpen(factor=5.0):
    """Query norms scaled so that a softmax has few large terms: a key that is missed or wrongly seen changes the result by
    much more than rounding, also among hundreds of keys."""
    def tweak(tensors):
        for name in tensors:
            if name.endswith(".q.norm"):
                tensors[name] = (tensors[name].float() * factor).to(tensors[name].dtype)
    return tweak


def uneven_maps():
    """Vectors behind lambda that make it differ from layer to layer and lie far from 0 and 1 (maps taken for each other show)."""
    def tweak(tensors):
        for name in tensors:
            if name.endswith((".lq1", ".lk1")):
                t = tensors[name]
                tensors[name] = torch.full_like(t, 0.6 / t.shape[0] ** 0.5)
            if name.endswith((".lq2", ".lk2")):
                t = tensors[name]
                tensors[name] = torch.full_like(t, (0.3 if name.endswith("q2") else -0.8) / t.shape[0] ** 0.5)
    return tweak


def slow_decays(shift=-4.0):
    """State-space decays near one: what a request wrote hundreds of tokens ago is still read."""
    def tweak(tensors):
        for name in tensors:
            if name.endswith(".A_log"):
                tensors[name] = (tensors[name].float() + shift).to(tensors[name].dtype)
    return tweak


def unread(config):
    """Tensors that a checkpoint may hold and nothing reads: the norm of a feed-forward that a layer does not have."""
    def tweak(tensors):
        some = next(iter(tensors.values()))
        for i, layer in enumerate(config["layers"]):
            if not layer["mlp"]:
                for n in ("norm2", "norm2.b"):
                    tensors["l%d.%s" % (i, n)] = torch.full((config["width"],), 2.0, dtype=some.dtype)
    return tweak


def both(*tweaks):
    def tweak(tensors):
        for t in tweaks:
            t(tensors)
    return tweak


def plain_logits(folder, requests):
    plain = PlainNolatar.from_folder(folder)
    return {rid: plain.forward(toks) for rid, toks in requests.items()}


def vocab_of(folder):
    with open(os.path.join(folder, "config.json")) as f:
        return json.load(f)["vocab"]
