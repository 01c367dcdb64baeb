"""Nolatar from parts: a plain embedding and an output head of its own, blocks whose sublayers read the stream itself and add
a layer norm of their result to it, mixers 'mamba2' (a state space), 'attention' (differential, some layers reading an
earlier layer's cache) and 'parallel' (an attention in chunks beside a retention) in the order the configuration lists,
mixtures of ungated experts with an expert for every token as feed-forwards.  Tensor names: ``embed``, ``l<i>.mix.*``,
``l<i>.norm1`` and ``.b``, ``l<i>.mlp.*``, ``l<i>.norm2`` and ``.b``, ``final.norm`` and ``.b``, ``head``."""
from __future__ import annotations

from ..config.model_config import NolatarConfig
from ..config.registry import register_architecture
from ..parts import (DenseMLP, DifferentialAttention, LayerNorm, LMHead, MoEMLP, OutputNormBlock, PagedAttention, Retention, RotaryEmbedding,
                     SideBySide, StateSpace, TokenEmbedding)
from ..weights.loader import WeightSpec
from .base import DecoderModel, LayerCall

ATTENTION_NAMES = dict(q=".q", k=".k", v=".v", o=".o", q_norm=".q.norm", k_norm=".k.norm")


def _rotation(m, interleaved: bool = False):
    rot = m["rot"]
    return RotaryEmbedding(m["dim"], rot["base"], rot["dims"], interleaved=interleaved) if rot else None


def build_nolatar(cfg: NolatarConfig) -> DecoderModel:
    W, eps = cfg.width, cfg.norm_eps
    layers, calls = [], []
    for i, layer in enumerate(cfg.layers):
        m, source = layer["mixer"], None
        if layer["type"] == "mamba2":
            mixer = StateSpace(W, m["heads"], m["vdim"], m["state"], m["groups"], m["conv"], m["norm_groups"], eps)
        elif layer["type"] == "attention":
            source = m["kv_from"]
            mixer = DifferentialAttention(W, m["heads"], m["kv_heads"], m["dim"], m["vdim"], _rotation(m, interleaved=True), m["scale"], eps,
                                          m["diff"], own_kv=source is None, names=ATTENTION_NAMES)
        else:
            a, r = m["left"], m["right"]
            left = PagedAttention(W, a["heads"], a["kv_heads"], a["dim"], _rotation(a), qk_norm_eps=eps, scale=a["scale"], value_dim=a["vdim"],
                                  names=ATTENTION_NAMES, chunk=a["chunk"], formed_angles=True)
            mixer = SideBySide(W, left, Retention(W, r["heads"], r["dim"], r["vdim"], r["decay"], _rotation(r), eps),
                               scales=(m["left_scale"], m["right_scale"]))
        f = layer["mlp"]
        ffn = None
        if f is not None:
            shared = DenseMLP(W, f["shared_ff"], "gelu") if f["shared_ff"] else None
            ffn = MoEMLP(W, f["ff"], f["experts"], f["top"], correction=False, activation="gelu", shared=shared)
        # (a layer without a feed-forward has no use for its norm; a checkpoint may hold it all the same)
        unread = [WeightSpec("norm2", (W,), "norm"), WeightSpec("norm2.b", (W,), "bias")] if ffn is None else ()
        layers.append(OutputNormBlock(mixer, LayerNorm(W, eps), ffn, LayerNorm(W, eps) if ffn is not None else None, unread=unread))
        calls.append(LayerCall(i, i if source is None else source, source is None))
    names = dict(embed="embed", layers="l%d", final_norm="final.norm", lm_head="head")
    return DecoderModel(cfg, TokenEmbedding(cfg.vocab, W, suffix=""), None, layers, LayerNorm(W, eps), LMHead(cfg.vocab, W, suffix=""), calls, names)


register_architecture("Nolatar", NolatarConfig, build_nolatar)
