"""Balelorn from parts: an embedding that is normed before the first layer and an output head of its own, blocks that norm a
sublayer's input and its result (the latter times a learned vector), attention in chunks with a sink per head, blended
values and an output gate, feed-forwards dense or as a mixture whose experts a table names by token id, or none.  Tensor
names: ``embed``, ``embed.norm``, ``l<i>.norm1``, ``l<i>.mix.*``, ``l<i>.norm1b``, ``l<i>.ls1``, ``l<i>.norm2``,
``l<i>.mlp.*``, ``l<i>.norm2b``, ``l<i>.ls2``, ``final.norm``, ``head``."""
from __future__ import annotations

from ..config.model_config import BalelornConfig
from ..config.registry import register_architecture
from ..kernels import ops
from ..parts import (GatedMLP, LMHead, PagedAttention, PreNormBlock, ResultNorm, RMSNorm, RotaryEmbedding, TableMoEMLP, TokenEmbedding)
from ..weights.loader import WeightSpec
from .base import DecoderModel

ATTENTION_NAMES = dict(q=".q", k=".k", v=".v", o=".o", g=".g", sink=".sink", vmix=".vmix")


def build_balelorn(cfg: BalelornConfig) -> DecoderModel:
    W, eps = cfg.width, cfg.norm_eps
    routes = ops.ExpertTables()
    layers, blended = [], False
    for layer in cfg.layers:
        m = layer["mixer"]
        rot = m["rot"]
        position = RotaryEmbedding(m["dim"], rot["base"], rot["dims"]) if rot else None
        mix = None
        if m["v_mix"]:
            mix, blended = ("blend" if blended else "first"), True
        mixer = PagedAttention(W, m["heads"], m["kv_heads"], m["dim"], position, scale=m["scale"], value_dim=m["vdim"], gate=True,
                               names=ATTENTION_NAMES, chunk=m["chunk"], sink=True, value_mix=mix)
        f = layer["mlp"]
        ffn = None
        if f is not None and f["kind"] == "dense":
            ffn = GatedMLP(W, f["ff"], "gelu_tanh", names=(".gate", ".up", ".down"))
        elif f is not None:
            ffn = TableMoEMLP(W, f["ff"], f["experts"], f["top"], cfg.vocab, routes, "clamped", f["limit"])
        # (a layer without a feed-forward has no use for its norms and scale; a checkpoint may hold them all the same)
        unread = [WeightSpec(n, (W,), "norm") for n in ("norm2", "norm2b", "ls2")] if ffn is None else ()
        results = (ResultNorm(W, eps, ("norm1b", "ls1")), ResultNorm(W, eps, ("norm2b", "ls2")) if ffn is not None else None)
        layers.append(PreNormBlock(RMSNorm(W, eps, suffix=""), mixer, RMSNorm(W, eps, suffix="") if ffn is not None else None, ffn,
                                   names=("norm1", "mix", "norm2", "mlp"), gates=results, gate_names=("", ""), unread=unread))
    names = dict(embed="embed", layers="l%d", final_norm="final.norm", lm_head="head")
    return DecoderModel(cfg, TokenEmbedding(cfg.vocab, W, suffix="", norm_eps=eps), None, layers, RMSNorm(W, eps, suffix=""),
                        LMHead(cfg.vocab, W, suffix=""), None, names)


register_architecture("Balelorn", BalelornConfig, build_balelorn)
