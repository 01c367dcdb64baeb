"""Plain, slow Balelorn forward pass: whole sequences, no cache, one function per mechanism.

Balelorn is a decoder whose token vectors are normed once before the first layer, and whose layers
norm a sublayer's input AND its result: ``x + s1 * n1b(mixer(n1(x)))``, then the same around the
feed-forward, with a learned vector (``s1``, ``s2``) on each result.  The token mixer is an attention
that looks no further back than the start of the chunk its position lies in, with a rotation of part
of every head, a learned sink per head in the softmax's denominator, values blended with those of the
first layer that blends, and a sigmoid gate on the concatenated heads.  The feed-forward is dense with
the tanh form of gelu, or a mixture of clamped experts that a table picks by token id.

This file shares no code with the ``spyinfer_amd`` package.  It takes a configuration as a
dictionary and the tensors as a dictionary of CPU tensors, and computes in ``dtype``
(float64 by default).
"""
import json
import math
import os

import torch


# ---- pieces ------------------------------------------------------------------------------
def rms_norm(x, w, eps):
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps) * w


def gelu_tanh(z):
    return 0.5 * z * (1.0 + torch.tanh(math.sqrt(2.0 / math.pi) * (z + 0.044715 * z ** 3)))


def dense_ff(h, gate, up, down):
    return (gelu_tanh(h @ gate.T) * (h @ up.T)) @ down.T


def clamped_expert(h, gate, up, down, limit):
    g = torch.clamp(h @ gate.T, max=limit)
    u = torch.clamp(h @ up.T, min=-limit, max=limit)
    return (g * torch.sigmoid(1.702 * g) * (u + 1.0)) @ down.T


def table_moe(h, tokens, w, mlp):
    """The experts of a token are a row of the table, each with the weight 1 / top."""
    limit = float(mlp["expert"]["limit"])
    out = torch.zeros_like(h)
    for t, token in enumerate(tokens):
        chosen = w["table"][token].tolist()
        for e in chosen:
            out[t] += clamped_expert(h[t], w["e%d.gate" % e], w["e%d.up" % e], w["e%d.down" % e], limit) / len(chosen)
    return out


def rotate_half(x, positions, base, dims):
    """x [T, n, d]: dimension i of the first ``dims`` and dimension i + dims / 2 form a pair."""
    half = dims // 2
    i = torch.arange(half, dtype=x.dtype)
    ang = positions.to(x.dtype)[:, None] * torch.pow(torch.tensor(base, dtype=x.dtype), -2.0 * i / dims)[None, :]
    cos, sin = torch.cos(ang)[:, None, :], torch.sin(ang)[:, None, :]
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * cos - v * sin, v * cos + u * sin, rest], dim=-1)


def seen(T, chunk):
    """[T, T] bool: may position i (row) look at position j (column)?  ``chunk`` None: at everything up to itself."""
    pos = torch.arange(T)
    ok = pos[None, :] <= pos[:, None]
    if chunk:
        ok = ok & (torch.div(pos[:, None], chunk, rounding_mode="floor") == torch.div(pos[None, :], chunk, rounding_mode="floor"))
    return ok


def softmax_with_sink(s, sink):
    """s [H, T, T], -inf where nothing is seen; one further term per head in the denominator that has no value."""
    m = torch.maximum(s.max(dim=-1, keepdim=True).values, sink[:, None, None])
    e = torch.exp(s - m)
    return e / (e.sum(dim=-1, keepdim=True) + torch.exp(sink[:, None, None] - m))


def blend_values(v, first, lam):
    return (1.0 - lam) * v + lam * first


def chunked_attention(h, w, m, first_values):
    """-> (result, the layer's own values before blending).  ``first_values``: those of the first layer that blends, or
    None if this layer does not blend (or is that first one)."""
    T = h.shape[0]
    H, d, dv = m["heads"], m["dim"], m["vdim"]
    G = m["kv_heads"] if m.get("kv_heads") is not None else H
    pos = torch.arange(T)
    q = (h @ w["q"].T).view(T, H, d)
    k = (h @ w["k"].T).view(T, G, d)
    own = (h @ w["v"].T).view(T, G, dv)
    if m.get("rot"):
        q = rotate_half(q, pos, float(m["rot"]["base"]), m["rot"]["dims"])
        k = rotate_half(k, pos, float(m["rot"]["base"]), m["rot"]["dims"])
    v = own if first_values is None else blend_values(own, first_values, w["vmix"])
    k = k.repeat_interleave(H // G, dim=1)
    v = v.repeat_interleave(H // G, dim=1)
    s = torch.einsum("ihd,jhd->hij", q, k) * float(m["scale"])
    s = s.masked_fill(~seen(T, m["mask"]["size"] if m.get("mask") else None), -math.inf)
    o = torch.einsum("hij,jhd->ihd", softmax_with_sink(s, w["sink"]), v).reshape(T, H * dv)
    return (o * torch.sigmoid(h @ w["g"].T)) @ w["o"].T, own


# ---- the model ---------------------------------------------------------------------------
class PlainBalelorn:
    def __init__(self, config, tensors, dtype=torch.float64):
        self.cfg = config
        self.w = {k: (v.to(dtype) if v.is_floating_point() else v) for k, v in tensors.items()}
        self.dtype = dtype

    @classmethod
    def from_folder(cls, folder, dtype=torch.float64):
        from safetensors.torch import load_file
        with open(os.path.join(folder, "config.json")) as f:
            cfg = json.load(f)
        return cls(cfg, load_file(os.path.join(folder, "model.safetensors")), dtype)

    def sub(self, prefix):
        return {k[len(prefix):]: v for k, v in self.w.items() if k.startswith(prefix)}

    def forward(self, tokens, keep_layers=None):
        """Logits [T, vocab] at every position of one sequence; ``keep_layers``: a list that gets the stream after
        every layer."""
        cfg, w, eps = self.cfg, self.w, float(self.cfg["norm"]["eps"])
        x = rms_norm(w["embed"][torch.tensor(tokens, dtype=torch.long)], w["embed.norm"], eps)
        first_values = None
        for i, layer in enumerate(cfg["layers"]):
            at = "l%d." % i
            if layer["type"] != "attention":
                raise ValueError(layer["type"])
            m = layer["mixer"]
            blends = bool(m.get("v_mix"))
            y, own = chunked_attention(rms_norm(x, w[at + "norm1"], eps), self.sub(at + "mix."), m, first_values if blends else None)
            if blends and first_values is None:
                first_values = own
            x = x + rms_norm(y, w[at + "norm1b"], eps) * w[at + "ls1"]
            mlp = layer.get("mlp")
            if mlp:
                h = rms_norm(x, w[at + "norm2"], eps)
                mw = self.sub(at + "mlp.")
                y = dense_ff(h, mw["gate"], mw["up"], mw["down"]) if mlp["kind"] == "dense" else table_moe(h, tokens, mw, mlp)
                x = x + rms_norm(y, w[at + "norm2b"], eps) * w[at + "ls2"]
            if keep_layers is not None:
                keep_layers.append(x.clone())
        return rms_norm(x, w["final.norm"], eps) @ w["head"].T

    def greedy(self, prompt, n):
        toks = list(prompt)
        for _ in range(n):
            toks.append(int(torch.argmax(self.forward(toks)[-1])))
        return toks[len(prompt):]
