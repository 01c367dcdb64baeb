"""Plain, slow Nolatar forward pass: whole sequences, no cache, one function per mechanism.

Nolatar is a decoder whose sublayers read the stream itself and whose layers add a layer norm (with a
bias) of what a sublayer returns: ``x + n1(mixer(x))``, then ``x + n2(ff(x))``.  Token mixers: a
state-space recurrence with a gate ahead of its grouped norm, a differential attention (two softmax maps
per head over the same values, one subtracted from the other; some layers read an earlier layer's keys
and values), and an attention in chunks beside a retention, their results weighted with two constants.
The feed-forward is a mixture of ungated experts plus an expert for every token.

This file shares no code with the ``spyinfer_amd`` package.  It takes a configuration as a
dictionary and the tensors as a dictionary of CPU tensors, and computes in ``dtype``
(float64 by default).
"""
import json
import math
import os

import torch


# ---- pieces ------------------------------------------------------------------------------
def layer_norm(x, w, b, eps):
    c = x - x.mean(dim=-1, keepdim=True)
    return c / torch.sqrt((c * c).mean(dim=-1, keepdim=True) + eps) * w + b


def over_rms(x, eps):
    """The last dimension over its root mean square."""
    return x / torch.sqrt((x * x).mean(dim=-1, keepdim=True) + eps)


def silu(z):
    return z * torch.sigmoid(z)


def gelu(z):
    return 0.5 * z * (1.0 + torch.erf(z / math.sqrt(2.0)))


def ungated_ff(h, up, down):
    return gelu(h @ up.T) @ down.T


def mixture(h, w, mlp):
    """The ``top`` experts with the largest logits, weighted with the softmax over those logits alone, plus the
    expert of every token."""
    top = mlp["router"]["top"]
    out = torch.zeros_like(h)
    logits = h @ w["router"].T
    for t in range(h.shape[0]):
        best = torch.topk(logits[t], top)
        weights = torch.softmax(best.values, dim=0)
        for e, a in zip(best.indices.tolist(), weights):
            out[t] += a * ungated_ff(h[t], w["e%d.up" % e], w["e%d.down" % e])
    if mlp.get("shared"):
        out = out + ungated_ff(h, w["shared.up"], w["shared.down"])
    return out


def angles(positions, base, dims, dtype):
    i = torch.arange(dims // 2, dtype=dtype)
    return positions.to(dtype)[:, None] * torch.pow(torch.tensor(base, dtype=dtype), -2.0 * i / dims)[None, :]


def rotate_half(x, positions, base, dims):
    """x [T, ..., d]: dimension i of the first ``dims`` and dimension i + dims / 2 form a pair."""
    half = dims // 2
    ang = angles(positions, base, dims, x.dtype).view((x.shape[0],) + (1,) * (x.dim() - 2) + (half,))
    u, v, rest = x[..., :half], x[..., half:dims], x[..., dims:]
    return torch.cat([u * torch.cos(ang) - v * torch.sin(ang), v * torch.cos(ang) + u * torch.sin(ang), rest], dim=-1)


def rotate_pairs(x, positions, base, dims):
    """x [T, ..., d]: dimensions 2 i and 2 i + 1 of the first ``dims`` form a pair."""
    ang = angles(positions, base, dims, x.dtype).view((x.shape[0],) + (1,) * (x.dim() - 2) + (dims // 2,))
    u, v, rest = x[..., 0:dims:2], x[..., 1:dims:2], x[..., dims:]
    turned = torch.stack([u * torch.cos(ang) - v * torch.sin(ang), v * torch.cos(ang) + u * torch.sin(ang)], dim=-1)
    return torch.cat([turned.flatten(-2), rest], dim=-1)


def seen(T, chunk):
    """[T, T] bool: may position i (row) look at position j (column)?  ``chunk`` None: at everything up to itself."""
    pos = torch.arange(T)
    ok = pos[None, :] <= pos[:, None]
    if chunk:
        ok = ok & (torch.div(pos[:, None], chunk, rounding_mode="floor") == torch.div(pos[None, :], chunk, rounding_mode="floor"))
    return ok


def attend(q, k, v, scale, chunk=None):
    """q [T, H, d], k [T, G, d], v [T, G, dv] -> [T, H, dv]; query head h reads key head h // (H / G)."""
    T, H = q.shape[:2]
    k, v = (x.repeat_interleave(H // x.shape[1], dim=1) for x in (k, v))
    s = torch.einsum("ihd,jhd->hij", q, k) * scale
    s = s.masked_fill(~seen(T, chunk), -math.inf)
    return torch.einsum("hij,jhd->ihd", torch.softmax(s, dim=-1), v)


def chunked_attention(h, w, m, eps):
    T, H, d = h.shape[0], m["heads"], m["dim"]
    G = m["kv_heads"]
    pos = torch.arange(T)
    q = over_rms((h @ w["q"].T).view(T, H, d), eps) * w["q.norm"]
    k = over_rms((h @ w["k"].T).view(T, G, d), eps) * w["k.norm"]
    v = (h @ w["v"].T).view(T, G, m["vdim"])
    base, dims = float(m["rot"]["base"]), m["rot"]["dims"]
    o = attend(rotate_half(q, pos, base, dims), rotate_half(k, pos, base, dims), v, float(m["scale"]), m["mask"]["size"])
    return o.reshape(T, -1) @ w["o"].T


def lambda_of(w, diff):
    return torch.exp((w["lq1"] * w["lk1"]).sum()) - torch.exp((w["lq2"] * w["lk2"]).sum()) + diff


def differential_attention(h, w, m, eps, other=None):
    """-> (result, (keys, values) as the layer's cache holds them).  ``other``: the keys and values of the layer that this
    one reads (None: its own)."""
    T, H, G, d = h.shape[0], m["heads"], m["kv_heads"], m["dim"]
    pos = torch.arange(T)
    base, dims, diff = float(m["rot"]["base"]), m["rot"]["dims"], float(m["diff"])
    q = rotate_pairs(over_rms((h @ w["q"].T).view(T, H, 2, d), eps) * w["q.norm"], pos, base, dims)
    if other is None:
        k = rotate_pairs(over_rms((h @ w["k"].T).view(T, G, 2, d), eps) * w["k.norm"], pos, base, dims)
        v = (h @ w["v"].T).view(T, G, m["vdim"])
    else:
        k, v = other
    a1, a2 = (attend(q[:, :, i], k[:, :, i], v, float(m["scale"])) for i in range(2))
    o = over_rms(a1 - lambda_of(w, diff) * a2, eps) * (1.0 - diff)
    return o.reshape(T, -1) @ w["o"].T, (k, v)


def retention(h, w, m, eps):
    T, H, d, dv = h.shape[0], m["heads"], m["dim"], m["vdim"]
    pos = torch.arange(T)
    base, dims = float(m["rot"]["base"]), m["rot"]["dims"]
    q = rotate_half((h @ w["q"].T).view(T, H, d), pos, base, dims)
    k = rotate_half((h @ w["k"].T).view(T, H, d), pos, base, dims) * d ** -0.5
    v = (h @ w["v"].T).view(T, H, dv)
    decay = torch.tensor([float(x) for x in m["decay"]], dtype=h.dtype)
    S = torch.zeros((H, d, dv), dtype=h.dtype)
    out = torch.zeros((T, H, dv), dtype=h.dtype)
    for t in range(T):
        S = decay[:, None, None] * S + k[t][:, :, None] * v[t][:, None, :]
        out[t] = torch.einsum("hij,hi->hj", S, q[t])
    return (over_rms(out, eps).reshape(T, H * dv) * silu(h @ w["g"].T)) @ w["o"].T


def side_by_side(h, w, m, eps):
    left = {k[len("left."):]: v for k, v in w.items() if k.startswith("left.")}
    right = {k[len("right."):]: v for k, v in w.items() if k.startswith("right.")}
    return float(m["left_scale"]) * chunked_attention(h, left, m["left"], eps) + float(m["right_scale"]) * retention(h, right, m["right"], eps)


def causal_conv(x, taps, bias):
    """x [T, C], taps [C, n]: the last column is the current token's."""
    T, n = x.shape[0], taps.shape[1]
    padded = torch.cat([torch.zeros((n - 1, x.shape[1]), dtype=x.dtype), x], dim=0)
    return sum(padded[j:j + T] * taps[:, j] for j in range(n)) + bias


def state_space(h, w, m, eps):
    T, H, dv, N, G = h.shape[0], m["heads"], m["vdim"], m["state"], m["groups"]
    inner = H * dv
    z, xbc, dt = torch.split(h @ w["in"].T, [inner, inner + 2 * G * N, H], dim=1)
    xbc = silu(causal_conv(xbc, w["conv"], w["conv.b"]))
    x = xbc[:, :inner].view(T, H, dv)
    B = xbc[:, inner:inner + G * N].view(T, G, N).repeat_interleave(H // G, dim=1)
    C = xbc[:, inner + G * N:].view(T, G, N).repeat_interleave(H // G, dim=1)
    dt = torch.nn.functional.softplus(dt + w["dt_bias"], threshold=1e9)
    decay = torch.exp(-torch.exp(w["A_log"]) * dt)
    S = torch.zeros((H, N, dv), dtype=h.dtype)
    y = torch.zeros((T, H, dv), dtype=h.dtype)
    for t in range(T):
        S = decay[t][:, None, None] * S + dt[t][:, None, None] * B[t][:, :, None] * x[t][:, None, :]
        y[t] = torch.einsum("hij,hi->hj", S, C[t]) + w["D"][:, None] * x[t]
    return grouped_gated_norm(y.reshape(T, inner), z, w["norm"], m["norm_groups"], eps) @ w["o"].T


def grouped_gated_norm(y, z, weight, groups, eps):
    y = y * silu(z)
    return over_rms(y.view(y.shape[0], groups, -1), eps).reshape(y.shape) * weight


# ---- the model ---------------------------------------------------------------------------
class PlainNolatar:
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
        x = w["embed"][torch.tensor(tokens, dtype=torch.long)]
        cached = {}
        for i, layer in enumerate(cfg["layers"]):
            at, m = "l%d." % i, layer["mixer"]
            mw = self.sub(at + "mix.")
            if layer["type"] == "mamba2":
                y = state_space(x, mw, m, eps)
            elif layer["type"] == "parallel":
                y = side_by_side(x, mw, m, eps)
            elif layer["type"] == "attention":
                y, cached[i] = differential_attention(x, mw, m, eps, cached[m["kv_from"]] if m.get("kv_from") is not None else None)
            else:
                raise ValueError(layer["type"])
            x = x + layer_norm(y, w[at + "norm1"], w[at + "norm1.b"], eps)
            if layer.get("mlp"):
                x = x + layer_norm(mixture(x, self.sub(at + "mlp."), layer["mlp"]), w[at + "norm2"], w[at + "norm2.b"], eps)
            if keep_layers is not None:
                keep_layers.append(x.clone())
        return layer_norm(x, w["final.norm"], w["final.norm.b"], eps) @ w["head"].T

    def greedy(self, prompt, n):
        toks = list(prompt)
        for _ in range(n):
            toks.append(int(torch.argmax(self.forward(toks)[-1])))
        return toks[len(prompt):]
