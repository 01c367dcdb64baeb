"""RMS norm and layer norm.  RMS norm: y = x / sqrt(mean(x^2) + eps) * w, sums and scale in float32, eps inside the
root, the weight multiplies as it is (src/backends/cpu/x64/kernels.cpp:168-180;
src/backends/cuda/native/common.cuh:57-188).  Layer norm (the reference has none): y = (x - mean) / sqrt(var + eps) * w + b."""
from __future__ import annotations

import torch

from ..kernels import ops
from ..weights.loader import WeightSpec
from .base import Norm


class RMSNorm(Norm):
    def __init__(self, size: int, eps: float, suffix: str = ".weight", offset: float = 0.0, groups: int = 1, scalar: bool = False):
        """``groups``: the vector is cut into that many equal consecutive parts, each over its own root mean square (the
        weight still spans the whole vector).  ``suffix``: what the weight's name has behind the part's prefix (some checkpoints name the vector by the
        prefix alone).  ``offset``: the stored vector is centred on zero and multiplies as ``offset + w`` (1.0 for norms
        whose weights are stored around zero); the sum is formed once, in float32, when the weights are bound.  ``scalar``:
        the stored weight is ONE number for all coordinates (a tensor without dimensions), spread over the vector when the
        weights are bound, so that the kernels see a weight vector as ever."""
        self.size = size
        self.eps = float(eps)
        self.suffix = suffix
        self.offset = float(offset)
        self.groups = int(groups)
        self.scalar = bool(scalar)
        if self.groups <= 0 or size % self.groups:
            raise ValueError("a norm in %d groups does not fit a vector of %d" % (self.groups, size))
        self.weight = None

    def weight_specs(self, prefix):
        # (the role says how random weights are drawn: around one, or around zero where the offset supplies the one)
        return [WeightSpec(prefix + self.suffix, () if self.scalar else (self.size,), "bias" if self.offset else "norm")]

    def bind(self, prefix, weights):
        self.weight = weights[prefix + self.suffix]
        if self.scalar:
            self.weight = self.weight.reshape(1).expand(self.size).contiguous()
        if self.offset:
            self.weight = (self.weight.float() + self.offset).contiguous()

    def capturable(self, batch):
        return True

    def add_norm(self, resid, delta, out_dtype, rows=None, second=None):
        """``delta``: None, one addend, a pair of addends (the results of two sublayers that read the same norm), an
        ``ops.GatedAddend`` or ``ops.NormedAddend`` (a result behind a gate or a norm of its own), or an
        ``ops.EntryAddends`` (any of these plus an earlier state of the stream and a vector for every row).  ``second``:
        another norm of this kind that reads the same sum: the result is the pair of both outputs, from one pass."""
        if isinstance(delta, ops.NormedAddend):
            # a sublayer's result behind a norm of its own: both norms and the sum in one pass
            if second is None and self.groups == 1:
                return ops.result_norm(resid, delta.y, delta.weight, delta.eps, self.weight, self.eps, out_dtype, rows)
            delta = delta.resolve().to(out_dtype)
        more = {}
        if isinstance(delta, ops.EntryAddends):
            more = dict(base=delta.base, vec=delta.vec)
            delta = None if isinstance(delta.pending, ops.ScaledInput) else delta.pending
            if isinstance(delta, ops.GatedAddend):
                delta = delta.resolve()
            elif isinstance(delta, ops.NormedAddend):
                delta = delta.resolve().to(out_dtype)
        if second is not None:
            if (second.size, second.eps, second.groups) != (self.size, self.eps, self.groups) or second.weight.dtype != self.weight.dtype:
                raise ValueError("two norms of one sum must have one size, eps, grouping and weight dtype")
            more["weight2"] = second.weight
        if more:
            if isinstance(delta, ops.GatedAddend):
                delta = delta.resolve()
            first, other = delta if isinstance(delta, (tuple, list)) else (delta, None)
            return ops.add_rms_norm(resid, first, self.weight, self.eps, out_dtype, rows, delta2=other, groups=self.groups, **more)
        if isinstance(delta, ops.GatedAddend):
            # a sublayer's result behind its gate: formed in this kernel's pass where the dtypes allow it
            if delta.bias.dtype != self.weight.dtype or not delta.gate.is_contiguous():
                delta = delta.resolve()
            else:
                return ops.add_rms_norm(resid, delta.y, self.weight, self.eps, out_dtype, rows, groups=self.groups,
                                        gate=(delta.gate, delta.bias, delta.mult))
        if isinstance(delta, (tuple, list)):
            first, second = delta
            return ops.add_rms_norm(resid, first, self.weight, self.eps, out_dtype, rows, delta2=second, groups=self.groups)
        return ops.add_rms_norm(resid, delta, self.weight, self.eps, out_dtype, rows, groups=self.groups)

    def add_normed(self, base, y, out=None, copy_dtype=None, mix=None):
        """out = base + norm(y) in float32 (the norm on a sublayer's output; ``out`` may be ``base``); returns (out, its
        copy in ``copy_dtype`` or None).  ``mix`` = (kept results [layers, T, H], n, weights [n]) with ``out`` the n-th
        kept result: the weighted sum of the n results is formed in the same pass and returned in place of ``out``."""
        if self.groups != 1:
            raise ValueError("a norm in groups on a sublayer's output is not implemented")
        if mix is not None and mix[2].dtype != self.weight.dtype:
            out, _ = ops.norm_residual(base, y, self.weight, self.eps, out, None)
            return ops.depth_mix(mix[0], mix[1], mix[2], copy_dtype)
        return ops.norm_residual(base, y, self.weight, self.eps, out, copy_dtype, mix)

    def foldable(self, out_dtype):
        if self.groups == 1 and not self.scalar and out_dtype == torch.bfloat16 and self.weight is not None and self.weight.dtype == torch.bfloat16:
            return self.weight, self.eps
        return None


class LayerNorm(Norm):
    """y = (x - mean) / sqrt(var + eps) * w + b, var the mean of the squared deviations; float32 inside.  Tensors: the weight
    under the prefix (and ``suffix``), the bias under the same name with ``bias_suffix`` behind it."""

    takes_unsummed = True          # ``add_normed`` sums a mixture's experts or a weighted pair of results in its own pass

    def __init__(self, size: int, eps: float, suffix: str = "", bias_suffix: str = ".b"):
        self.size, self.eps, self.suffix, self.bias_suffix = size, float(eps), suffix, bias_suffix
        self.weight = self.bias = None

    def weight_specs(self, prefix):
        name = prefix + self.suffix
        return [WeightSpec(name, (self.size,), "norm"), WeightSpec(name + self.bias_suffix, (self.size,), "bias")]

    def bind(self, prefix, weights):
        name = prefix + self.suffix
        self.weight, self.bias = weights[name], weights[name + self.bias_suffix]
        if self.weight.dtype != self.bias.dtype:
            self.weight, self.bias = self.weight.float(), self.bias.float()

    def capturable(self, batch):
        return True

    def add_norm(self, resid, delta, out_dtype, rows=None):
        """The norm of the stream (at ``rows`` only, if given); ``delta`` (whatever a block may leave pending) is summed into
        it first."""
        if delta is not None and not isinstance(delta, ops.ScaledInput):
            if rows is not None:
                resid = resid.clone()                     # (picked rows: the stream stays as it is)
            if isinstance(delta, ops.EntryAddends):
                delta.resolve(resid)
            else:
                for d in (delta if isinstance(delta, (tuple, list)) else (delta,)):
                    resid.add_((d.resolve() if hasattr(d, "resolve") else d).float())
        return ops.layer_norm(resid, self.weight, self.bias, self.eps, out_dtype, rows)

    def add_normed(self, base, y, out=None, copy_dtype=None, mix=None):
        """out = base + norm(y) in float32; ``y``: rows, ``ops.ExpertRows`` or ``ops.WeightedPair``.  Returns (out, copy)."""
        if mix is not None:
            raise ValueError("a layer norm whose result is mixed with kept layer results is not implemented")
        return ops.layer_norm_residual(base, y, self.weight, self.bias, self.eps, out, copy_dtype)
