"""Norms.  RMSNorm: y = x / sqrt(mean(x^2) + eps) * (weight_offset + w), all in 32-bit.  LayerNorm:
y = (x - m) / sqrt(mean((x - m)^2) + eps) * w + b with m = mean(x), likewise.  DynamicTanh: y = tanh(a x) * w + b, element
by element, with one stored number a.

The reference multiplies by the stored weight (llama3.rs:5244-5256), its files holding 1 + w; a
safetensors file holds w, so Gemma 2 passes weight_offset = 1.  The offset, eps and the width are
constructor arguments: another convention is another argument value.  `tensor_name` is the weight's local
name ("" where the tensor carries the part's own name).  `output_scale` is a constant factor of the norm's output
(a layer that adds s * norm(branch) to its stream): it is folded into the weight once, at load, in 32-bit, together
with the offset.  `keep_float32` keeps the weight in 32-bit whatever its file stores (the fused add-and-norm kernel
wants the two norms it meets in one dtype, so a design that scales some of its norms keeps them all so).
"""
from __future__ import annotations

from typing import Dict, Optional, Tuple

import torch

from ..hip import ops
from .base import NORMS, ParamSpec, Part, Precision


@NORMS.register("rmsnorm")
class RMSNorm(Part):
    graph_safe = True

    def __init__(self, precision: Precision, *, dim: int, eps: float, weight_offset: float = 0.0,
                 tensor_name: str = "weight", output_scale: float = 1.0, keep_float32: bool = False):
        self.tensor_name = tensor_name
        self.precision = precision
        self.dim = dim
        self.eps = float(eps)
        self.weight_offset = float(weight_offset)
        self._stored_offset = float(weight_offset)
        self.output_scale = float(output_scale)
        self.keep_float32 = bool(keep_float32) or self.output_scale != 1.0
        self.weight: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {self.tensor_name: ParamSpec((self.dim,), init_std=0.1)}

    def assign(self, name: str, tensor: torch.Tensor) -> None:
        if name != self.tensor_name:
            raise KeyError(name)
        if self.output_scale != 1.0:
            # s * (offset + w) as one 32-bit weight; the kernels then see no offset
            tensor = (tensor.float() + self._stored_offset) * self.output_scale
            self.weight_offset = 0.0
        elif self.keep_float32:
            tensor = tensor.float()
        self.weight = tensor.contiguous()

    def fused(self) -> Optional[Tuple[torch.Tensor, float, float]]:
        """(weight, eps, offset) for the fused residual-add / norm kernel; a norm that cannot take
        part in the fusion returns None and is run through `forward`."""
        return self.weight, self.eps, self.weight_offset

    def forward(self, x: torch.Tensor, out_dtype: torch.dtype, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x: float32 [T, dim]; with `rows` only these rows are normed (in their order)."""
        n = x.shape[0] if rows is None else rows.numel()
        out = torch.empty((n, self.dim), dtype=out_dtype, device=x.device)
        ops.add_norm(x, None, None, self.weight, out, eps_pre=self.eps, off_pre=self.weight_offset,
                     rows=rows, full_precision=self.precision.full)
        return out


@NORMS.register("layernorm")
class LayerNorm(Part):
    """y = (x - mean(x)) / sqrt(mean((x - mean(x))^2) + eps) * w + b.  Weight and bias (`tensor_name` and `bias_name`)
    are kept in 32-bit.  As the norm in front of a part it rides on the fused residual-add kernel (`fused_pre`); behind
    a part it runs through `forward`."""
    graph_safe = True

    def __init__(self, precision: Precision, *, dim: int, eps: float, tensor_name: str = "weight", bias_name: str = "bias"):
        self.precision = precision
        self.dim, self.eps = dim, float(eps)
        self.tensor_name, self.bias_name = tensor_name, bias_name
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {self.tensor_name: ParamSpec((self.dim,), init_std=0.1), self.bias_name: ParamSpec((self.dim,), init_std=0.1)}

    def assign(self, name: str, tensor: torch.Tensor) -> None:
        if name == self.tensor_name:
            self.weight = tensor.float().contiguous()
        elif name == self.bias_name:
            self.bias = tensor.float().contiguous()
        else:
            raise KeyError(name)

    def fused_pre(self) -> Tuple[torch.Tensor, float, float, torch.Tensor]:
        """(weight, eps, offset, bias) for the fused residual-add kernel, as the norm of the stream's new rows."""
        return self.weight, self.eps, 0.0, self.bias

    def forward(self, x: torch.Tensor, out_dtype: torch.dtype, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x: float32 [T, dim]; with `rows` only these rows are normed (in their order)."""
        n = x.shape[0] if rows is None else rows.numel()
        out = torch.empty((n, self.dim), dtype=out_dtype, device=x.device)
        ops.add_norm(x, None, None, self.weight, out, eps_pre=self.eps, b_pre=self.bias, rows=rows,
                     full_precision=self.precision.full)
        return out


@NORMS.register("dynamic_tanh")
class DynamicTanh(Part):
    """y = tanh(alpha x) * w + b: no mean, no variance, every element by itself.  Weight and bias are kept in 32-bit, the one
    number alpha (`alpha_name`, a tensor without dimensions) is read to the host once, at load.  It rides on the residual
    add behind a part and ahead of one alike (`pointwise`)."""
    graph_safe = True

    def __init__(self, precision: Precision, *, dim: int, tensor_name: str = "weight", bias_name: str = "bias", alpha_name: str = "alpha"):
        self.precision = precision
        self.dim = dim
        self.tensor_name, self.bias_name, self.alpha_name = tensor_name, bias_name, alpha_name
        self.weight: Optional[torch.Tensor] = None
        self.bias: Optional[torch.Tensor] = None
        self.alpha: Optional[float] = None

    def param_specs(self) -> Dict[str, ParamSpec]:
        return {self.tensor_name: ParamSpec((self.dim,), init_std=0.1, init_mean=1.0), self.bias_name: ParamSpec((self.dim,), init_std=0.02),
                self.alpha_name: ParamSpec((), init_std=0.05, init_mean=0.5)}

    def assign(self, name: str, tensor: torch.Tensor) -> None:
        if name == self.tensor_name:
            self.weight = tensor.float().contiguous()
        elif name == self.bias_name:
            self.bias = tensor.float().contiguous()
        elif name == self.alpha_name:
            self.alpha = float(tensor)
        else:
            raise KeyError(name)

    def pointwise(self) -> Tuple[float, torch.Tensor, torch.Tensor]:
        """(alpha, weight, bias) for the residual add whose norms act element by element."""
        return self.alpha, self.weight, self.bias

    def forward(self, x: torch.Tensor, out_dtype: torch.dtype, rows: Optional[torch.Tensor] = None) -> torch.Tensor:
        """x: float32 [T, dim]; with `rows` only these rows are normed (in their order)."""
        n = x.shape[0] if rows is None else rows.numel()
        out = torch.empty((n, self.dim), dtype=out_dtype, device=x.device)
        ops.add_dyntanh(x, None, None, self.pointwise(), out, rows=rows, full_precision=self.precision.full)
        return out
