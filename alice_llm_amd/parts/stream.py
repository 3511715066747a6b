"""The residual stream of a step: a float32 [tokens, width] tensor and one pending branch.

Blocks push a branch output (with the norm that applies to it before the add, if any) and ask
for the normed stream that feeds their next part.  The add of the pending branch and the next
norm run as one kernel when both norms can be fused; otherwise the same result is computed in
separate kernels.  Norms that act element by element (`pointwise`, on either side of the add) have such a kernel of
their own.  The stream itself is only ever added to, in 32-bit
(llama3.rs:14468-14470, 14555-14557).
"""
from __future__ import annotations

from typing import Optional

import torch

from ..hip import ops
from .base import FragmentActs, Precision


ADD_BRANCHES_FROM_ROWS = 256


def _fused_pre(norm):
    """(weight, eps, offset, bias or None) of a norm that the fused add-and-norm kernel can apply to the new rows, else None."""
    if norm is None:
        return None
    if hasattr(norm, "fused_pre"):
        return norm.fused_pre()
    f = norm.fused() if hasattr(norm, "fused") else None
    return None if f is None else (*f, None)


def _pointwise(norm):
    """(alpha, weight, bias) of a norm that acts element by element, else None."""
    return norm.pointwise() if norm is not None and hasattr(norm, "pointwise") else None


class ResidualStream:
    def __init__(self, x: torch.Tensor, precision: Precision):
        assert x.dtype == torch.float32 and x.dim() == 2
        self.x = x
        self.precision = precision
        self._branch: Optional[torch.Tensor] = None
        self._post = None
        self._many = None               # several pending branches [(tensor, weight, eps, offset)], added by one kernel

    def push_many(self, branches) -> None:
        """Queue `x += sum of post_norm_j(branch_j)` for [(branch, post norm or None)]: one kernel adds them all
        where every norm can be fused (and there are at most ops.MAX_BRANCHES); otherwise one push each."""
        fused = []
        for b, post in branches:
            f = post.fused() if post is not None and hasattr(post, "fused") else None
            if post is not None and f is None:
                fused = None
                break
            fused.append((b, f[0], f[1], f[2]) if f is not None else (b, None, 0.0, 0.0))
        dtypes = {w.dtype for _, w, _, _ in (fused or []) if w is not None}
        # Few rows: the single-branch kernel, one launch a branch, is as fast at 8 rows and faster at 64 (a block
        # of the fused kernel reads every branch's partial results of its row by itself); many rows: one pass
        # over the stream instead of one a branch.
        if (fused is None or len(fused) > ops.MAX_BRANCHES or len(fused) < 2 or len(dtypes) > 1
                or self.x.shape[1] > ops.ADD_BRANCHES_MAX_WIDTH or self.x.shape[0] < ADD_BRANCHES_FROM_ROWS):
            for b, post in branches:
                self.push(b, post)
            return
        self.flush()
        self._many = fused

    def _flush_many(self, out=None) -> None:
        ops.add_branches(self.x, self._many, out, full_precision=self.precision.full)
        self._many = None

    def push(self, branch: torch.Tensor, post_norm=None) -> None:
        """Queue `x += post_norm(branch)`.  branch: float32 [T, H], or [S, T, H] partial sums."""
        if self._branch is not None or self._many is not None:
            self.flush()
        self._branch = branch
        self._post = post_norm

    def _partials(self):
        b = self._branch
        return (b.shape[0], b) if b.dim() == 3 else (1, b)

    def flush(self) -> None:
        if self._many is not None:
            self._flush_many()
        if self._branch is None:
            return
        n, b = self._partials()
        post = self._post
        fused = post.fused() if post is not None and hasattr(post, "fused") else None
        if _pointwise(post) is not None:
            self._add_pointwise(None, None)
        elif post is None or fused is not None:
            w, eps, off = fused if fused is not None else (None, 0.0, 0.0)
            ops.add_norm(self.x, b, w, None, None, eps_post=eps, off_post=off, n_partials=n,
                         full_precision=self.precision.full)
        else:
            if n > 1:
                b = b.sum(dim=0)
            normed = post.forward(b.contiguous(), torch.float32)
            ops.add_norm(self.x, normed, None, None, None, full_precision=self.precision.full)
        self._branch = None
        self._post = None

    def _add_pointwise(self, norm, out, out_layout: int = ops.LAYOUT_ROW) -> None:
        """The pending add (none, or with no norm behind the branch or one that acts element by element) and norm(x), likewise."""
        n, b = self._partials() if self._branch is not None else (1, None)
        ops.add_dyntanh(self.x, b, _pointwise(self._post) if b is not None else None, _pointwise(norm), out.data if out_layout else out,
                        n_partials=n, full_precision=self.precision.full, out_layout=out_layout)
        self._branch = None
        self._post = None

    def normed(self, norm, out_dtype: Optional[torch.dtype] = None, fragments: bool = False):
        """Apply the pending add, then return norm(x) in the activation dtype (x itself if norm is None).
        fragments: the consumer reads fragment order; given where possible (see FragmentActs), else a tensor."""
        out_dtype = out_dtype or self.precision.act
        T, H = self.x.shape
        if self._many is not None:
            if norm is None:                                   # the sum and the stream's copy in the activation dtype, one kernel
                out = torch.empty((T, H), dtype=out_dtype, device=self.x.device)
                self._flush_many(out)
                return out
            self._flush_many()
        if _pointwise(norm) is not None:
            if self._branch is not None and self._post is not None and _pointwise(self._post) is None:
                self.flush()
            frag = fragments and out_dtype == torch.bfloat16 and FragmentActs.possible(self.precision, T, H)
            out = FragmentActs.empty(T, H, self.x.device) if frag else torch.empty((T, H), dtype=out_dtype, device=self.x.device)
            self._add_pointwise(norm, out, ops.LAYOUT_FRAG16 if frag else ops.LAYOUT_ROW)
            return out
        pre = _fused_pre(norm)
        if fragments and pre is not None and out_dtype == torch.bfloat16 and FragmentActs.possible(self.precision, T, H):
            post = self._post
            pf = post.fused() if post is not None and hasattr(post, "fused") else None
            if self._branch is not None and not ((post is None or pf is not None) and (pf is None or pf[0].dtype == pre[0].dtype)):
                self.flush()
            n, b = self._partials() if self._branch is not None else (1, None)
            w_post, eps_post, off_post = pf if (pf is not None and b is not None) else (None, 0.0, 0.0)
            out = FragmentActs.empty(T, H, self.x.device)
            ops.add_norm(self.x, b, w_post, pre[0], out.data, eps_post=eps_post, eps_pre=pre[1], off_post=off_post,
                         off_pre=pre[2], b_pre=pre[3], n_partials=n, full_precision=self.precision.full, out_layout=ops.LAYOUT_FRAG16)
            self._branch = None
            self._post = None
            return out
        if self._branch is not None and (norm is None or pre is not None):
            post = self._post
            pf = post.fused() if post is not None and hasattr(post, "fused") else None
            same = pf is None or pre is None or pf[0].dtype == pre[0].dtype
            if (post is None or pf is not None) and same:
                n, b = self._partials()
                out = torch.empty((T, H), dtype=out_dtype, device=self.x.device)
                w_post, eps_post, off_post = pf if pf is not None else (None, 0.0, 0.0)
                w_pre, eps_pre, off_pre, b_pre = pre if pre is not None else (None, 0.0, 0.0, None)
                ops.add_norm(self.x, b, w_post, w_pre, out, eps_post=eps_post, eps_pre=eps_pre,
                             off_post=off_post, off_pre=off_pre, b_pre=b_pre, n_partials=n,
                             full_precision=self.precision.full)
                self._branch = None
                self._post = None
                return out
        self.flush()
        if norm is None:
            return self.x.to(out_dtype)
        return norm.forward(self.x, out_dtype)

    def rows_normed(self, norm, rows: torch.Tensor, out_dtype: Optional[torch.dtype] = None, fragments: bool = False):
        """norm(x[rows]) after all pending adds: what the output head reads."""
        self.flush()
        out_dtype = out_dtype or self.precision.act
        point = _pointwise(norm)
        if fragments and point is not None and out_dtype == torch.bfloat16 and FragmentActs.possible(self.precision, rows.numel(), self.x.shape[1]):
            out = FragmentActs.empty(rows.numel(), self.x.shape[1], self.x.device)
            ops.add_dyntanh(self.x, None, None, point, out.data, rows=rows, full_precision=self.precision.full, out_layout=ops.LAYOUT_FRAG16)
            return out
        pre = _fused_pre(norm)
        if fragments and pre is not None and out_dtype == torch.bfloat16 and \
                FragmentActs.possible(self.precision, rows.numel(), self.x.shape[1]):
            out = FragmentActs.empty(rows.numel(), self.x.shape[1], self.x.device)
            ops.add_norm(self.x, None, None, pre[0], out.data, eps_pre=pre[1], off_pre=pre[2], b_pre=pre[3], rows=rows,
                         full_precision=self.precision.full, out_layout=ops.LAYOUT_FRAG16)
            return out
        if norm is None:
            return self.x.index_select(0, rows.long()).to(out_dtype)
        return norm.forward(self.x, out_dtype, rows=rows)
