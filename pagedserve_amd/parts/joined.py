"""Two mixers that read the same input and whose results are added."""

import torch

from ..ops import kernels
from ..weights.loader import MATRIX, ParamSpec
from .base import Mixer, packed_projection, site_memo
from .registry import MIXERS, build_part, register_mixer


@register_mixer("joined")
class JoinedMixers(Mixer):
    """``out = left(x) + right(x)`` as two products for both: one packed product ``[left | right]`` of the input, the
    two mixers' own work on their columns of it, and one product over ``[left | right]`` columns with the output
    matrices side by side, so that their sum is made inside it.

    ``left`` and ``right`` are ``PartSpec`` records of mixers that work between two products (``CoreMixer``, or
    attention that prepares its heads); a factor on a result is the child's own (``out_scale``).  Each child keeps
    a cache entry of its own kind (``cache_spec`` is the pair); its parameters live under ``left.`` / ``right.``.
    ``ride``: see ``CoreMixer``."""

    accepts_pending_norm = True

    def __init__(self, width: int, dtype, left, right, ride: int = 0):
        self.width = width
        self.dtype = dtype
        self.left = build_part(MIXERS, "mixer (left)", left, width=width, dtype=dtype)
        self.right = build_part(MIXERS, "mixer (right)", right, width=width, dtype=dtype)
        self.children = (("left", self.left), ("right", self.right))
        for name, child in self.children:
            if not hasattr(child, "core"):
                raise ValueError(f"the {name} mixer does not work between two products of the caller")
        self.ride = int(ride)
        self._memo_in, self._memo_out = {}, {}

    @property
    def graph_safe(self):
        return all(getattr(child, "graph_safe", False) for _, child in self.children)

    @property
    def query_tile(self):
        sizes = set()
        for _, child in self.children:
            asked = getattr(child, "query_tile", None)
            if asked:
                sizes.update(asked if isinstance(asked, (tuple, list)) else (asked,))
        return tuple(sorted(sizes))

    def set_position(self, position):
        self.position = position
        for _, child in self.children:
            child.set_position(position)

    def parameters(self):
        rows = self.left.core_rows + self.right.core_rows + self.ride
        params = {
            "in.weight": ParamSpec((rows, self.width), MATRIX),
            "out.weight": ParamSpec((self.width, self.left.stored_columns + self.right.stored_columns), MATRIX),
        }
        for prefix, child in self.children:
            for name, spec in child.core_parameters().items():
                params[f"{prefix}.{name}"] = spec
        return params

    def bind(self, tensors):
        self.in_weight = tensors["in.weight"]
        stored = tensors["out.weight"]
        cut = self.left.stored_columns
        self.out_weight = torch.cat([self.left.pad_out(stored[:, :cut]), self.right.pad_out(stored[:, cut:])],
                                    dim=1).contiguous()
        for prefix, child in self.children:
            child.bind_core({name: tensors[f"{prefix}.{name}"] for name in child.core_parameters()},
                            self.in_weight.device)
        self.in_packed = kernels.pack_decode_weight(self.in_weight)
        self.out_packed = kernels.pack_decode_weight(self.out_weight)
        self._memo_in.clear()
        self._memo_out.clear()

    def cache_spec(self):
        return tuple(child.cache_spec() for _, child in self.children)

    def forward(self, x, residual, ctx, cache):
        tokens, workspace = ctx.tokens, ctx.workspace
        left, right = self.left, self.right
        core_rows = left.core_rows + right.core_rows
        proj, ridden = packed_projection(workspace, core_rows, self.ride, tokens)
        kernels.linear(x, self.in_weight, None, proj, packed=self.in_packed,
                       memo=site_memo(self._memo_in, workspace), shared=ctx.shared_calls)
        columns = left.core_columns + right.core_columns
        # (rows of the buffer begin at multiples of 16 bytes whatever the columns are)
        _, both, _ = workspace.column_views("core_out", -(-columns // 8) * 8, self.dtype, tokens,
                                            (columns, -columns % 8))
        left.core(proj, 0, both[:, :left.core_columns], ctx, cache.children[0])
        right.core(proj, left.core_rows, both[:, left.core_columns:], ctx, cache.children[1])
        kernels.linear(both, self.out_weight, None, residual, epilogue="residual", packed=self.out_packed,
                       memo=site_memo(self._memo_out, workspace), shared=ctx.shared_calls)
        return ridden if self.ride else None
