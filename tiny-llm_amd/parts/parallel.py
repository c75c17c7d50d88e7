"""Mixers side by side: every branch reads the same input, the result is the sum of the branches'
results, each times a constant of its own.

A branch is any registered mixer that takes `out_scale` (it applies the constant itself, in float32,
before its output product) and adds into the `residual` it is given: the first branch's output product
writes the sum's buffer, every further one adds to it, so the sum costs no kernel of its own.  At most one
branch may keep a paged cache, which becomes the part's own; the branches' per-request states lie side by side
in the part's state rows, and a branch is handed its own columns of them.

Where every branch says `splits_products` (its first product, `mix` and its output product by themselves), the branches'
first products are ONE product over the rows of all of them, and their output products ONE product over their operands
side by side, which forms the sum of the branches on its way.
"""
from __future__ import annotations

from typing import Dict, List, Optional, Sequence, Tuple

import torch

from ..kernels import ops
from .base import MIXERS, CacheSpec, Mixer, StateSpec, WeightSpec, register_mixer


class ParallelMixer(Mixer):
    def __init__(self, prefix, dtype, device, *, branches: Sequence[dict]):
        """branches: [{"kind": registered mixer, "name": weight-name component, "scale": constant,
        "params": the mixer's own parameters}, ...]"""
        super().__init__(prefix, dtype, device)
        if not branches:
            raise ValueError(f"{prefix}: a parallel mixer needs at least one branch")
        self.w_in = self.w_o = None
        self.branches: List[Mixer] = []
        for b in branches:
            params = dict(b.get("params") or {})
            params["out_scale"] = float(b.get("scale", 1.0))
            self.branches.append(MIXERS.get(b["kind"])(f"{prefix}.{b['name']}", dtype, device, **params))
        self.joined = all(getattr(m, "splits_products", False) for m in self.branches)
        with_cache = [m for m in self.branches if m.cache_spec() is not None]
        with_state = [m for m in self.branches if m.state_spec() is not None]
        if len(with_cache) > 1:
            raise ValueError(f"{prefix}: at most one branch may keep a cache")
        self._cache_branch = with_cache[0] if with_cache else None
        # one stateful branch: its state is the part's, whatever its shape; several: rows of one type side by side, each
        # from a multiple of four elements (16-byte rows)
        self._state_spec: Optional[StateSpec] = with_state[0].state_spec() if with_state else None
        self._state_cols: Dict[int, Optional[Tuple[int, int]]] = {id(m): None for m in with_state}
        if len(with_state) > 1:
            specs = [m.state_spec() for m in with_state]
            if any(len(s.shape) != 1 or s.dtype != specs[0].dtype for s in specs):
                raise ValueError(f"{prefix}: branches that keep states side by side keep rows of one type")
            at = 0
            for m, s in zip(with_state, specs):
                self._state_cols[id(m)] = (at, at + s.shape[0])
                at = -(-(at + s.shape[0]) // 4) * 4
            self._state_spec = StateSpec((at,), specs[0].dtype)

    @property
    def graph_safe(self) -> bool:
        parts = list(self.branches) + [getattr(m, "position", None) for m in self.branches]
        return all(p.graph_safe for p in parts if p is not None)

    def weights(self) -> List[WeightSpec]:
        return [w for m in self.branches for w in m.weights()]

    def bind(self, tensors: Dict[str, torch.Tensor]) -> None:
        for m in self.branches:
            m.bind(tensors)
        if self.joined:
            self.w_in = torch.cat([m.w_in for m in self.branches], dim=0).contiguous()
            self.w_o = torch.cat([m.w_o for m in self.branches], dim=1).contiguous()
            for m in self.branches:
                m.w_in = m.w_o = None

    def cache_spec(self) -> Optional[CacheSpec]:
        return self._cache_branch.cache_spec() if self._cache_branch is not None else None

    def state_spec(self) -> Optional[StateSpec]:
        return self._state_spec

    def _state_of(self, branch, state):
        if id(branch) not in self._state_cols:
            return None
        cols = self._state_cols[id(branch)]
        return state if cols is None else state[:, cols[0]:cols[1]]

    def forward(self, h, ctx, cache, state, residual):
        if self.joined:
            return self._forward_joined(h, ctx, cache, state, residual)
        y = residual
        for m in self.branches:
            y = m.forward(h, ctx, cache if m is self._cache_branch else None, self._state_of(m, state), y)
        return y


    def _forward_joined(self, h, ctx, cache, state, residual):
        T, dev = h.shape[0], h.device
        p = ops.linear(h, self.w_in, ops.scratch("parallel_in", (T, self.w_in.shape[0]), torch.float32, dev))
        z = ops.scratch("parallel_out", (T, self.w_o.shape[1]), self.dtype, dev)
        at_p = at_z = 0
        for m in self.branches:
            m.mix(p[:, at_p:at_p + m.in_width], ctx, cache if m is self._cache_branch else None, self._state_of(m, state),
                  z[:, at_z:at_z + m.out_width])
            at_p += m.in_width
            at_z += m.out_width
        if residual is None:
            return ops.linear(z, self.w_o, ops.scratch("sublayer_out", (T, self.w_o.shape[0]), torch.float32, dev))
        return ops.linear(z, self.w_o, residual, residual)


register_mixer("parallel", ParallelMixer)
