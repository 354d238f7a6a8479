"""Several mixers side by side: each reads the same input, and the layer's result is their weighted sum.

    y = sum_b scale_b * mixer_b(h)
    y = sum_b scale_b * rms(mixer_b(h)) * gain_b         for branches with a norm of their own behind them

``branches`` names the mixers (``{name: {"kind", "params", "scale", "norm"}}``); a branch's tensors are this part's tensors
``<name>.<the branch's own name>``, the gain of its norm (``"norm": {"eps": e}``) is ``<name>.result_norm``.  The run of the
layer still owns one set of pages and one state row: at most one branch may keep pages, and where several keep a state
the row holds theirs one behind the other; each finds its own in the ``LayerCache`` it is handed.  The sum is not taken
here: the terms go on with their factors (``ScaledSum``, ``NormedSum``), and whoever adds the result into the residual adds
them one by one.

Branches that can start from a projection computed for them (``takes_projection``, ``w_in``, ``forward_projected``) have
their input products stacked into one.
"""

from __future__ import annotations

import torch

from .context import LayerCache, NormedSum, ScaledSum
from .plan import StateNeed, TensorSpec
from .registry import MIXERS, register_mixer


@register_mixer("parallel")
class ParallelMixers:
    """params: branches ({name: {"kind": mixer kind, "params": its params, "scale": its factor (default 1), "norm": {"eps"}
    or nothing}})."""

    def __init__(self, params, env):
        branches = params["branches"]
        if not branches:
            raise ValueError("mixers side by side need at least one branch")
        self.branches = [(str(name), MIXERS.get(b["kind"])(b["params"], env), float(b.get("scale", 1.0)))
                         for name, b in branches.items()]
        self.norms = {str(name): (float(b["norm"]["eps"]), int(b["params"]["hidden_size"])) for name, b in branches.items()
                      if b.get("norm")}
        if self.norms and len(self.norms) != len(self.branches):
            raise ValueError("either every mixer side by side has a norm behind it or none has")
        if sum(m.cache_need() is not None for _, m, _ in self.branches) > 1:
            raise ValueError("at most one of the mixers side by side keeps pages")
        if any(getattr(m, "kv_from_layer", None) is not None for _, m, _ in self.branches):
            raise ValueError("a mixer beside another reads no other layer's pages")
        needs = [(name, m.state_need()) for name, m, _ in self.branches if m.state_need() is not None]
        self.state_at, self.state = {}, needs[0][1] if needs else None
        if len(needs) > 1:      # one row for all of them, each behind the one before (at a multiple of 16 bytes)
            at = 0
            for name, need in needs:
                if len(need.shape) != 1 or need.dtype != "float32" or need.init != needs[0][1].init:
                    raise ValueError("mixers side by side that each keep a state keep flat rows of floats with one initial value")
                self.state_at[name] = (at, need.shape[0])
                at += need.shape[0] + (-need.shape[0]) % 4
            self.state = StateNeed((at,), "float32", needs[0][1].init)
        self.env = env
        self.gains = {}
        self.w_in, self.columns = None, {}

    takes_scaled_rows = False

    def weight_specs(self):
        specs = {f"{name}.{local}": spec for name, m, _ in self.branches for local, spec in m.weight_specs().items()}
        specs.update({f"{name}.result_norm": TensorSpec((size,), "vector") for name, (_, size) in self.norms.items()})
        return specs

    def bind(self, tensors):
        for name, m, _ in self.branches:
            m.bind({local: tensors[f"{name}.{local}"] for local in m.weight_specs()})
        self.gains = {name: tensors[f"{name}.result_norm"].float().contiguous() for name in self.norms}
        self.w_in, self.columns = None, {}
        if all(getattr(m, "takes_projection", False) for _, m, _ in self.branches):
            at = 0
            for name, m, _ in self.branches:      # every branch's own stacked matrix is a multiple of 8 rows tall
                self.columns[name] = (at, m.w_in.shape[0])
                at += m.w_in.shape[0]
            self.w_in = torch.cat([m.w_in for _, m, _ in self.branches], dim=0).contiguous()

    def cache_need(self):
        return next((m.cache_need() for _, m, _ in self.branches if m.cache_need() is not None), None)

    def state_need(self):
        return self.state

    def _own(self, name, cache):
        if name not in self.state_at:
            return cache
        at, size = self.state_at[name]
        return LayerCache(cache.k_pages, cache.v_pages, cache.block_table, cache.page_size,
                          cache.state[:, at:at + size] if cache.state is not None else None)

    def forward(self, h, ctx, cache):
        k = self.env.kernels
        proj = k.linear(h, self.w_in) if self.w_in is not None else None
        terms = []
        for name, m, scale in self.branches:
            if proj is not None:
                at, size = self.columns[name]
                y = m.forward_projected(proj[:, at:at + size], ctx, self._own(name, cache))
            else:
                y = m.forward(h, ctx, self._own(name, cache))
            terms.append((y, scale, self.gains[name], self.norms[name][0]) if self.norms else (y, scale))
        return (NormedSum if self.norms else ScaledSum)(terms, k)
