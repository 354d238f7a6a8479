"""Grouped-query attention over the paged cache (reference: ``ops/attention.py:70-228``,
serving form ``serving/paged_decoder.py:133-185``).

Order inside the mixer, as in the reference's serving path: project q, k, v (no
bias) -> rotate q and k by absolute position -> write k (rotated) and v into
the pages -> attend over the pages, the tokens just written included -> output
projection.  Query head ``h`` reads key/value head ``h // (Hq / Hkv)`` (reference:
``kernels/attention_kernel.py:108-251``).  Scores are ``(q . k) * scale`` with the
scale applied after the dot; key ``j`` is visible to a query at position ``p`` iff
``j <= p`` and, with a window ``w``, ``j > p - w``.

The three projections are stacked into one ``[(Hq + 2 Hkv) D, H]`` matrix at load.
A mixer whose ``kv_from_layer`` is set projects only q and reads the pages that
the named layer's latest run wrote.

Further forms, each switched on by a parameter of its own and free to combine:

* ``value_head_dim``: value heads of another width ``Dv`` than the keys'; the stacked matrix is then
  ``[Hq D + Hkv D + Hkv Dv, H]`` and the output projection takes ``Hq Dv`` columns.
* ``bias``: q, k and v have biases, added to the projections before anything else.
* ``qk_norm`` (``{"eps": e}``): every q and k head is divided by its root mean square over the head
  (``x / sqrt(mean(x^2) + e)``) and multiplied by a gain of size ``D`` that all heads share (one for q, one for k),
  after the bias and before the rotation.
* ``chunk``: the sequence's absolute positions are cut into blocks ``[b*chunk, (b+1)*chunk)``; a query attends
  causally inside its block and to nothing before the block's first position (how a prompt was fed in portions
  does not move the blocks).
* ``sink``: a learned logit per query head that competes in the softmax but carries no value: the weights of
  the real keys are ``exp(s_j) / (sum_i exp(s_i) + exp(sink_h))``, with ``sink_h`` taken as it is (``scale``
  applies to the dot products only).
* ``qk_norm`` with ``"gain": False``: the same division by the root mean square without learned gains.
* ``q_temp`` (``{"coef": c, "every": n}``): a query at position ``p`` is multiplied by
  ``1 + c * ln(floor((p + 1) / n) + 1)`` after its norm, so late queries score more sharply.
* ``out_gate``: head ``h``'s output is multiplied by ``sigmoid((G x)_h)``, a scalar for every token and head, ``G
  [Hq, H]`` reading the mixer's own input; its rows ride at the end of the stacked projection.
  ``out_gate: "element"``: every element of the heads has a gate of its own, ``sigmoid((G x)_i)`` with ``G [Hq Dv, H]``.
* ``softcap``: scores are capped softly after the scale, ``c * tanh(s / c)``.
* ``keep_first``: with a window, the sequence's first ``keep_first`` positions stay visible to every query, at their
  true positions; their pages stay with the request.
* ``value_mix``: values are mixed between layers.  The layer that ``"gives"`` leaves the values it projected to the
  step; a layer that ``"takes"`` caches ``(1 - m) v + m v_given`` of the same token, ``m`` its learned scalar (the
  layer that gives has one too and does not use it).
* ``value_from_key``: there is no value projection: a position's values are its keys as projected (with their bias,
  before norm and rotation); the stacked matrix is ``[(Hq + Hkv) D, H]``.
* ``conv_taps``: q, k and v pass a short causal convolution per channel right after the projection and its bias (before
  norm and rotation): ``c_t = sum_j w[:, j] u_(t - taps + 1 + j)``, zeros before the sequence.  The mixer then has a state
  beside its pages: the last inputs as a ring of float32 rows, that of position ``p`` in row ``p mod taps``.
* ``qk_norm`` with ``"over": "row"``: one RMS norm over all of a token's q elements (and one over all its k elements) at
  once, with gains of that size, instead of one per head.
* a rotary position encoding whose ``pairing`` is ``"interleaved"`` turns elements ``2i`` and ``2i + 1`` together.
* ``o_bias``: the output projection has a bias; it is handed on with the result (``BiasedDelta``) so that the sum
  into the residual can take it in passing.
"""

from __future__ import annotations

import torch

from .context import BiasedDelta
from .plan import PagedKVNeed, StateNeed, TensorSpec
from .registry import POSITION_ENCODINGS, register_mixer


def _shared_position_encoding(spec, env):
    kind = spec["kind"] if isinstance(spec, dict) else spec.kind
    params = spec["params"] if isinstance(spec, dict) else spec.params
    key = ("position", kind, repr(sorted(params.items(), key=lambda kv: kv[0])))
    if key not in env._shared:
        env._shared[key] = POSITION_ENCODINGS.get(kind)(params, env)
    return env._shared[key]


@register_mixer("attention")
class Attention:
    """params: hidden_size, num_heads, num_kv_heads, head_dim, position
    (``{"kind", "params"}``), and optionally window, scale, kv_from_layer, value_head_dim, bias, qk_norm, chunk,
    sink, q_temp, out_gate (True or "element"), o_bias, value_from_key, softcap, keep_first, value_mix ("gives" or
    "takes"), conv_taps."""

    def __init__(self, params, env):
        self.hidden = int(params["hidden_size"])
        self.num_heads = int(params["num_heads"])
        self.num_kv_heads = int(params["num_kv_heads"])
        self.head_dim = int(params["head_dim"])
        if self.num_heads % self.num_kv_heads:
            raise ValueError(f"num_heads {self.num_heads} is not a multiple of num_kv_heads {self.num_kv_heads}")
        self.window = params.get("window")
        if self.window is not None:
            self.window = int(self.window)
            if self.window <= 0:
                raise ValueError(f"window must be positive, got {self.window}")
        scale = params.get("scale")
        self.scale = float(scale) if scale is not None else 1.0 / (self.head_dim ** 0.5)
        self.kv_from_layer = params.get("kv_from_layer")
        self.value_dim = int(params.get("value_head_dim") or self.head_dim)
        self.bias = bool(params.get("bias", False))
        qk_norm = params.get("qk_norm")
        self.qk_norm_eps = float(qk_norm["eps"]) if qk_norm else None
        self.qk_norm_gain = bool(qk_norm.get("gain", True)) if qk_norm else False
        self.qk_norm_over = str(qk_norm.get("over", "head")) if qk_norm else None
        if self.qk_norm_over not in (None, "head", "row"):
            raise ValueError(f"a q/k norm is over a head or over the row, not {self.qk_norm_over!r}")
        self.conv_taps = int(params["conv_taps"]) if params.get("conv_taps") is not None else None
        if self.conv_taps is not None and self.conv_taps < 1:
            raise ValueError(f"a convolution has a tap or more, got {self.conv_taps}")
        q_temp = params.get("q_temp")
        self.q_temp = (float(q_temp["coef"]), int(q_temp["every"])) if q_temp else None
        if self.q_temp is not None and self.q_temp[1] <= 0:
            raise ValueError(f"q_temp.every must be positive, got {self.q_temp[1]}")
        out_gate = params.get("out_gate") or False
        if out_gate not in (False, True, "element"):
            raise ValueError(f"out_gate is True (a gate a head) or 'element', got {out_gate!r}")
        self.out_gate = bool(out_gate)
        self.element_gate = out_gate == "element"
        self.softcap = float(params["softcap"]) if params.get("softcap") else None
        if self.softcap is not None and not self.softcap > 0:
            raise ValueError(f"a soft cap must be positive, got {self.softcap}")
        self.keep_first = int(params.get("keep_first") or 0)
        if self.keep_first < 0 or (self.keep_first and params.get("chunk") is not None):
            raise ValueError(f"keep_first is a count of first positions behind a window, got {self.keep_first}")
        if self.window is None:
            self.keep_first = 0        # every position is visible anyway
        self.value_mix = params.get("value_mix")
        if self.value_mix not in (None, "gives", "takes"):
            raise ValueError(f"value_mix is 'gives' or 'takes', got {self.value_mix!r}")
        self.o_bias = bool(params.get("o_bias", False))
        self.value_from_key = bool(params.get("value_from_key", False))
        if self.value_from_key and (self.value_dim != self.head_dim or params.get("kv_from_layer") is not None):
            raise ValueError("values that are the keys have the keys' width, and the mixer projects its own keys")
        self.chunk = params.get("chunk")
        if self.chunk is not None:
            self.chunk = int(self.chunk)
            if self.chunk <= 0:
                raise ValueError(f"chunk must be positive, got {self.chunk}")
        self.sink = bool(params.get("sink", False))
        if self.kv_from_layer is not None and (self.bias or self.qk_norm_eps is not None or self.value_dim != self.head_dim
                                               or self.out_gate or self.q_temp is not None or self.value_mix):
            raise ValueError("a mixer that reads another layer's keys and values has plain q heads of the keys' width")
        self.position = _shared_position_encoding(params.get("position", {"kind": "none", "params": {}}), env)
        if self.position.rotary_dim > self.head_dim:
            raise ValueError(f"rotary_dim {self.position.rotary_dim} exceeds head_dim {self.head_dim}")
        self.pairing = getattr(self.position, "pairing", "half")
        if self.row_form and (self.kv_from_layer is not None or self.q_temp is not None or self.out_gate or self.value_mix
                              or self.value_from_key or (self.qk_norm_eps is not None and not self.qk_norm_gain)):
            raise ValueError("convolved, row-normed or neighbour-rotated heads do not combine with a query temperature, an "
                             "output gate, mixed values, values that are keys, or another layer's pages")
        check = getattr(env.kernels, "check_attention_geometry", None)
        if check is not None:     # sizes the kernels refuse are refused here, when the model is built
            check(self.num_heads, self.num_kv_heads, max(self.head_dim, self.value_dim))
        check = getattr(env.kernels, "check_row_prepare", None)
        if check is not None and self.row_form:
            check(self.num_heads, self.num_kv_heads, self.head_dim, self.conv_taps or 1)
        # kernels that want keys and values of one width say at which width this mixer should keep its pages
        page_dim = getattr(env.kernels, "attention_page_dim", None)
        self.page_dim = page_dim(self.head_dim, self.value_dim, env.dtype) if page_dim is not None and self._options() else None
        self.env = env
        self.w_qkv = None
        self.w_o = None
        self.b_qkv = self.q_gain = self.k_gain = self.sinks = self.b_o = None
        self.gate_columns = 0
        self.mix = self.conv_w = None
        self.row_columns = ()

    @property
    def row_form(self) -> bool:
        """Whether what lies between projection and attention needs a token's whole row at once (the kernels'
        ``row_prepare``)."""
        return (self.conv_taps is not None or self.qk_norm_over == "row"
                or (self.position.rotary_dim > 0 and self.pairing == "interleaved"))

    @property
    def takes_projection(self) -> bool:
        """Whether ``forward_projected`` may be handed the rows of ``w_in``'s product."""
        return self.row_form

    @property
    def w_in(self):
        return self.w_qkv

    takes_scaled_rows = True   # the input goes to ``qkv_to_cache`` only

    @property
    def writes_kv(self) -> bool:
        return self.kv_from_layer is None

    @property
    def gates(self) -> int:
        """Gates a token has on the heads' outputs."""
        return self.num_heads * self.value_dim if self.element_gate else self.num_heads

    def weight_specs(self):
        q = self.num_heads * self.head_dim
        kv = self.num_kv_heads * self.head_dim
        v = self.num_kv_heads * self.value_dim
        specs = {"q": TensorSpec((q, self.hidden)), "o": TensorSpec((self.hidden, self.num_heads * self.value_dim))}
        if self.writes_kv:
            specs["k"] = TensorSpec((kv, self.hidden))
            if not self.value_from_key:
                specs["v"] = TensorSpec((v, self.hidden))
        if self.bias:
            specs.update({"q_bias": TensorSpec((q,), "vector"), "k_bias": TensorSpec((kv,), "vector")})
            if not self.value_from_key:
                specs["v_bias"] = TensorSpec((v,), "vector")
        if self.qk_norm_eps is not None and self.qk_norm_gain:
            sizes = (q, kv) if self.qk_norm_over == "row" else (self.head_dim, self.head_dim)
            specs.update({"q_norm": TensorSpec((sizes[0],), "vector"), "k_norm": TensorSpec((sizes[1],), "vector")})
        if self.conv_taps is not None:
            specs.update({"q_conv": TensorSpec((q, self.conv_taps), "vector"), "k_conv": TensorSpec((kv, self.conv_taps), "vector"),
                          "v_conv": TensorSpec((v, self.conv_taps), "vector")})
        if self.sink:
            specs["sink"] = TensorSpec((self.num_heads,), "vector")
        if self.out_gate:
            specs["gate"] = TensorSpec((self.gates, self.hidden))
        if self.value_mix:
            specs["value_mix"] = TensorSpec((), "vector")
        if self.o_bias:
            specs["o_bias"] = TensorSpec((self.hidden,), "vector")
        return specs

    def bind(self, tensors):
        stacked = [tensors["q"]]
        if self.writes_kv:
            stacked += [tensors["k"]] if self.value_from_key else [tensors["k"], tensors["v"]]
        if self.out_gate:   # the gate's rows behind v, filled up with zero rows so that a projected row stays aligned
            self.gate_columns = -(-self.gates // 8) * 8
            g = tensors["gate"]
            stacked += [g, g.new_zeros((self.gate_columns - self.gates, self.hidden))]
        if self.value_mix == "takes":
            self.mix = tensors["value_mix"].reshape(1).float().contiguous()
        if self.row_form:     # q, k and v each start aligned in a projected row, behind zero rows
            at, columns, parts = 0, [], []
            for t in stacked:
                columns.append(at)
                parts += [t, t.new_zeros((-t.shape[0] % 8, self.hidden))]
                at += t.shape[0] + (-t.shape[0] % 8)
            self.row_columns, stacked = tuple(columns), parts
        self.w_qkv = torch.cat(stacked, dim=0).contiguous()
        if self.conv_taps is not None:
            self.conv_w = torch.cat([tensors[n] for n in ("q_conv", "k_conv", "v_conv")], dim=0).float().t().contiguous()   # [taps, channels]
        self.w_o = tensors["o"].contiguous()
        if self.page_dim is not None and not self.element_gate:
            # the attention's rows come with page_dim elements a head: zero columns for the rest (the elements' gate
            # leaves the heads' own elements only)
            wide = self.w_o.new_zeros((self.hidden, self.num_heads, self.page_dim))
            wide[:, :, :self.value_dim] = self.w_o.view(self.hidden, self.num_heads, self.value_dim)
            self.w_o = wide.view(self.hidden, self.num_heads * self.page_dim)
        if self.bias:
            self.b_qkv = torch.cat([tensors[n] for n in ("q_bias", "k_bias", "v_bias") if n in tensors]).contiguous()
        if self.qk_norm_eps is not None and self.qk_norm_gain:
            self.q_gain, self.k_gain = tensors["q_norm"].contiguous(), tensors["k_norm"].contiguous()
        elif self.qk_norm_eps is not None:
            self.q_gain = self.k_gain = torch.ones(self.head_dim, dtype=torch.float32, device=self.w_qkv.device)
        if self.o_bias:
            self.b_o = tensors["o_bias"].contiguous()
        if self.sink:
            self.sinks = tensors["sink"].contiguous()
        prepare = getattr(self.env.kernels, "prepare_pending_weight", None)
        if prepare is not None:   # the kernels may keep a copy of their own of a weight whose product is left pending
            prepare(self.w_o)

    def plain_form(self):
        """What this mixer is, as plain data, for kernels that can run a whole block in one call; None for the forms
        that only ``forward`` covers (reading another layer's keys and values)."""
        if not self.writes_kv or type(self).forward is not Attention.forward or self._options():
            return None     # a subclass with a forward of its own is no longer what this form describes
        cos, sin = self.position.tables()
        return {"kind": "paged_attention", "w_qkv": self.w_qkv, "w_o": self.w_o, "hidden": self.hidden,
                "n_heads": self.num_heads, "n_kv_heads": self.num_kv_heads, "head_dim": self.head_dim,
                "rotary_dim": self.position.rotary_dim, "cos": cos, "sin": sin, "scale": self.scale,
                "window": self.window}

    def _options(self) -> bool:
        """Whether any of the further forms is switched on (the kernels then get them as keyword arguments)."""
        return (self.bias or self.qk_norm_eps is not None or self.sink or self.chunk is not None
                or self.value_dim != self.head_dim or self.q_temp is not None or self.out_gate or self.value_from_key
                or self.softcap is not None or self.keep_first > 0 or self.value_mix is not None or self.row_form)

    def cache_need(self):
        if self.page_dim is not None:
            return PagedKVNeed(self.num_kv_heads, self.page_dim, self.window, None, self.chunk, self.keep_first)
        return PagedKVNeed(self.num_kv_heads, self.head_dim, self.window,
                           self.value_dim if self.value_dim != self.head_dim else None, self.chunk, self.keep_first)

    def state_need(self):
        if self.conv_taps is None or self.conv_taps == 1:
            return None
        channels = (self.num_heads + self.num_kv_heads) * self.head_dim + self.num_kv_heads * self.value_dim
        return StateNeed((self.conv_taps * channels,), "float32", 0.0)

    def forward_projected(self, proj, ctx, cache):
        """The mixer from the rows of the stacked projection on (``[q | k | v]`` at ``row_columns``, perhaps columns of a
        wider matrix)."""
        k = self.env.kernels
        cos, sin = self.position.tables()
        norm = (self.q_gain, self.k_gain, self.qk_norm_eps, self.qk_norm_over) if self.qk_norm_eps is not None else None
        q = k.row_prepare(proj, self.row_columns, self.num_heads, self.num_kv_heads, self.head_dim, self.value_dim,
                          self.position.rotary_dim, cos, sin, self.pairing, self.b_qkv, self.conv_w, norm, self.page_dim,
                          ctx, cache)
        attend = {}
        if self.value_dim != self.head_dim and self.page_dim is None:
            attend["value_dim"] = self.value_dim
        for name, value in (("chunk", self.chunk), ("sinks", self.sinks), ("softcap", self.softcap)):
            if value is not None:
                attend[name] = value
        if self.keep_first:
            attend["keep_first"] = self.keep_first
        out = k.paged_attention(q, self.num_heads, self.num_kv_heads, self.page_dim or self.head_dim, self.scale,
                                self.window, ctx, cache, **attend)
        y = k.pending_linear(out, self.w_o)
        return BiasedDelta(y, self.b_o, k) if self.o_bias else y

    def forward(self, h, ctx, cache):
        k = self.env.kernels
        if self.row_form:
            return self.forward_projected(k.linear(h, self.w_qkv), ctx, cache)
        cos, sin = self.position.tables()
        project, attend = {}, {}
        if self._options():   # only then: a kernels object that knows none of these forms serves the plain mixer
            if self.value_dim != self.head_dim:
                project["value_dim"] = self.value_dim
                if self.page_dim is None:
                    attend["value_dim"] = self.value_dim
            if self.page_dim is not None:
                project["page_dim"] = self.page_dim
            if self.bias:
                project["bias"] = self.b_qkv
            if self.qk_norm_eps is not None:
                project["qk_norm"] = (self.q_gain, self.k_gain, self.qk_norm_eps)
            if self.chunk is not None:
                attend["chunk"] = self.chunk
            if self.sink:
                attend["sinks"] = self.sinks
            if self.q_temp is not None:
                project["q_temp"] = self.q_temp
            if self.out_gate:
                project["extra_columns"] = self.gate_columns
            if self.value_from_key:
                project["values_are_keys"] = True
            if self.softcap is not None:
                attend["softcap"] = self.softcap
            if self.keep_first:
                attend["keep_first"] = self.keep_first
            if self.value_mix == "gives":
                project["give_values"] = True
            elif self.value_mix == "takes":
                project["value_mix"] = (ctx.shared["given_values"], self.mix)
        qkv = k.qkv_to_cache(
            h, self.w_qkv, self.num_heads, self.num_kv_heads if self.writes_kv else 0, self.head_dim,
            self.position.rotary_dim, cos, sin, ctx, cache, **project)
        gate_logits = None
        if self.value_mix == "gives":
            *qkv, ctx.shared["given_values"] = qkv
            qkv = qkv if self.out_gate else qkv[0]
        if self.out_gate:
            qkv, further = qkv
            gate_logits = further[:, :self.gates]
        out = k.paged_attention(
            qkv, self.num_heads, self.num_kv_heads, self.page_dim or self.head_dim, self.scale, self.window, ctx, cache,
            **attend)
        if gate_logits is not None:
            out = (k.element_gate(out, gate_logits, self.num_heads) if self.element_gate
                   else k.head_gate(out, gate_logits, self.num_heads))
        y = k.pending_linear(out, self.w_o)   # the norm after it may have it added into the residual
        return BiasedDelta(y, self.b_o, k) if self.o_bias else y
