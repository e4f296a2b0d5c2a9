"""Grouped-query softmax attention from one product's float32 sums, with the variations a design may ask for.

One product computes everything that reads the mixer's input: queries, keys, values (unless the values are the
keys as projected, ``values_from_keys``) and, with ``head_gate``, one gate number a query head.  From its float32
sums one kernel makes what attention reads (KernelBackend.qkv_finish): an optional RMS norm over the whole query
(key) projection with a weight of that size (``qk_norm``), the rotation of the first ``position.rotary_dim`` numbers
of every head by angles computed in 32-bit (``position``: RotaryInterleaved or RotaryHalfAngles), an optional
temperature a query head (``head_temperature``: a checkpoint vector that multiplies the head's scores), and the
key and value rows of the cache.  Attention: scores * scale over the last ``window`` keys (None: all earlier
keys), softmax in 32-bit, with ``sink`` (a number) one more term exp(sink) in every denominator that has no value.
Head h's output is multiplied by sigmoid(gate_h) (``head_gate``) and the heads go through the output projection.
With ``bias`` the query, key and value projections have biases.  ``position_temperature`` = (coef, every): the query at
position p is multiplied by 1 + coef * ln(floor((p + 1) / every) + 1).  ``distance_bias`` = (buckets, farthest): a
checkpoint table [buckets, heads] adds table[bucket(n), h] to head h's score of a key n positions back (after the
scale): one bucket a distance for n < buckets / 2, then buckets whose reach grows geometrically,
bucket(n) = min(buckets - 1, half + floor(ln(n / half) / ln(farthest / half) * (buckets - half))), half = buckets / 2.
The table is spread over distances once, when the weights are loaded ([heads, N], N the first distance of the last
bucket + 1: every key further back adds the last entry).

``conv`` (taps K): every channel of the three projections first passes a causal convolution over time,
y_t = sum_j w[:, j] u_(t - K + 1 + j), inputs before a request's first token zero; the request's last K - 1 projected values
are kept beside its keys and values (cache members ``kv`` and ``conv``).  ``qk_norm`` "head": the norm is taken head by head
over the head's numbers, with one weight of that size for all heads.  ``keep_first``: beside the window a query also sees
the request's first so many keys.  ``sink`` "head": the sink is a checkpoint number per query head.  ``element_gate``: the
concatenated heads are multiplied number by number with sigmoid(W_g h).  ``share_values`` / ``take_values`` (a name): the
layer leaves its values in ``step.shared`` for later layers of the step / caches (1 - lambda) v + lambda v_shared instead of
its own values v, lambda a checkpoint number (the layer that leaves them has one too, which nothing reads).

``qk_norm`` "turned": queries and keys are divided head by head by their root mean square after the rotation, without
weights.  ``chunk``: a query sees the earlier keys of its own chunk only, floor(i / chunk) = floor(j / chunk), chunks counted
from the request's first position (pages that lie wholly before the chunk of a request's next token are given back: the cache
sees the chunk as a window of that many keys, which no chunk exceeds).  ``out_bias``: the output projection has a bias.

Keys and queries of ``dim`` and values of ``vdim`` numbers a head are kept in a cache of P = the next multiple of
16 of the larger one, zeros beyond their own size, so that every head size runs the same attention kernels; the
output projection's columns are spread to match when the weights are loaded.
"""
from __future__ import annotations

from ..kernels.api import BiasedBranch, Sink
from .base import CombinedCache, Mixer, PagedKV, ParamSpec, register_mixer
from .input_conv import ConvTail

DEFAULT_NAMES = dict(q="q", k="k", v="v", g="g", o="o", temp="temp", q_norm="q.norm", k_norm="k.norm", q_bias="q.b",
                     k_bias="k.b", v_bias="v.b", o_bias="o.b", distance_bias="rel", q_conv="q.conv", k_conv="k.conv", v_conv="v.conv",
                     sink="sink", value_mix="vmix")


def log_distance_buckets(buckets: int, farthest: float) -> list:
    """bucket(n) for n = 0 .. N - 1, N - 1 the first distance that falls into the last bucket (every larger one does too)."""
    import math
    half = buckets // 2
    if buckets < 2 or not farthest > half:
        raise ValueError(f"{buckets} distance buckets up to {farthest}: at least 2, and the farthest beyond the first half")
    out = []
    while True:
        n = len(out)
        b = n if n < half else min(buckets - 1, half + int(math.floor(math.log(n / half) / math.log(farthest / half) * (buckets - half))))
        out.append(b)
        if b == buckets - 1:
            return out


@register_mixer("softmax_attention")
class SoftmaxAttention(Mixer):
    lazy_input = True

    def __init__(self, width: int, num_heads: int, num_kv_heads: int, dim: int, vdim: int, scale: float, position, prefix: str,
                 window: int | None = None, sink=None, values_from_keys: bool = False,
                 head_temperature: bool = False, head_gate: bool = False, qk_norm=False, eps: float = 1e-6,
                 float32_output: bool = False, tensor_names=None, bias: bool = False, position_temperature=None,
                 distance_bias=None, conv: int | None = None, keep_first: int = 0, element_gate: bool = False,
                 share_values: str | None = None, take_values: str | None = None, chunk: int | None = None,
                 out_bias: bool = False):
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} query heads are not a multiple of {num_kv_heads} kv heads")
        if values_from_keys and vdim != dim:
            raise ValueError(f"values that are the keys have the keys' size {dim}, not {vdim}")
        if window is not None and window < 1:
            raise ValueError("window must be >= 1 or None")
        if position is not None and position.rotary_dim > dim:
            raise ValueError(f"the position encoding turns {position.rotary_dim} numbers; a head has {dim}")
        self.width, self.num_heads, self.num_kv_heads = int(width), int(num_heads), int(num_kv_heads)
        self.dim, self.vdim, self.scale = int(dim), int(vdim), float(scale)
        self.padded_dim = -(-max(self.dim, self.vdim) // 16) * 16
        if self.padded_dim > 1024:
            raise ValueError(f"heads of {max(dim, vdim)} numbers are beyond the 1024 the attention kernels take")
        self.position, self.prefix = position, prefix
        if chunk is not None and chunk < 1:
            raise ValueError("chunk must be >= 1 or None")
        self.window, self.chunk = window, chunk
        self.head_sink = sink == "head"
        self.sink = None if sink is None or self.head_sink else float(sink)
        self.values_from_keys, self.head_temperature = bool(values_from_keys), bool(head_temperature)
        if qk_norm not in (False, True, "head", "turned"):
            raise ValueError(f"qk_norm {qk_norm!r}: False, True (the whole projection), 'head' or 'turned' (after the rotation)")
        self.norm_turned = qk_norm == "turned"
        self.head_gate, self.qk_norm, self.eps = bool(head_gate), bool(qk_norm) and not self.norm_turned, float(eps)
        self.norm_per_head = qk_norm == "head"
        self.element_gate = bool(element_gate)
        if self.element_gate and self.head_gate:
            raise ValueError("one output gate: per head or per number")
        self.conv = None if conv is None else int(conv)
        if self.conv is not None and (self.conv < 1 or self.values_from_keys):
            raise ValueError("a convolution on the projections has at least one tap, and is not built with values that are the keys")
        self.keep_first = int(keep_first)
        if self.keep_first < 0 or (self.keep_first and window is None):
            raise ValueError(f"keep_first {keep_first} belongs beside a window")
        self.share_values, self.take_values = share_values, take_values
        if (share_values or take_values) and (self.values_from_keys or (share_values and take_values)):
            raise ValueError("a layer leaves its own values or takes another's, and projects them itself")
        self.has_taps = self.conv is not None
        if self.conv is None and (share_values or take_values or self.norm_turned or (position is not None and position.magnitude != 1.0)):
            if head_temperature or position_temperature is not None or (self.qk_norm and not self.norm_per_head):
                raise ValueError("a scaled rotation, norms after it and shared values are built with norms head by head, without temperatures")
            self.conv = 1           # built for convolved projections only: one tap of one leaves them as they are
        self.taps = self.value_mix = None
        self.mix = 0.0
        self.float32_output = bool(float32_output)
        self.names = dict(DEFAULT_NAMES, **(tensor_names or {}))
        self.has_bias, self.out_bias = bool(bias), bool(out_bias)
        self.b_o = None
        self.position_temperature = None
        if position_temperature is not None:
            coef, every = float(position_temperature[0]), int(position_temperature[1])
            if every < 1 or every != position_temperature[1]:
                raise ValueError(f"a query temperature every {position_temperature[1]} positions: a whole number >= 1")
            self.position_temperature = (coef, every)
        self.distance_buckets = None
        if distance_bias is not None:
            self.distance_buckets = log_distance_buckets(int(distance_bias[0]), float(distance_bias[1]))
            self.num_buckets = int(distance_bias[0])
        self.b_in = self.rel = self.distance_table = None
        H, G = self.num_heads, self.num_kv_heads
        self.q_col, self.k_col = 0, H * self.dim
        self.v_col = None if self.values_from_keys else self.k_col + G * self.dim
        self.gate_col = self.k_col + G * self.dim + (0 if self.values_from_keys else G * self.vdim)
        self.channels = (H + G) * self.dim + G * self.vdim      # of the three projections, in column order

    def children(self):
        return [self.position] if self.position is not None else []

    def params(self):
        n, w, H, G = self.names, self.width, self.num_heads, self.num_kv_heads
        name = lambda k: f"{self.prefix}.{n[k]}"        # noqa: E731
        pieces = [(name("q"), (H * self.dim, w)), (name("k"), (G * self.dim, w))]
        if not self.values_from_keys:
            pieces.append((name("v"), (G * self.vdim, w)))
        if self.head_gate:
            pieces.append((name("g"), (H, w)))
        if self.element_gate:
            pieces.append((name("g"), (H * self.vdim, w)))
        specs = [ParamSpec.stacked("w_in", pieces), ParamSpec.single("w_o", name("o"), (w, H * self.vdim))]
        if self.head_temperature:
            specs.append(ParamSpec.single("temperature", name("temp"), (H,), init="scale"))
        if self.qk_norm:
            specs += [ParamSpec.single("q_norm", name("q_norm"), (self.dim if self.norm_per_head else H * self.dim,), init="scale"),
                      ParamSpec.single("k_norm", name("k_norm"), (self.dim if self.norm_per_head else G * self.dim,), init="scale")]
        if self.has_taps:
            specs.append(ParamSpec.stacked("taps", [(name("q_conv"), (H * self.dim, self.conv)), (name("k_conv"), (G * self.dim, self.conv)),
                                                    (name("v_conv"), (G * self.vdim, self.conv))]))
        if self.head_sink:
            specs.append(ParamSpec.single("sink", name("sink"), (H,)))
        if self.share_values or self.take_values:
            specs.append(ParamSpec.single("value_mix", name("value_mix"), ()))
        if self.has_bias:
            if self.values_from_keys:
                raise ValueError("biased projections with values that are the keys are not built")
            specs.append(ParamSpec.stacked("b_in", [(name("q_bias"), (H * self.dim,)), (name("k_bias"), (G * self.dim,)),
                                                    (name("v_bias"), (G * self.vdim,))]))
        if self.out_bias:
            specs.append(ParamSpec.single("b_o", name("o_bias"), (w,)))
        if self.distance_buckets is not None:
            specs.append(ParamSpec.single("rel", name("distance_bias"), (self.num_buckets, H)))
        return specs

    def cache_requirement(self):
        reach = min((n for n in (self.window, self.chunk) if n is not None), default=None)
        kv = PagedKV(self.num_kv_heads, self.padded_dim, reach, self.keep_first)
        return kv if self.conv is None else CombinedCache([("kv", kv), ("conv", ConvTail(self.channels, self.conv))])

    def prepare(self, device, dtype):
        import torch
        if getattr(self, "_prepared", False):
            return
        self._prepared = True
        rows = self.w_in.shape[0]
        if rows % 16:       # the product kernels like whole tiles of weight rows: the sums get a few columns nobody reads
            padded = torch.zeros((-(-rows // 16) * 16, self.width), dtype=self.w_in.dtype, device=self.w_in.device)
            padded[:rows] = self.w_in
            self.w_in = padded
        P, H = self.padded_dim, self.num_heads
        if P != self.vdim and not self.element_gate:  # the attention's output has P numbers a head, the last P - vdim of them zero
            spread = torch.zeros((self.width, H, P), dtype=self.w_o.dtype, device=self.w_o.device)
            spread[:, :, :self.vdim] = self.w_o.view(self.width, H, self.vdim)
            self.w_o = spread.view(self.width, H * P)
        for attr in ("temperature", "q_norm", "k_norm", "taps", "b_o") + (("sink",) if self.head_sink else ()):     # 32-bit whatever the checkpoint stores
            if getattr(self, attr, None) is not None:
                setattr(self, attr, getattr(self, attr).float().contiguous())
        if self.conv is not None and not self.has_taps:
            self.taps = torch.ones((self.channels, 1), dtype=torch.float32, device=self.w_in.device)
        if self.value_mix is not None:
            self.mix = float(self.value_mix)
        if self.b_in is not None:       # one number a column of the product's sums, zeros for the columns nobody reads
            b = torch.zeros(self.w_in.shape[0], dtype=torch.float32, device=self.w_in.device)
            b[:self.b_in.shape[0]] = self.b_in.float()
            self.b_in = b
        if self.rel is not None:        # [heads, distances]: the table's row for every distance up to the last bucket's first
            rows = torch.tensor(self.distance_buckets, dtype=torch.long, device=self.rel.device)
            self.distance_table = self.rel.float()[rows].t().contiguous()

    def _finish_options(self) -> dict:
        """What only some designs ask of qkv_finish (a backend that knows none of them is not handed any)."""
        opts = {}
        if self.b_in is not None:
            opts["col_bias"] = self.b_in
        if self.position_temperature is not None:
            opts["position_temperature"] = self.position_temperature
        if self.norm_per_head:
            opts["norm_per_head"] = True
        if self.norm_turned:
            opts["norm_turned"] = True
        if self.position is not None and self.position.magnitude != 1.0:
            opts["rotation_scale"] = self.position.magnitude
        return opts

    def _attend(self, sums, base, step, cache):
        """Attention over what the product's sums hold from column ``base`` on -> [T, heads * padded_dim]."""
        import torch
        ops, H, G, P = self.ops, self.num_heads, self.num_kv_heads, self.padded_dim
        opts = self._finish_options()
        if self.conv is not None:
            opts["conv"] = (self.taps, cache.sub("conv").tensors["tail"], step)
            cache = cache.sub("kv")
        if cache.k.shape[-1] != P:
            raise ValueError(f"the cache holds heads of {cache.k.shape[-1]} numbers; this layer's are {P}")
        group = step.groups[cache.group]
        if self.share_values:
            step.shared[self.share_values] = torch.empty((sums.shape[0], G * self.vdim), dtype=torch.float32, device=sums.device)
            opts["values_out"] = step.shared[self.share_values]
        elif self.take_values:
            opts["value_mix"] = (self.mix, step.shared[self.take_values])
        pos = self.position
        q = ops.qkv_finish(sums, base + self.q_col, base + self.k_col, None if self.v_col is None else base + self.v_col,
                           H, G, self.dim, self.vdim, P, step.positions,
                           pos.inv_freq if pos is not None else None, pos.layout if pos is not None else "half",
                           cache.k, cache.v, group.slot_mapping, q_norm=self.q_norm if self.qk_norm else None,
                           k_norm=self.k_norm if self.qk_norm else None, eps=self.eps,
                           q_head_scale=self.temperature if self.head_temperature else None,
                           **opts)
        more = {}
        if self.distance_table is not None:
            more["distance_bias"] = self.distance_table
        if self.keep_first:
            more["keep_first"] = self.keep_first
        if self.chunk is not None:
            more["chunk"] = self.chunk
        return ops.paged_attention(q, H, G, P, cache.k, cache.v, group, step, self.scale, self.window, sink=self.sink, **more)

    @property
    def branch_width(self) -> int:
        """Numbers a token that the output matrix reads (``branch_into``)."""
        return self.num_heads * self.vdim

    def branch_into(self, out, scale, sums, base, step, cache):
        """What the output matrix reads, times ``scale``, into ``out`` [T, branch_width] (a caller that joins several
        parts' outputs in one product); ``sums``, ``base`` as for forward."""
        if not self.element_gate or self.out_bias:
            raise ValueError("joining outputs is built for heads with a gate per number and no output bias")
        o = self._attend(sums, base, step, cache)
        self.ops.gate_heads(o, sums, base + self.gate_col, self.num_heads, self.vdim, self.padded_dim, out=out, scale=scale)

    def forward(self, x, step, cache, add_to=None, sums=None, base=0):
        """``sums``: the float32 sums of a product that holds this part's ``w_in`` rows from column ``base`` on (a
        caller that stacked several parts' input matrices); ``x`` is then not read."""
        import torch
        ops, H, P = self.ops, self.num_heads, self.padded_dim
        if sums is None:
            sums, base = ops.linear(x, self.w_in, out_dtype=torch.float32), 0
        elif self.b_in is not None:
            raise ValueError("biased projections inside another part's product are not built")
        o = self._attend(sums, base, step, cache)
        if self.head_gate:
            o = ops.head_gate_(o, sums, base + self.gate_col, H, P)
        elif self.element_gate:
            o = ops.gate_heads(o, sums, base + self.gate_col, H, self.vdim, P)
        if self.out_bias:
            if add_to is None:
                return ops.linear(o, self.w_o, out_dtype=torch.float32).add_(self.b_o)
            y = ops.linear(o, self.w_o, add_to=Sink(add_to.stream) if isinstance(add_to, Sink) else add_to)
            return BiasedBranch(y, self.b_o)        # the bias is added by whoever reads the stream next
        if add_to is None and self.float32_output:
            return ops.linear(o, self.w_o, out_dtype=torch.float32)
        return ops.linear(o, self.w_o, add_to=add_to)
