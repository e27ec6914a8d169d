"""Causal self-attention over a paged cache, with grouped KV heads.

q, k, v projections without bias; rotary on q and k before the keys are
cached; for the token at position p, head h reads KV head h // (H/KV) and keys
[0, p] (or the last ``window`` of them); scores times 1/sqrt(head_dim),
softmax in 32-bit, values, output projection
(backend/model.cu:1090-1104, :343-408, :224-225).

Parameters: ``hidden``, ``heads``, ``kv_heads``, ``head_dim``, ``window``
(0: all keys), ``position`` (a PartSpec or None), ``own_kv`` (False: the run
reads keys and values that another run cached and has no k/v projections),
``scale`` (default 1/sqrt(head_dim)), ``distance_slope_bits`` (None: no bias; b:
head h's scaled scores lose 2^(-b (h+1) / heads) times the distance from the
query to the key), ``chunk`` (0: none; c: a chunked mask, the query at position
p reads no key before p - p % c, chunks counted from the request's position 0),
``sink`` (False; True: the softmax's denominator has one more term, exp(0): a
key whose score is 0 and that has no value; "learned": exp of a number per head, a
tensor of the part, for parts that have one), ``value_dim`` (width of a value;
default: the key's), ``keep_first`` (with a window: the first ``keep_first``
positions of a request stay readable behind it, at their true positions).
Tensors: ``<prefix>.{q,k,v,o}_proj.weight``.  The three input projections are
kept as one matrix so that a step reads one weight for them.
"""

from __future__ import annotations

import math

import torch

from .. import kernels as K
from .base import Normed, Part, register_part
from .linear import decode_linear, linear, linear_into, tiled_copy
from .spec import CacheNeed, WeightSpec


@register_part("mixer", "attention")
class CausalSelfAttention(Part):
    graph_safe = True
    records_launches = True
    takes_normed = True     # the q, k, v product of a decode batch applies the norm's row scale itself
    fills_sink = True       # the output projection of a decode batch adds itself to the residual stream
    # How the attention kernels want a step's spans listed: the tokens of spans of at most
    # SHORT_SPAN tokens one by one (for the kernel that cuts a token's keys into slices),
    # longer spans in blocks of QUERY_BLOCK tokens (for the prompt kernel).
    step_lists_key = "attention.spans"
    SHORT_SPAN = 4
    QUERY_BLOCK = K.PREFILL_QUERY_BLOCK
    FAST_KERNELS_OFF = False
    learns_sinks = False      # whether the part has a tensor for ``sink`` "learned"
    pads_heads = False        # whether the pages' slots may be wider than the heads

    def step_lists(self, starts, lens):
        short, blocks = [], []
        for s, n in enumerate(lens):
            a = starts[s]
            if n <= self.SHORT_SPAN:
                short.extend(range(a, a + n))
            else:
                for t in range(a, a + n, self.QUERY_BLOCK):
                    blocks += [t, s]
        return {"short": short, "blocks": blocks}

    def step_values(self, starts, lens, positions):
        """How many keys the step's query blocks read, all together and the longest block
        alone: a whole prompt's blocks read more and more, a portion far into its context reads
        many in every block, and the prompt kernel is chosen by that."""
        total = longest = 0
        for pos, n in zip(positions, lens):
            if n <= self.SHORT_SPAN:
                continue
            for first in range(0, n, self.QUERY_BLOCK):
                last = pos + min(first + self.QUERY_BLOCK, n)          # keys [0, last) are before the block's end
                keys = min(last, self.window + self.QUERY_BLOCK) if self.window else last
                if self.chunk:      # nothing before the chunk of the block's first query
                    keys = min(keys, last - (pos + first) // self.chunk * self.chunk)
                total += keys
                longest = max(longest, keys)
        return {"keys_total": total, "keys_longest": longest}

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        self.hidden = int(self.param("hidden"))
        self.heads = int(self.param("heads"))
        self.kv_heads = int(self.param("kv_heads"))
        self.head_dim = int(self.param("head_dim"))
        self.window = int(self.param("window", 0) or 0)
        self.chunk = int(self.param("chunk", 0) or 0)
        self.sink = self.param("sink", False)
        self.sinks = None           # float32 [heads] on the device once bound: the score of a key without a value
        if self.sink not in (False, True, None) and not (self.sink == "learned" and self.learns_sinks):
            raise ValueError(f"attention: sink {self.sink!r} is not built for this part")
        self.value_dim = int(self.param("value_dim", None) or self.head_dim)
        self.keep_first = int(self.param("keep_first", 0) or 0) if self.window else 0
        if self.chunk < 0 or self.keep_first < 0 or not 0 < self.value_dim <= 256:
            raise ValueError(f"attention: chunk {self.chunk}, keep_first {self.keep_first} or value_dim "
                             f"{self.value_dim} out of range")
        # layers with the same window and chunk read alike
        self.step_values_key = (f"attention.keys.window{self.window}" + (f".chunk{self.chunk}" if self.chunk else "")
                                + (f".first{self.keep_first}" if self.keep_first else ""))
        self.own_kv = bool(self.param("own_kv", True))
        if self.heads % self.kv_heads:
            raise ValueError(f"attention: {self.heads} heads are not a multiple of {self.kv_heads} KV heads")
        if (self.head_dim % 2 and not self.pads_heads) or self.head_dim > 256:
            raise ValueError(f"attention: head_dim {self.head_dim} must be even and at most 256")
        pos = self.param("position", None)
        self.position = runtime.shared_part("position", pos) if pos is not None else None
        # How the position part wants a head rotated (default: the whole head, halves paired, which
        # is what the fused epilogues of the small-batch products do; anything else goes through
        # the separate rotate-and-append kernel, which takes the pairing as arguments).
        rotates = self.position is not None and hasattr(self.position, "tables")
        self.rotary_dim = int(getattr(self.position, "rotary_dim", self.head_dim)) if rotates else self.head_dim
        self.interleaved = bool(getattr(self.position, "interleaved", False)) if rotates else False
        if self.rotary_dim % 2 or not 0 <= self.rotary_dim <= self.head_dim:
            raise ValueError(f"attention: rotary dimension {self.rotary_dim} of a head of {self.head_dim}")
        self.plain_rotation = self.rotary_dim == self.head_dim and not self.interleaved
        scale = self.param("scale", None)
        self.scale = float(scale) if scale is not None else 1.0 / math.sqrt(self.head_dim)
        bits = self.param("distance_slope_bits", None)
        self.slope_bits = float(bits) if bits is not None else None
        self.slopes = None          # float32 [heads] on the device once bound
        self.q_dim = self.heads * self.head_dim
        self.kv_dim = self.kv_heads * self.head_dim
        self.out_dim = self.heads * self.value_dim
        self.w_in = None
        self.w_o = None
        self._tiled = {}

    def weight_specs(self):
        specs = [WeightSpec(self.tensor_name("q_proj.weight"), (self.q_dim, self.hidden))]
        if self.own_kv:
            specs += [WeightSpec(self.tensor_name("k_proj.weight"), (self.kv_dim, self.hidden)),
                      WeightSpec(self.tensor_name("v_proj.weight"), (self.kv_dim, self.hidden))]
        specs.append(WeightSpec(self.tensor_name("o_proj.weight"), (self.hidden, self.q_dim)))
        return specs

    def _bind_slopes(self):
        if self.sink is True:
            self.sinks = torch.zeros(self.heads, dtype=torch.float32, device=self.runtime.device)
        if self.slope_bits is not None:
            values = [2.0 ** (-self.slope_bits * (h + 1) / self.heads) for h in range(self.heads)]
            self.slopes = torch.tensor(values, dtype=torch.float32, device=self.runtime.device)

    # ---- parts that ``pads_heads``: pages hold one width for keys and values, the smallest that the
    # kernels on the matrix cores take for both (the rest of a slot is zero)
    def _pad_heads(self):
        self.key_dim, self.val_dim = self.head_dim, self.value_dim
        widest = max(self.key_dim, self.val_dim)
        self.width = next(w for w in K.PREFILL_HEAD_DIMS if w >= widest)
        # the rest of this class sees heads of the pages' width
        self.head_dim = self.value_dim = self.width
        self.q_dim = self.out_dim = self.heads * self.width
        self.kv_dim = self.kv_heads * self.width

    def _padded_output(self, w_o):
        """The output projection with columns of zeros where a head's output is padding."""
        if self.width == self.val_dim:
            return w_o
        by_head = w_o.reshape(self.hidden, self.heads, self.val_dim)
        return torch.nn.functional.pad(by_head, (0, self.width - self.val_dim)).reshape(self.hidden, -1).contiguous()

    def bind(self, weights):
        self._bind_slopes()
        names = ["q_proj.weight"] + (["k_proj.weight", "v_proj.weight"] if self.own_kv else [])
        mats = [weights[self.tensor_name(n)] for n in names]
        self.w_in = torch.cat(mats, dim=0).contiguous() if len(mats) > 1 else mats[0]
        self.w_o = weights[self.tensor_name("o_proj.weight")]
        # second copies for decode batches, in the order that kernel reads them (not tensors of
        # the part in the sense of read_bytes: a step reads one copy or the other)
        self._tiled = {}
        if self.plain_rotation:
            heads = K.Rope(None, None, True if self.own_kv else None, None, None, None, 0, self.heads, self.kv_heads,
                           self.head_dim)
            self._tiled["in"] = tiled_copy(self.runtime, self.w_in, K.LINEAR_ROPE, heads)
        self._tiled["o"] = tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)

    def cache_need(self):
        return CacheNeed("paged", kv_heads=self.kv_heads, head_dim=self.head_dim, window=self.window,
                         value_dim=self.value_dim if self.value_dim != self.head_dim else None,
                         keep_first=self.keep_first)

    def flops(self, tokens, keys_read=0.0):
        # the projections, and per key read a score and a value product for every head
        return super().flops(tokens) + 4.0 * self.heads * self.head_dim * keys_read

    def check_cache(self, page_size):
        # The kernel that takes every size walks a chunk of up to 256 keys at a time, whole
        # pages of them; the faster kernels are chosen per step where the sizes fit them.
        if not 1 <= page_size <= K.GENERIC_MAX_PAGE_SIZE:
            raise ValueError(f"attention: pages of {page_size} tokens are not built "
                             f"(1 to {K.GENERIC_MAX_PAGE_SIZE})")

    def _fused_tiles(self, n):
        """Tiles per workgroup of the decode-batch kernel for the input projections of n
        tokens, or 0 where it is not taken."""
        if (self.runtime.dtype != torch.bfloat16 or n > K.FUSED_ROPE_BEST_ROWS or not self.plain_rotation
                or self.runtime.options.get("no_fused_linear")):
            return 0
        return K.fused_linear_tiles(n, self.w_in.shape[0], self.hidden)

    def forward(self, ctx, xn, cache, sink=None):
        dtype = self.runtime.dtype
        if isinstance(xn, Normed):
            n = xn.rows
            opts = self.runtime.options
            gemv = (K.gemv_fits(n, self.w_in.shape[0], self.hidden, dtype) and n <= K.normed_max_rows()
                    and not opts.get("no_fused_gemv") and self.plain_rotation and xn.xw is None)
            scaled = (not gemv and xn.xw is not None and self._fused_tiles(n) > 0)
            # the small-batch kernel below normalises while it stages its input, the decode-batch
            # kernel scales its sums by the row
            xn = xn.kernel_input() if gemv else xn.scaled_rows() if scaled else xn.materialize(ctx)
        n = xn.shape[0]
        writes = self.own_kv
        if writes != bool(cache.write):
            raise ValueError("attention: a run must write its cache exactly when it has k/v projections")
        q = ctx.buf("attn.q", (n, self.q_dim), dtype)
        cos = sin = None
        if self.position is not None and hasattr(self.position, "tables"):
            cos, sin = self.position.tables(ctx)
        plain_rotation = self.plain_rotation
        pages = cache.pages if writes else None
        opts = self.runtime.options
        if (K.gemv_fits(n, self.w_in.shape[0], self.hidden, dtype) and not opts.get("no_fused_gemv") and plain_rotation
                and not isinstance(xn, K.ScaledRows)):
            # few tokens: projections, rotation and append in one launch
            K.gemv_rope_append(xn, self.w_in, q, cos, sin, pages, ctx.positions, ctx.span_of_token,
                               cache.block_table, cache.page_size, self.heads, self.kv_heads,
                               self.head_dim)
        elif self._fused_tiles(n) > 0:
            # a decode batch: the same on the matrix cores
            K.fused_linear(self._tiled.get("in") or self.w_in, q, K.LINEAR_ROPE, x=xn,
                           tiles_per_wg=self._fused_tiles(n),
                           rope=K.Rope(cos, sin, pages, ctx.positions, ctx.span_of_token, cache.block_table,
                                       cache.page_size, self.heads, self.kv_heads, self.head_dim))
        else:
            qkv = linear(ctx, xn, self.w_in, "attn.qkv")
            K.rope_append(qkv, q, cos, sin, pages, ctx.positions, ctx.span_of_token,
                          cache.block_table, cache.page_size, self.heads, self.kv_heads,
                          self.head_dim, self.rotary_dim, self.interleaved)
        out = ctx.buf("attn.out", (n, self.q_dim), dtype)
        self.attend(ctx, q, out, cache)
        if sink is not None:
            normed = linear_into(ctx, out, self.w_o, sink, "attn.proj", w_tiled=self._tiled.get("o"))
            if normed is not None:
                return normed
        return linear(ctx, out, self.w_o, "attn.proj")

    def attend(self, ctx, q, out, cache, gate=None):
        """Choose the attention kernels by the spans' lengths: tokens of short
        spans (decode tokens) go to the kernel that splits a token's keys over
        many waves, longer spans to the prompt kernel in blocks of 128 queries
        (both on the matrix cores, in bfloat16 or with 32-bit operands); sizes
        those kernels do not take go to the kernel that takes every size.  ``gate``
        (``K.Columns`` of sums): its logistic function multiplies the output."""
        mode = self.runtime.options.get("attention", "auto")
        if q.dtype == torch.bfloat16:
            fast = cache.page_size % 16 == 0 and self.head_dim in K.DECODE_HEAD_DIMS
            prompt_ok = self.head_dim in K.PREFILL_HEAD_DIMS
        else:
            fast = prompt_ok = K.attn_f32_fits(self.head_dim, cache.page_size)
        # the kernels on the matrix cores take keys and values of one width; the 32-bit ones one run of
        # keys a query (no kept first positions)
        fast = (fast and mode != "generic" and self.value_dim == self.head_dim and not self.FAST_KERNELS_OFF
                and not (self.keep_first and (q.dtype != torch.bfloat16 or self.slopes is not None)))
        if not fast:
            K.attn_generic(q, out, cache.pages, ctx.positions, ctx.span_of_token, cache.block_table,
                           cache.page_size, self.heads, self.kv_heads, self.head_dim, self.window,
                           self.scale, slopes=self.slopes, value_dim=self.value_dim, chunk=self.chunk, sink=self.sinks,
                           keep_first=self.keep_first, gate=gate)
            return
        n = q.shape[0]
        short = ctx.lists.get("attention.spans.short")
        blocks = ctx.lists.get("attention.spans.blocks")
        n_short = short.numel() if short is not None else 0
        n_blocks = blocks.numel() // 2 if blocks is not None else 0
        if n_short + n_blocks == 0 or (n_blocks and not prompt_ok):   # a context built by hand may carry no lists
            self._decode(ctx, q, out, cache, None, n, gate)   # token by token
            return
        if n_short:
            self._decode(ctx, q, out, cache, None if n_short == n else short, n_short, gate)
        if n_blocks:
            total, longest = self._keys_read(ctx)
            part = None
            slices = (1 if self.runtime.options.get("no_attention_slices")
                      else K.attn_prefill_slices(n_blocks, self.heads, self.head_dim, q.dtype))
            if slices > 1:     # few blocks of a large head: their keys in slices over workgroups, merged in the same call
                part = ctx.buf("attn.block_part", (n * self.heads * slices * (self.head_dim + 2),), torch.float32)
            K.attn_prefill(q, out, cache.pages, blocks, n_blocks, ctx.span_start,
                           ctx.span_pos, cache.block_table, cache.page_size, self.heads,
                           self.kv_heads, self.head_dim, self.window, self.scale, total, longest, part=part,
                           nslices=slices, slopes=self.slopes, chunk=self.chunk, sink=self.sinks,
                           keep_first=self.keep_first, gate=gate)

    def _keys_read(self, ctx):
        """The step's key counts (see ``step_values``), as the engine worked them out for this
        step, or from the host's copies of the spans for a context built by hand."""
        v, key = ctx.values, self.step_values_key
        if key + ".keys_total" in v:
            return v[key + ".keys_total"], v[key + ".keys_longest"]
        own = self.step_values(ctx.h_span_start, ctx.h_span_len, ctx.h_span_pos)
        return own["keys_total"], own["keys_longest"]

    def _decode(self, ctx, q, out, cache, token_list, count, gate=None):
        n = q.shape[0]
        # The block table's width bounds the keys of the step's longest request.  It is rounded up
        # to a power of two of pages (from 8), as recorded steps round theirs: a step then cuts
        # the keys alike, and gives the same sums bit for bit, whether it runs directly or as
        # a replayed recording with a wider table.
        pages = 8
        while pages < cache.block_table.shape[1]:
            pages *= 2
        max_keys = pages * cache.page_size
        if self.window:
            max_keys = min(max_keys, self.window + self.keep_first + cache.page_size)
        if self.chunk:
            max_keys = min(max_keys, self.chunk)
        nslices = K.attn_decode_slices(count, self.kv_heads, self.heads, self.head_dim, q.dtype, max_keys)
        part = ctx.buf("attn.part", (n * self.heads * nslices * (self.head_dim + 2),), torch.float32)
        K.attn_decode(q, out, part, cache.pages, ctx.positions, ctx.span_of_token, cache.block_table,
                      cache.page_size, self.heads, self.kv_heads, self.head_dim, self.window,
                      self.scale, nslices, token_list, count, slopes=self.slopes, chunk=self.chunk, sink=self.sinks,
                      keep_first=self.keep_first, gate=gate)


@register_part("mixer", "attention_keys_as_values")
class KeysAsValuesAttention(CausalSelfAttention):
    """Attention whose values are its keys: there is no value projection, the key as projected
    is cached as the value and its normalised form as the key.  Queries and keys have biases
    and are each normalised over the whole projection, all heads at once (RMS, plain weights);
    the query is multiplied by 1 + coef * ln(floor((p + 1) / every) + 1) at position p; no
    rotation.  Scores, the distance bias, the softmax and the kernels are the base class's.

    Parameters beyond the base class's: ``eps`` (of the two norms), ``q_temp`` (None or a
    (coef, every) pair), ``bias`` (default True: q, k and the output projection have one).
    Tensors: ``<prefix>.{q,k,o}.weight``, ``.{q,k,o}.bias``, ``.{q,k}.norm``."""
    takes_normed = False
    fills_sink = False

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        if not self.own_kv or self.position is not None:
            raise ValueError("attention_keys_as_values: keeps its own keys and takes no position part")
        self.eps = float(self.param("eps"))
        temp = self.param("q_temp", None)
        self.temp_coef, self.temp_every = (float(temp[0]), int(temp[1])) if temp else (0.0, 0)
        if temp and self.temp_every < 1:
            raise ValueError(f"attention_keys_as_values: q_temp every {self.temp_every} must be positive")
        self.has_bias = bool(self.param("bias", True))
        self.q_bias = self.k_bias = self.out_bias = self.q_norm = self.k_norm = None

    def weight_specs(self):
        specs = [WeightSpec(self.tensor_name("q.weight"), (self.q_dim, self.hidden)),
                 WeightSpec(self.tensor_name("k.weight"), (self.kv_dim, self.hidden)),
                 WeightSpec(self.tensor_name("o.weight"), (self.hidden, self.q_dim)),
                 WeightSpec(self.tensor_name("q.norm"), (self.q_dim,), "vector"),
                 WeightSpec(self.tensor_name("k.norm"), (self.kv_dim,), "vector")]
        if self.has_bias:
            specs += [WeightSpec(self.tensor_name("q.bias"), (self.q_dim,), "vector"),
                      WeightSpec(self.tensor_name("k.bias"), (self.kv_dim,), "vector"),
                      WeightSpec(self.tensor_name("o.bias"), (self.hidden,), "vector")]
        return specs

    def bind(self, weights):
        self._bind_slopes()
        self.w_in = torch.cat([weights[self.tensor_name("q.weight")], weights[self.tensor_name("k.weight")]],
                              dim=0).contiguous()
        self.w_o = weights[self.tensor_name("o.weight")]
        self.q_norm = weights[self.tensor_name("q.norm")]
        self.k_norm = weights[self.tensor_name("k.norm")]
        if self.has_bias:
            self.q_bias = weights[self.tensor_name("q.bias")]
            self.k_bias = weights[self.tensor_name("k.bias")]
            self.out_bias = weights[self.tensor_name("o.bias")]     # the arrangement adds it with the output
        # second copies for decode batches, in the order that kernel reads them
        self._tiled = {"in": tiled_copy(self.runtime, self.w_in, K.LINEAR_PARTS),
                       "o": tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)}

    def forward(self, ctx, xn, cache):
        n = xn.shape[0]
        dtype = self.runtime.dtype
        if not cache.write:
            raise ValueError("attention_keys_as_values: the run writes its own cache")
        qk = decode_linear(ctx, xn, self.w_in, "attn.qk", self._tiled.get("in"))
        q = ctx.buf("attn.q", (n, self.q_dim), dtype)
        K.qk_norm_append(qk, q, cache.pages, ctx.positions, ctx.span_of_token, cache.block_table, cache.page_size,
                         self.heads, self.kv_heads, self.head_dim, q_bias=self.q_bias, k_bias=self.k_bias,
                         q_weight=self.q_norm, k_weight=self.k_norm, eps=self.eps, temp_coef=self.temp_coef,
                         temp_every=self.temp_every)
        out = ctx.buf("attn.out", (n, self.q_dim), dtype)
        self.attend(ctx, q, out, cache)
        return decode_linear(ctx, out, self.w_o, "attn.proj", self._tiled.get("o"))


@register_part("mixer", "attention_unit_qk")
class UnitNormAttention(CausalSelfAttention):
    """Attention whose queries and keys are rotated and then divided, head by head, by their root
    mean square (an RMS norm without a weight): q = W_q h + b_q, k = W_k h + b_k, v = W_v h + b_v;
    the first ``rotary_dim`` elements of every query and key head turn with the position (the
    position part says how); q and k become q / sqrt(mean(q^2) + eps) per head; the score is
    (q . k) * ``scale``; mask (``window``, ``chunk``), ``sink`` and the kernels are the base
    class's; values may have a width of their own (``value_dim``); the output projection has no
    bias.

    Parameters beyond the base class's: ``eps``, ``bias`` (default True: q, k and v have one).
    Tensors: ``<prefix>.{q,k,v,o}.weight``, ``.{q,k,v}.bias``."""
    takes_normed = False
    fills_sink = False

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        if not self.own_kv:
            raise ValueError("attention_unit_qk: keeps its own keys and values")
        self.eps = float(self.param("eps"))
        self.has_bias = bool(self.param("bias", True))
        self.v_dim = self.kv_heads * self.value_dim
        self.bias = None

    def weight_specs(self):
        specs = [WeightSpec(self.tensor_name("q.weight"), (self.q_dim, self.hidden)),
                 WeightSpec(self.tensor_name("k.weight"), (self.kv_dim, self.hidden)),
                 WeightSpec(self.tensor_name("v.weight"), (self.v_dim, self.hidden)),
                 WeightSpec(self.tensor_name("o.weight"), (self.hidden, self.out_dim))]
        if self.has_bias:
            specs += [WeightSpec(self.tensor_name("q.bias"), (self.q_dim,), "vector"),
                      WeightSpec(self.tensor_name("k.bias"), (self.kv_dim,), "vector"),
                      WeightSpec(self.tensor_name("v.bias"), (self.v_dim,), "vector")]
        return specs

    def bind(self, weights):
        self._bind_slopes()
        self.w_in = torch.cat([weights[self.tensor_name(t + ".weight")] for t in ("q", "k", "v")], dim=0).contiguous()
        self.w_o = weights[self.tensor_name("o.weight")]
        self.bias = (torch.cat([weights[self.tensor_name(t + ".bias")] for t in ("q", "k", "v")]).contiguous()
                     if self.has_bias else None)
        # second copies for decode batches, in the order that kernel reads them
        self._tiled = {"in": tiled_copy(self.runtime, self.w_in, K.LINEAR_PARTS),
                       "o": tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)}

    def forward(self, ctx, xn, cache):
        n = xn.shape[0]
        dtype = self.runtime.dtype
        if not cache.write:
            raise ValueError("attention_unit_qk: the run writes its own cache")
        qkv = decode_linear(ctx, xn, self.w_in, "attn.qkv", self._tiled.get("in"))
        q = ctx.buf("attn.q", (n, self.q_dim), dtype)
        cos = sin = None
        if self.position is not None and hasattr(self.position, "tables"):
            cos, sin = self.position.tables(ctx)
        K.qkv_norm_append(qkv, q, cache.pages, ctx.positions, ctx.span_of_token, cache.block_table, cache.page_size,
                          self.heads, self.kv_heads, self.head_dim, self.value_dim, bias=self.bias, cos=cos, sin=sin,
                          rotary_dim=self.rotary_dim, interleaved=self.interleaved, unit_norm=True, eps=self.eps)
        out = ctx.buf("attn.out", (n, self.out_dim), dtype)
        self.attend(ctx, q, out, cache)
        return decode_linear(ctx, out, self.w_o, "attn.proj", self._tiled.get("o"))


@register_part("mixer", "attention_qk_norm")
class NormedQueryKeyAttention(CausalSelfAttention):
    """Attention whose queries and keys pass an RMS norm per head, with a weight of the head's size
    that all heads share, in front of the rotation: q = W_q h, k = W_k h, v = W_v h without biases;
    every query and key head is divided by its root mean square and multiplied by the weight; the
    first ``rotary_dim`` elements of every head then turn with the position (the position part
    says how); the score is (q . k) * ``scale``; mask (``window``, ``keep_first``, ``chunk``),
    ``sink`` and the kernels are the base class's; values may have a width of their own.

    Parameters beyond the base class's: ``eps``.
    Tensors: ``<prefix>.{q,k,v,o}.weight``, ``.{q,k}.norm``."""
    takes_normed = False
    fills_sink = False

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        if not self.own_kv:
            raise ValueError("attention_qk_norm: keeps its own keys and values")
        self.eps = float(self.param("eps"))
        self.v_dim = self.kv_heads * self.value_dim
        self.q_norm = self.k_norm = None

    def weight_specs(self):
        return [WeightSpec(self.tensor_name("q.weight"), (self.q_dim, self.hidden)),
                WeightSpec(self.tensor_name("k.weight"), (self.kv_dim, self.hidden)),
                WeightSpec(self.tensor_name("v.weight"), (self.v_dim, self.hidden)),
                WeightSpec(self.tensor_name("o.weight"), (self.hidden, self.out_dim)),
                WeightSpec(self.tensor_name("q.norm"), (self.head_dim,), "vector"),
                WeightSpec(self.tensor_name("k.norm"), (self.head_dim,), "vector")]

    def bind(self, weights):
        self._bind_slopes()
        self.w_in = torch.cat([weights[self.tensor_name(t + ".weight")] for t in ("q", "k", "v")], dim=0).contiguous()
        self.w_o = weights[self.tensor_name("o.weight")]
        self.q_norm = weights[self.tensor_name("q.norm")]
        self.k_norm = weights[self.tensor_name("k.norm")]
        # second copies for decode batches, in the order that kernel reads them
        self._tiled = {"in": tiled_copy(self.runtime, self.w_in, K.LINEAR_PARTS),
                       "o": tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)}

    def forward(self, ctx, xn, cache):
        n = xn.shape[0]
        dtype = self.runtime.dtype
        if not cache.write:
            raise ValueError("attention_qk_norm: the run writes its own cache")
        qkv = decode_linear(ctx, xn, self.w_in, "attn.qkv", self._tiled.get("in"))
        q = ctx.buf("attn.q", (n, self.q_dim), dtype)
        cos = sin = None
        if self.position is not None and hasattr(self.position, "tables"):
            cos, sin = self.position.tables(ctx)
        K.qkv_norm_append(qkv, q, cache.pages, ctx.positions, ctx.span_of_token, cache.block_table, cache.page_size,
                          self.heads, self.kv_heads, self.head_dim, self.value_dim, cos=cos, sin=sin,
                          rotary_dim=self.rotary_dim, interleaved=self.interleaved, unit_norm=False, eps=self.eps,
                          q_weight=self.q_norm, k_weight=self.k_norm)
        out = ctx.buf("attn.out", (n, self.out_dim), dtype)
        self.attend(ctx, q, out, cache)
        return decode_linear(ctx, out, self.w_o, "attn.proj", self._tiled.get("o"))


@register_part("mixer", "attention_whole_norm")
class WholeNormAttention(CausalSelfAttention):
    """Attention whose queries and keys pass an RMS norm over the whole projection, all heads at
    once, with plain weights as long as the projection: q = W_q h, k = W_k h, v = W_v h without
    biases; the first ``rotary_dim`` elements of every query and key head then turn with the
    position, if there is a position part (it says how); the query is multiplied by 1 + coef *
    ln(floor((p + 1) / every) + 1) at position p (``q_temp``); the score is (q . k) * ``scale``;
    mask (``window``, ``chunk``), ``sink`` and the kernels are the base class's; values may have a
    width of their own.

    Parameters beyond the base class's: ``eps`` (of the two norms), ``q_temp`` (None or a (coef,
    every) pair).  Tensors: ``<prefix>.{q,k,v,o}.weight``, ``.{q,k}.norm``."""
    takes_normed = False
    fills_sink = False

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        if not self.own_kv:
            raise ValueError("attention_whole_norm: keeps its own keys and values")
        self.eps = float(self.param("eps"))
        temp = self.param("q_temp", None)
        self.temp_coef, self.temp_every = (float(temp[0]), int(temp[1])) if temp else (0.0, 0)
        if temp and self.temp_every < 1:
            raise ValueError(f"attention_whole_norm: q_temp every {self.temp_every} must be positive")
        self.v_dim = self.kv_heads * self.value_dim
        self.q_norm = self.k_norm = None

    def weight_specs(self):
        return [WeightSpec(self.tensor_name("q.weight"), (self.q_dim, self.hidden)),
                WeightSpec(self.tensor_name("k.weight"), (self.kv_dim, self.hidden)),
                WeightSpec(self.tensor_name("v.weight"), (self.v_dim, self.hidden)),
                WeightSpec(self.tensor_name("o.weight"), (self.hidden, self.out_dim)),
                WeightSpec(self.tensor_name("q.norm"), (self.q_dim,), "vector"),
                WeightSpec(self.tensor_name("k.norm"), (self.kv_dim,), "vector")]

    def bind(self, weights):
        self._bind_slopes()
        self.w_in = torch.cat([weights[self.tensor_name(t + ".weight")] for t in ("q", "k", "v")], dim=0).contiguous()
        self.w_o = weights[self.tensor_name("o.weight")]
        self.q_norm = weights[self.tensor_name("q.norm")]
        self.k_norm = weights[self.tensor_name("k.norm")]
        # second copies for decode batches, in the order that kernel reads them
        self._tiled = {"in": tiled_copy(self.runtime, self.w_in, K.LINEAR_PARTS),
                       "o": tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)}

    def forward(self, ctx, xn, cache):
        n = xn.shape[0]
        dtype = self.runtime.dtype
        if not cache.write:
            raise ValueError("attention_whole_norm: the run writes its own cache")
        qkv = decode_linear(ctx, xn, self.w_in, "attn.qkv", self._tiled.get("in"))
        q = ctx.buf("attn.q", (n, self.q_dim), dtype)
        cos = sin = None
        if self.position is not None and hasattr(self.position, "tables"):
            cos, sin = self.position.tables(ctx)
        K.qk_norm_append(qkv, q, cache.pages, ctx.positions, ctx.span_of_token, cache.block_table, cache.page_size,
                         self.heads, self.kv_heads, self.head_dim, q_weight=self.q_norm, k_weight=self.k_norm,
                         eps=self.eps, temp_coef=self.temp_coef, temp_every=self.temp_every, value_dim=self.value_dim,
                         cos=cos, sin=sin, rotary_dim=self.rotary_dim, interleaved=self.interleaved)
        out = ctx.buf("attn.out", (n, self.out_dim), dtype)
        self.attend(ctx, q, out, cache)
        return decode_linear(ctx, out, self.w_o, "attn.proj", self._tiled.get("o"))


@register_part("mixer", "attention_conv")
class ConvolvedAttention(CausalSelfAttention):
    """Attention whose queries, keys and values are smoothed channel by channel over the last
    positions (a convolution of ``taps`` weights, the last one the current token's, zeros before position 0) right behind
    their projections: q = conv(W_q h), k = conv(W_k h), v = conv(W_v h) without biases; the first
    ``rotary_dim`` elements of every query and key head then turn with the position, if there is a
    position part (it says how); the score is (q . k) * ``scale``; mask (``window``, ``chunk``), ``sink`` and the
    kernels are the base class's; values may have a width of their own.

    A request keeps its pages and, in a state slot, the projections of its last taps - 1 positions
    (``cache_need`` is the list of both).  Pages hold one width for keys and values, the smallest that
    the kernels on the matrix cores take for both (the rest of a slot is zero); the output projection's
    columns are padded likewise.

    Parameters beyond the base class's: ``taps``.
    Tensors: ``<prefix>.{q,k,v,o}.weight``, ``.{q,k,v}.conv`` [channels, taps]."""
    takes_normed = False
    fills_sink = False
    shares_input = True       # its input product may be a part of a larger one (``sums``)
    folds_scale = True        # a factor on its output (``out_scale``) is a factor on its values
    pads_heads = True
    MAX_TAPS = 16

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        if not self.own_kv or self.keep_first:
            raise ValueError("attention_conv: keeps its own keys and values, all of them behind one edge")
        self.taps = int(self.param("taps"))
        if not 1 <= self.taps <= self.MAX_TAPS:
            raise ValueError(f"attention_conv: a convolution of {self.taps} taps is not built (1 to {self.MAX_TAPS})")
        self._pad_heads()
        self.channels = (self.heads + self.kv_heads) * self.key_dim + self.kv_heads * self.val_dim
        self.out_scale = 1.0
        self.conv = None

    def weight_specs(self):
        d, name = self.hidden, self.tensor_name
        rows = {"q": self.heads * self.key_dim, "k": self.kv_heads * self.key_dim, "v": self.kv_heads * self.val_dim}
        return ([WeightSpec(name(t + ".weight"), (rows[t], d)) for t in ("q", "k", "v")]
                + [WeightSpec(name(t + ".conv"), (rows[t], self.taps), "vector") for t in ("q", "k", "v")]
                + [WeightSpec(name("o.weight"), (d, self.heads * self.val_dim))])

    def bind(self, weights):
        self._bind_slopes()
        w = lambda n: weights[self.tensor_name(n)]
        self.w_in = torch.cat([w(t + ".weight") for t in ("q", "k", "v")], dim=0).contiguous()
        self.conv = torch.cat([w(t + ".conv") for t in ("q", "k", "v")], dim=0).contiguous()
        self.w_o = self._padded_output(w("o.weight"))
        self._tiled = {"in": tiled_copy(self.runtime, self.w_in, K.LINEAR_PARTS),
                       "o": tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)}

    def input_matrix(self):
        return self.w_in

    def share_input(self, rows):
        """The input matrix is ``rows`` of a larger one, whose product is made by the caller."""
        self.w_in = rows
        self._tiled.pop("in", None)

    def cache_need(self):
        pages = super().cache_need()
        if self.taps == 1:
            return pages
        return [pages, CacheNeed("state", state_shape=(self.channels * (self.taps - 1),))]

    def flops(self, tokens, keys_read=0.0):
        return (2.0 * tokens * (self.w_in.numel() + self.hidden * self.heads * self.val_dim)
                + 2.0 * self.heads * (self.key_dim + self.val_dim) * keys_read)

    def forward(self, ctx, xn, cache, sums=None):
        pages, inputs = (cache[0], cache[1]) if isinstance(cache, (list, tuple)) else (cache, None)
        if not pages.write:
            raise ValueError("attention_conv: the run writes its own cache")
        if sums is None:
            sums = K.Columns(decode_linear(ctx, xn, self.w_in, "attn.qkv", self._tiled.get("in")))
        n, dtype = sums.sums.shape[-2], self.runtime.dtype
        q = ctx.buf("attn.q", (n, self.q_dim), dtype)
        cos = sin = None
        if self.position is not None and hasattr(self.position, "tables"):
            cos, sin = self.position.tables(ctx)
        state, slots = (inputs.state, inputs.slots) if inputs is not None else (None, ctx.slots)
        K.qkv_conv_append(sums, self.conv, self.taps, state, 0, ctx.all_decode, q, pages.pages, ctx.positions,
                          ctx.span_of_token, slots, ctx.span_start, ctx.span_pos, pages.block_table, pages.page_size,
                          self.heads, self.kv_heads, self.key_dim, self.val_dim, self.width, cos=cos, sin=sin,
                          rotary_dim=self.rotary_dim, interleaved=self.interleaved, v_scale=self.out_scale)
        if self.taps > 1 and not ctx.all_decode:
            # (behind the launch that read the earlier inputs: the spans' last ones take their place)
            K.conv_state_update(sums.sums, sums.first, self.channels, self.taps, state, 0, slots, ctx.span_start,
                                ctx.span_pos, ctx.n_spans)
        out = ctx.buf("attn.out", (n, self.out_dim), dtype)
        self.attend(ctx, q, out, pages)
        return decode_linear(ctx, out, self.w_o, "attn.proj", self._tiled.get("o"))


@register_part("mixer", "attention_bias")
class BiasedAttention(CausalSelfAttention):
    """Attention whose projections have biases and whose output passes a gate: q = W_q h + b_q, k = W_k h
    + b_k, v = W_v h + b_v, no rotation; scores ((q . k) * ``scale``, less the distance bias), mask
    (``window``, ``chunk``), ``sink`` and the kernels are the base class's, and with ``sink``
    "learned" the softmax's extra term is exp of a number per head.  With ``gate`` the concatenated
    heads are multiplied element by element by the logistic function of W_g h, where attention's
    kernels write their output.  The output projection's bias is left to whoever adds the output to
    the stream (``out_bias``).  Values may have a width of their own.

    With ``own_kv`` False the part has no k and v: it reads the keys and values that another run cached.

    Pages hold one width for keys and values, the smallest that the kernels on the matrix cores take
    for both (the rest of a slot is zero); the output projection's columns are padded likewise.

    Parameters beyond the base class's: ``gate`` (default False).
    Tensors: ``<prefix>.{q,k,v,g,o}.weight``, ``.{q,k,v,o}.bias``, ``.sink`` [heads]."""
    takes_normed = False
    fills_sink = False
    learns_sinks = True
    pads_heads = True

    def __init__(self, spec, runtime):
        super().__init__(spec, runtime)
        if self.position is not None or self.keep_first:
            raise ValueError("attention_bias: takes no position part and keeps no first positions")
        self.gated = bool(self.param("gate", False))
        self._pad_heads()
        own = self.kv_heads if self.own_kv else 0
        self.rows = {"q": self.heads * self.key_dim}
        if own:
            self.rows.update(k=own * self.key_dim, v=own * self.val_dim)
        self.channels = sum(self.rows.values())
        self.gate_dim = self.heads * self.val_dim
        self.bias = self.out_bias = None

    def weight_specs(self):
        d, name = self.hidden, self.tensor_name
        specs = [WeightSpec(name(t + ".weight"), (n, d)) for t, n in self.rows.items()]
        specs += [WeightSpec(name(t + ".bias"), (n,), "vector") for t, n in self.rows.items()]
        if self.gated:
            specs.append(WeightSpec(name("g.weight"), (self.gate_dim, d)))
        if self.sink == "learned":
            specs.append(WeightSpec(name("sink"), (self.heads,), "vector"))
        return specs + [WeightSpec(name("o.weight"), (d, self.gate_dim)), WeightSpec(name("o.bias"), (d,), "vector")]

    def bind(self, weights):
        self._bind_slopes()
        w = lambda n: weights[self.tensor_name(n)]
        # one product for everything that reads the layer's input: queries | keys | values | gate
        self.w_in = torch.cat([w(t + ".weight") for t in [*self.rows] + (["g"] if self.gated else [])], dim=0).contiguous()
        self.bias = torch.cat([w(t + ".bias") for t in self.rows]).contiguous()
        if self.sink == "learned":
            self.sinks = w("sink")
        self.w_o, self.out_bias = self._padded_output(w("o.weight")), w("o.bias")
        # second copies for decode batches, in the order that kernel reads them
        self._tiled = {"in": tiled_copy(self.runtime, self.w_in, K.LINEAR_PARTS),
                       "o": tiled_copy(self.runtime, self.w_o, K.LINEAR_PARTS)}

    def flops(self, tokens, keys_read=0.0):
        return (2.0 * tokens * (self.w_in.numel() + self.hidden * self.gate_dim)
                + 2.0 * self.heads * (self.key_dim + self.val_dim) * keys_read)

    def forward(self, ctx, xn, cache):
        n = xn.shape[0]
        if self.own_kv != bool(cache.write):
            raise ValueError("attention_bias: a run must write its cache exactly when it has k and v projections")
        sums = decode_linear(ctx, xn, self.w_in, "attn.qkvg", self._tiled.get("in"))
        q = ctx.buf("attn.q", (n, self.q_dim), self.runtime.dtype)
        K.qkv_conv_append(K.Columns(sums, 0, self.channels), None, 1, None, 0, ctx.all_decode, q,
                          cache.pages if self.own_kv else None, ctx.positions, ctx.span_of_token, ctx.slots, ctx.span_start,
                          ctx.span_pos, cache.block_table, cache.page_size, self.heads, self.kv_heads if self.own_kv else 0,
                          self.key_dim, self.val_dim, self.width, bias=self.bias)
        out = ctx.buf("attn.out", (n, self.out_dim), self.runtime.dtype)
        self.attend(ctx, q, out, cache, gate=K.Columns(sums, self.channels, self.gate_dim) if self.gated else None)
        return decode_linear(ctx, out, self.w_o, "attn.proj", self._tiled.get("o"))
