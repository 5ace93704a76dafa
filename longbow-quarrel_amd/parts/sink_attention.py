"""Attention over a sliding window that also keeps the first tokens of the sequence, with a sink.

q = h Wq^T, k = h Wk^T, v = h Wv^T without biases; keys are `key_dim` wide, values `value_dim` (they may
differ); query head h reads kv head h // (heads / kv_heads).  Position i sees position j when j <= i and
(i - j < window or j < keep_first); window = 0 means every earlier position.  With `sink` the softmax has one
more term in its denominator, a key of score 0 that carries no value: p_j = e^(s_j) / (1 + sum e^(s_j)), so a
query may look at nothing (Xiao, Tian, Chen, Han, Lewis: "Efficient Streaming Language Models with Attention
Sinks" keeps first tokens for the same purpose).  `sink="learned"`: the term is e^(b_h) with a stored number b_h for
every query head (`<prefix>.sink`), which is not scaled: p_j = e^(s_j) / (e^(b_h) + sum e^(s_j)).  With `head_gate` every head's result is multiplied by the
sigmoid of one more projection of h, a number per head.  Scores, probabilities and the sums over values are
32-bit whatever the run's dtype.  A position encoding is optional (`position=None`: positions do not enter
the scores).

`rotary` (a mapping: `dims`, `base`, optionally `scaling` as `rope.rotary_frequencies` takes it and `pairing`,
"interleaved" or "half") rotates the first `dims` entries of every query and key head by the position, the rest
pass; `qk_norm_eps` then divides every query and key head by its root mean square over key_dim (no weight).  Both
are taken in 32-bit on the product's 32-bit result, by one kernel that also leaves q, k and v in the dtype of the
cache.

`chunk` = c: position i sees only the keys of its own run of c positions, floor(i / c) = floor(j / c), counted from the
start of the sequence.

`probabilities="bfloat16"` says that a design lets the softmax's weights be rounded to bfloat16 as operands of their
product with the values (the sums stay 32-bit): plain causal attention with keys and values of one size then runs, in
a bfloat16 run, on the causal kernel of the matrix cores, several times as fast over a prompt.  The default keeps the
weights 32-bit through that product.

What a design may ask for beside these, each with a parameter (none of the first five together with `qk_norm_eps`):
* `qkv_bias`: biases on q, k and v (`<name>.b`); `out_bias`: one on the output projection (`<prefix>.o.b`).
* `qk_norm` "head" or "row": RMS norm with a weight (`<prefix>.q.norm`, `<prefix>.k.norm`) on every head of q and k (the
  weight is shared by the heads), or on all heads' entries of a row together; "unit": every head of q and k divided by
  its root mean square, no weight; `value_norm`: every value head divided by its root mean square, without a weight.
  `norm_eps` for all of them.
* `values_from_keys`: there is no Wv, the values are the keys as projected (with their bias, before rotation and norm).
* `rotary` together with any of these: the rotation comes after the bias and before the norm (not with "row").
* `temperature`: a stored number a head (`<prefix>.temp`) multiplies the scaled score; `softcap`: score <- softcap
  tanh(score / softcap) (0: not).
* `log_bias`: r1_h ln(1 + r2_h n) is taken off the score of a key n positions back (`<prefix>.r1`, `.r2`, a number a
  head); `table_bias` (`rows`, `most`): a learned number for the distance's row of a table and the head is added
  (`<prefix>.rel` [rows, heads], rows by `distance_rows`).
* `entry_gate`: every entry of the heads' result times the sigmoid of one more projection of h (`<prefix>.g`, a row an
  entry).
Biases, rotation, norms and the store into the cache are one kernel (`qkv_norm_store`) on the product's 32-bit result; what
shapes a score and the gate are inside the attention kernel.

All projections of h are one matrix product ([q | k | v | gate]).
"""
from __future__ import annotations

import math
from typing import Dict, List, Mapping, Optional

import torch

from .base import (MIXERS, POSITION_ENCODINGS, VECTOR32, BuildEnv, KVNeed, LayerCache, Mixer, PartSpec, StepContext,
                   TensorSpec, build_part, product_weight, project)
from .rope import rotary_frequencies, rotary_magnitude, step_angles


def split_scratch(ctx: StepContext, dtype, heads: int, kv_heads: int, key_dim: int, value_dim: int, block_size: int,
                  window: int, keep_first: int, chunk: int = 0) -> Dict[str, object]:
    """The keywords with which `sink_attention` may share a decoding step's keys out over several workgroups a tile:
    the step's bound of the lengths and the scratch that the kernel object asks for (nothing where it asks for none)."""
    ask = getattr(ctx.kernels, "sink_attention_workspace", None)
    if ask is None or not ctx.decode:
        return {}
    need = ask(dtype, ctx.rows, ctx.batch, heads, kv_heads, key_dim, value_dim, block_size, window, keep_first, ctx.max_len,
               **({"chunk": chunk} if chunk else {}))
    return dict(max_len=ctx.max_len, workspace=ctx.ws.alloc((need,), torch.float32)) if need else {}


def distance_rows(rows: int, most: float, window: int = 0) -> List[int]:
    """The row of a `rows`-row table for the distances 0, 1, ...: a distance below half = rows // 2 has a row of its own,
    a farther one shares half + floor(ln(n / half) / ln(most / half) (rows - half)), at most the last row.  The list
    ends where every farther distance has the last row, or with the farthest distance that a window shows."""
    half = rows // 2
    if rows < 2 or not most > half:
        raise ValueError(f"a table of {rows} rows cannot end at a distance of {most}")
    out: List[int] = []
    while (not window or len(out) < window) and (not out or out[-1] < rows - 1):
        n = len(out)
        # (an exact step, which rounding may leave just below its whole number, counts as reached)
        out.append(n if n < half else
                   min(rows - 1, half + math.floor(math.log(n / half) / math.log(most / half) * (rows - half) + 1e-9)))
    return out


@MIXERS.register("sink_window_attention")
class SinkWindowAttention(Mixer):
    takes_out = True

    def __init__(self, width: int, heads: int, kv_heads: int, key_dim: int, value_dim: int, scale: float,
                 prefix: str, window: int = 0, keep_first: int = 0, sink=True, head_gate: bool = False,
                 position: Optional[PartSpec] = None, rotary: Optional[Mapping] = None,
                 qk_norm_eps: Optional[float] = None, names: Optional[Mapping[str, str]] = None,
                 probabilities: str = "float32", qkv_bias: bool = False, out_bias: bool = False,
                 qk_norm: Optional[str] = None, value_norm: bool = False, norm_eps: float = 0.0,
                 values_from_keys: bool = False, temperature: bool = False, softcap: float = 0.0, log_bias: bool = False,
                 table_bias: Optional[Mapping] = None, entry_gate: bool = False, chunk: int = 0) -> None:
        if heads % kv_heads != 0:
            raise ValueError(f"{heads} heads cannot share {kv_heads} kv heads evenly")
        self.rot_dims, self.rot_interleaved, self.rot_magnitude, self.freq_table = 0, False, 1.0, []
        if rotary is not None:
            if position is not None:
                raise ValueError("a position encoding part or the `rotary` parameters, not both")
            self.rot_dims = int(rotary["dims"])
            pairing = rotary.get("pairing", "interleaved")
            if pairing not in ("half", "interleaved"):
                raise ValueError(f"rotary pairing {pairing!r} is not known (known: 'half', 'interleaved')")
            if self.rot_dims % 2 or not 2 <= self.rot_dims <= int(key_dim):
                raise ValueError(f"{self.rot_dims} rotated entries do not fit a head of {key_dim}")
            scaling = dict(rotary["scaling"]) if rotary.get("scaling") else None
            self.rot_interleaved = pairing == "interleaved"
            self.freq_table = rotary_frequencies(self.rot_dims, float(rotary["base"]), scaling)
            self.rot_magnitude = rotary_magnitude(scaling)
        self.qk_norm_eps = None if qk_norm_eps is None else float(qk_norm_eps)
        if (rotary is not None or qk_norm_eps is not None) and head_gate:
            raise ValueError("a gate per head and a rotation or norm of q and k are not combined")
        if qk_norm not in (None, "head", "row", "unit"):
            raise ValueError(f"q and k are normed by 'head', 'row' or 'unit' (or not: None), found {qk_norm!r}")
        self.qkv_bias, self.has_out_bias, self.qk_norm, self.value_norm = bool(qkv_bias), bool(out_bias), qk_norm, bool(value_norm)
        self.norm_eps, self.values_from_keys, self.temperature = float(norm_eps), bool(values_from_keys), bool(temperature)
        self.softcap, self.log_bias, self.entry_gate = float(softcap), bool(log_bias), bool(entry_gate)
        self.table_bias = None if table_bias is None else (int(table_bias["rows"]), float(table_bias["most"]))
        self.stored = bool(qkv_bias or qk_norm or value_norm or values_from_keys or entry_gate)  # by `qkv_norm_store`
        self.shaped = bool(temperature or softcap or log_bias or table_bias is not None or entry_gate)
        if self.stored and (qk_norm_eps is not None or position is not None or head_gate):
            raise ValueError("biases, weighted norms, values from keys or a gate an entry are not combined with a position "
                             "part, `qk_norm_eps` or a gate a head")
        if rotary is not None and qk_norm == "row":
            raise ValueError("a norm over all heads of a row together is not combined with a rotation ahead of it")
        # without any of those, q, k and v pass the kernel that rotates and norms them (`rotary_qkv`)
        self.prepared = not self.stored and (rotary is not None or qk_norm_eps is not None)
        if self.values_from_keys and key_dim != value_dim:
            raise ValueError(f"values that are the keys are as wide as they are ({key_dim}, {value_dim})")
        if self.softcap < 0:
            raise ValueError("the cap on the scores must not be negative")
        if window < 0 or keep_first < 0 or chunk < 0:
            raise ValueError("window, keep_first and chunk must not be negative")
        if chunk and keep_first:
            raise ValueError("chunks keep no first tokens")
        self.chunk = int(chunk)
        self.width, self.heads, self.kv_heads = int(width), int(heads), int(kv_heads)
        self.key_dim, self.value_dim = int(key_dim), int(value_dim)
        self.scale, self.window, self.keep_first = float(scale), int(window), int(keep_first)
        if sink not in (True, False, "learned"):
            raise ValueError(f"the sink is True (a score of 0), False or 'learned' (a stored score a head), found {sink!r}")
        self.sink, self.head_gate, self.learned_sink = bool(sink), bool(head_gate), sink == "learned"
        self.sink_w: Optional[torch.Tensor] = None
        if probabilities not in ("float32", "bfloat16"):
            raise ValueError(f"probabilities are 'float32' or 'bfloat16', found {probabilities!r}")
        self.probabilities = probabilities
        n = {"q": "q", "k": "k", "v": "v", "gate": "g", "o": "o", "sink": "sink", "q_norm": "q.norm", "k_norm": "k.norm",
             "temp": "temp", "r1": "r1", "r2": "r2", "rel": "rel"}
        n.update(names or {})
        self.names: Dict[str, str] = {key: f"{prefix}.{val}" for key, val in n.items()}
        self.position = build_part(POSITION_ENCODINGS, position) if position is not None else None
        self.q_width = self.heads * self.key_dim
        self.k_width = self.kv_heads * self.key_dim
        self.v_width = self.kv_heads * self.value_dim
        self.o_width = self.heads * self.value_dim
        self.w_in: Optional[torch.Tensor] = None
        self.w_o: Optional[torch.Tensor] = None

    @property
    def graph_safe(self) -> bool:
        return self.position is None or self.position.graph_safe

    def _projections(self):
        """The projections of h, in the order of their one product: (key of the name, rows)."""
        return [("q", self.q_width), ("k", self.k_width)] + \
            ([] if self.values_from_keys else [("v", self.v_width)]) + \
            ([("gate", self.heads)] if self.head_gate else [("gate", self.o_width)] if self.entry_gate else [])

    def tensor_specs(self) -> List[TensorSpec]:
        nm = self.names
        specs = []
        for key, width in self._projections():
            specs.append(TensorSpec(nm[key], (width, self.width)))
            if self.qkv_bias and key != "gate":
                specs.append(TensorSpec(nm[key] + ".b", (width,), kind=VECTOR32))
        if self.qk_norm in ("head", "row"):
            whole = self.qk_norm == "row"
            specs += [TensorSpec(nm["q_norm"], (self.q_width if whole else self.key_dim,), kind=VECTOR32, init="around_one"),
                      TensorSpec(nm["k_norm"], (self.k_width if whole else self.key_dim,), kind=VECTOR32, init="around_one")]
        for key in (["temp"] if self.temperature else []) + (["r1", "r2"] if self.log_bias else []):
            specs.append(TensorSpec(nm[key], (self.heads,), kind=VECTOR32, init="around_one"))
        if self.table_bias is not None:
            specs.append(TensorSpec(nm["rel"], (self.table_bias[0], self.heads), kind=VECTOR32))
        if self.has_out_bias:
            specs.append(TensorSpec(nm["o"] + ".b", (self.width,), kind=VECTOR32))
        if self.learned_sink:
            specs.append(TensorSpec(self.names["sink"], (self.heads,), kind=VECTOR32))
        specs.append(TensorSpec(self.names["o"], (self.width, self.o_width)))
        return specs + (self.position.tensor_specs() if self.position is not None else [])

    def bind(self, tensors: Mapping[str, torch.Tensor], env: BuildEnv) -> None:
        super().bind(tensors, env)
        nm = self.names
        mats = [tensors[nm[key]] for key, _ in self._projections()]
        if len({m.dtype for m in mats}) != 1:
            raise ValueError(f"{self.names['q']}: the projections of one input are stored in different dtypes")
        self.w_in = product_weight(env, torch.cat(mats, dim=0))
        self.w_o = product_weight(env, tensors[self.names["o"]])
        if self.learned_sink:
            self.sink_w = tensors[self.names["sink"]].contiguous()
        get = lambda key, there: tensors[nm[key]].contiguous() if there else None
        weighted = self.qk_norm in ("head", "row")
        self.q_norm_w, self.k_norm_w = get("q_norm", weighted), get("k_norm", weighted)
        self.in_bias = torch.cat([tensors[nm[key] + ".b"] for key, _ in self._projections() if key != "gate"]).contiguous() \
            if self.qkv_bias else None
        self.out_bias = tensors[nm["o"] + ".b"].contiguous() if self.has_out_bias else None
        self.shape_kw: Dict[str, object] = {}  # how `sink_attention` shapes the scores
        if self.softcap:
            self.shape_kw["softcap"] = self.softcap
        if self.temperature:
            self.shape_kw["temp"] = get("temp", True)
        if self.log_bias:
            self.shape_kw["log_bias"] = (get("r1", True), get("r2", True))
        if self.table_bias is not None:  # looked up by distance: one number a head and distance
            rows = torch.tensor(distance_rows(*self.table_bias, self.window), device=tensors[nm["rel"]].device)
            self.shape_kw["distance_bias"] = tensors[nm["rel"]].index_select(0, rows).t().contiguous()
        if self.position is not None:
            self.position.bind(tensors, env)
        self.freqs = torch.tensor(self.freq_table, dtype=torch.float64, device=env.device) if self.rot_dims else None

    def cache_need(self) -> KVNeed:
        # a window that keeps first tokens still gives its middle blocks back
        return KVNeed(self.kv_heads, self.key_dim, self.window, self.value_dim, self.keep_first if self.window else 0,
                      self.chunk)

    def lengths_uneven(self, kernels, lengths) -> bool:
        ask = getattr(kernels, "decode_lengths_uneven", None)
        plain = not (self.sink or self.head_gate or self.keep_first or self.window or self.chunk or self.shaped) and self.key_dim == self.value_dim \
            and self.probabilities == "bfloat16"
        return bool(ask(lengths)) if ask is not None and plain else False

    def _plain_causal(self, kn, ctx: StepContext, cache: LayerCache) -> bool:
        """Whether this step's attention is the causal kernel's (`attention`): the design lets the probabilities be
        rounded to bfloat16 for their product with the values (that kernel's way; the general kernel keeps them
        32-bit), the mask and softmax are plain, and the kernel object runs the shape on its matrix cores."""
        if self.probabilities != "bfloat16" or self.sink or self.head_gate or self.keep_first or self.chunk or self.shaped \
                or self.key_dim != self.value_dim:
            return False
        ask = getattr(kn, "attention_on_matrix_cores", None)
        return ask is not None and bool(ask(ctx.dtype, self.heads, self.kv_heads, self.key_dim, cache.block_size))

    def forward(self, h: torch.Tensor, ctx: StepContext, cache: Optional[LayerCache],
                out: Optional[torch.Tensor] = None, leave_bias: bool = False) -> torch.Tensor:
        if cache is None or cache.k is None:
            raise RuntimeError("attention needs a key/value cache")
        kn = ctx.kernels
        rows = h.shape[0]
        total = sum(n for _, n in self._projections())
        total_padded = (total + 3) // 4 * 4  # rows of the product start on 16 bytes
        wide_gate = None
        if self.stored:
            # biases and norms are taken on the product's 32-bit result; keys and values go straight into the cache
            proj = ctx.ws.alloc((rows, total_padded), torch.float32)[:, :total]
            project(kn, ctx, h, self.w_in, proj)
            q, k, v, gate = ctx.ws.alloc((rows, self.q_width), ctx.dtype), None, None, None
            n_qkv = total - (self.o_width if self.entry_gate else 0)
            place = dict(row_pos=ctx.row_pos, row_seq=ctx.row_seq, seq_slot=ctx.seq_slot, block_table=cache.block_table,
                         kcache=cache.k, vcache=cache.v, block_size=cache.block_size) if cache.write else {}
            if self.rot_dims:
                place.update(cos_sin=step_angles(ctx, self.freqs, self.freq_table), interleaved=self.rot_interleaved,
                             magnitude=self.rot_magnitude)
            kn.qkv_norm_store(proj[:, :n_qkv], q, self.heads, self.kv_heads, self.key_dim, self.value_dim, self.norm_eps,
                              bias=self.in_bias, q_weight=self.q_norm_w, k_weight=self.k_norm_w,
                              norm_qk="head" if self.qk_norm == "unit" else self.qk_norm,
                              norm_v=self.value_norm, v_from_k=self.values_from_keys, **place)
            wide_gate = proj[:, n_qkv:] if self.entry_gate else None
        elif self.prepared:
            # the product's 32-bit result is rotated and normed in 32-bit, then rounded to what the cache holds
            proj = ctx.ws.alloc((rows, total_padded), torch.float32)[:, :total]
            project(kn, ctx, h, self.w_in, proj)
            q = ctx.ws.alloc((rows, self.q_width), ctx.dtype)
            k = ctx.ws.alloc((rows, self.k_width), ctx.dtype)
            v = ctx.ws.alloc((rows, self.v_width), ctx.dtype)
            gate = None
            kn.rotary_qkv(proj, q, k, v, self.heads, self.kv_heads, self.key_dim, self.value_dim, self.rot_dims,
                          self.rot_interleaved, self.freqs, self.rot_magnitude, self.qk_norm_eps, ctx.row_pos)
        else:
            # q, k and v in the run's dtype (what the cache holds); the gate's logits ride in the same product
            proj = ctx.ws.alloc((rows, total_padded), ctx.dtype)[:, :total]
            project(kn, ctx, h, self.w_in, proj)
            q = proj[:, : self.q_width]
            k = proj[:, self.q_width : self.q_width + self.k_width]
            v = proj[:, self.q_width + self.k_width : self.q_width + self.k_width + self.v_width]
            gate = proj[:, self.q_width + self.k_width + self.v_width :] if self.head_gate else None
            if self.position is not None:
                self.position.apply(q, k, ctx)
        if cache.write and k is not None:
            kn.kv_store(k, v, self.kv_heads, self.key_dim, self.value_dim, ctx.row_pos, ctx.row_seq, ctx.seq_slot,
                        cache.block_table, cache.k, cache.v, cache.block_size)
        att = ctx.ws.alloc((rows, self.o_width), ctx.dtype)
        if self._plain_causal(kn, ctx, cache):
            # no sink, gate or kept first tokens, keys and values of one size: the causal kernel on the matrix cores
            need = kn.attention_workspace(ctx.dtype, rows, self.heads, self.kv_heads, self.key_dim, cache.block_size,
                                          ctx.decode, ctx.max_len)
            kn.attention(q, att, self.heads, self.kv_heads, self.key_dim, ctx.row_pos, ctx.row_seq, ctx.seq_slot,
                         ctx.cu_rows, cache.block_table, cache.k, cache.v, cache.block_size, self.scale, self.window,
                         decode=ctx.decode, max_len=ctx.max_len,
                         workspace=ctx.ws.alloc((need,), torch.float32) if need else None, uneven=ctx.uneven)
            return self._project_out(ctx, att, out, leave_bias)
        kn.sink_attention(q, att, self.heads, self.kv_heads, self.key_dim, self.value_dim, ctx.row_pos, ctx.row_seq,
                          ctx.seq_slot, cache.block_table, cache.k, cache.v, cache.block_size, self.scale,
                          window=self.window, keep_first=self.keep_first, sink=self.sink, gate=gate,
                          decode=ctx.decode, **self.shape_kw, **({"wide_gate": wide_gate} if wide_gate is not None else {}),
                          **({"sink_values": self.sink_w} if self.learned_sink else {}),
                          **({"chunk": self.chunk} if self.chunk else {}),
                          **split_scratch(ctx, q.dtype, self.heads, self.kv_heads, self.key_dim, self.value_dim,
                                          cache.block_size, self.window, self.keep_first, self.chunk))
        return self._project_out(ctx, att, out, leave_bias)

    def _project_out(self, ctx: StepContext, att: torch.Tensor, out: Optional[torch.Tensor], leave_bias: bool) -> torch.Tensor:
        if out is None:
            out = ctx.ws.alloc((att.shape[0], self.width), torch.float32)
        project(ctx.kernels, ctx, att, self.w_o, out)
        if self.out_bias is not None and not leave_bias:
            ctx.kernels.add_bias(out, self.out_bias)
        return out
