"""Grouped-query causal attention over a paged cache: the token mixer of Qwen3.

Reference: ``jllm/model/common.py:114-137`` (projections, head layout, output
projection; the reference's projections have no bias, here ``qkv_bias`` and ``o_bias`` are options of the
part), ``:107-111`` (optional per-head q/k RMSNorm before the rotation),
``:173-214`` (scores, mask, softmax, kv head = q head // group).  The three input
projections are one matrix product against the row-concatenated weight; scores,
mask and softmax are float inside the attention kernels; keys are stored after
norm and rotation, values as projected (``jllm/engine/generate.py:54-59``).
"""
from __future__ import annotations

import math
from typing import Optional

import torch

from ..ops import kernels as K
from .spec import (LayerMemory, PagedCacheSpec, PartSpec, StateSpec, StepContext, TensorSpec, build_part, is_replayable,
                   kv_cache_spec, register_part)


FIRST_VALUES = "first_values"      # in ``StepContext.extras``: the step's values of the first layer that blends them


class GroupedQueryAttention:
    def __init__(self, hidden_size: int, num_heads: int, num_kv_heads: int, head_dim: int,
                 qk_norm_eps: Optional[float] = None, position: Optional[PartSpec] = None,
                 window: Optional[int] = None, scale: Optional[float] = None, qkv_bias: bool = False,
                 o_bias: bool = False, v_head_dim: Optional[int] = None, qk_norm: str = "head", v_scale: float = 1.0,
                 output_gate: bool = False, values_are_keys: bool = False, q_temperature: Optional[tuple] = None,
                 chunk: Optional[int] = None, filter_taps: Optional[int] = None, value_position: Optional[PartSpec] = None,
                 softmax_plus_one: bool = False, softcap: Optional[float] = None, keep_first: int = 0, sinks: bool = False,
                 qk_norm_weight: bool = True, value_blend: Optional[str] = None):
        """``v_head_dim``: a value size that differs from the key size; ``qk_norm`` "whole": the q/k norm spans all
        of q's (and all of k's) columns at once, with weights of that size, instead of every head on its own;
        ``v_scale``: a constant on the values (and so on the mixer's result before its output projection);
        ``output_gate``: the concatenated heads are multiplied by sigmoid(W_g x) before the output projection (W_g is
        one more block of rows of the fused input projection);
        ``values_are_keys``: there is no value projection, the values are the keys as projected (before their norm and
        rotation); ``q_temperature`` (coef, every): the query at position p is multiplied by
        1 + coef * ln(floor((p + 1) / every) + 1), after its norm;
        ``chunk``: a token sees the keys of its own block of ``chunk`` positions only (counted from position 0);
        ``filter_taps``: q, k and v as projected go through a causal filter over time per channel before the rotation,
        y_t = sum_j w[:, j] u_(t - taps + 1 + j) (the last taps - 1 projected rows are the request's state ``filter``);
        ``value_position``: a rotation of the whole value heads by their token's position, cached so, and every head's
        result turned back by the query's position (before the gate): the weighted sum sees the values at their
        distance from the query; ``softmax_plus_one``: one is added to the softmax denominator (a sink of score 0);
        ``softcap`` c: a scaled score s becomes c tanh(s / c); ``keep_first``: beside a window the first so many keys of the
        sequence stay in sight; ``sinks``: a learned number per q head whose exponential joins the softmax denominator (no
        key, no value, neither scaled nor capped); ``qk_norm_weight`` False: the per-head q/k norm has no weight (it is then
        the same before and behind the rotation, which keeps a head's length); ``value_blend`` "first": the layer's values
        are kept for the step; "later": the values become (1 - l) v + l v_first with v_first those of the same token and l a
        learned number, before they are cached.
        Any of these but ``chunk``, ``softmax_plus_one``, ``softcap``, ``keep_first`` and ``sinks`` takes the ``wide`` path (so does
        ``qkv_bias``, unless pairs (2i, 2i + 1) turn): heads cached
        under one padded size (``K.padded_head_dim``), prepared by ``K.attn_prepare_wide``, read by the same paged
        attention kernels."""
        if num_heads % num_kv_heads:
            raise ValueError(f"{num_heads} q heads are not a multiple of {num_kv_heads} kv heads")
        if qk_norm not in ("head", "whole"):
            raise ValueError(f"qk_norm is 'head' or 'whole', not {qk_norm!r}")
        self.hidden_size, self.nq, self.nkv = int(hidden_size), int(num_heads), int(num_kv_heads)
        self.dk = int(head_dim)
        self.dv = int(v_head_dim) if v_head_dim else self.dk
        self.qk_norm, self.v_scale = qk_norm, float(v_scale)
        self.output_gate = bool(output_gate)
        self.values_are_keys = bool(values_are_keys)
        self.q_temperature = (float(q_temperature[0]), int(q_temperature[1])) if q_temperature else None
        if self.q_temperature is not None and self.q_temperature[1] <= 0:
            raise ValueError("the period of a query temperature must be positive")
        if self.values_are_keys and (self.dv != self.dk or qkv_bias or (qk_norm == "whole" and qk_norm_eps is not None)):
            raise ValueError("values that are the keys: one head size, no input bias, a per-head q/k norm or none")
        self.chunk = int(chunk) if chunk else None
        if self.chunk and window:
            raise ValueError("a window or blocks, not both")
        self.taps = int(filter_taps) if filter_taps else 0
        self.plus_one = bool(softmax_plus_one)
        self.softcap = float(softcap) if softcap else None
        self.keep_first = int(keep_first or 0)
        if self.keep_first and not window:
            raise ValueError("kept first keys belong to a window")
        self.learned_sinks = bool(sinks)
        if self.plus_one and self.learned_sinks:
            raise ValueError("one is added to the denominator, or a learned sink, not both")
        self.qk_norm_weight = bool(qk_norm_weight)
        if not self.qk_norm_weight and qk_norm != "head":
            raise ValueError("a q/k norm without a weight is per head")
        if value_blend not in (None, "first", "later"):
            raise ValueError(f"value_blend is 'first' or 'later', not {value_blend!r}")
        self.value_blend = value_blend
        self.value_position = build_part("position", value_position) if value_position is not None else None
        self.filtered = bool(self.taps or self.value_position is not None)
        if self.filtered and (self.values_are_keys or self.q_temperature is not None or qk_norm_eps is not None or qkv_bias
                              or self.v_scale != 1.0):
            raise ValueError("filters and turned values: without a q/k norm, biases, values taken from the keys, a constant "
                             "on the values or a query temperature")
        if self.value_position is not None:
            turn = self.value_position.as_rotation()
            if turn is None or turn != (self.dv, True):
                raise ValueError("values turn whole, in pairs (2m, 2m + 1)")
        self.position = build_part("position", position) if position is not None else None
        # what the position part asks of this mixer's kernels: a rotation of q and k by position
        # (rotary_dim, interleaved), or nothing (a part that acts elsewhere, or no part at all)
        self.rotation = self.position.as_rotation() if self.position is not None else None
        self.wide = (self.filtered or self.values_are_keys or self.q_temperature is not None or self.dv != self.dk or (qk_norm == "whole" and qk_norm_eps is not None) or self.v_scale != 1.0
                     or self.output_gate or not self.qk_norm_weight or self.value_blend is not None
                     # biases are added where the heads are prepared; only pairs (2i, 2i + 1) need a pass of their own
                     or (bool(qkv_bias) and not (self.rotation is not None and self.rotation[1])))
        if self.value_blend is not None and (self.filtered or qkv_bias or values_are_keys or qk_norm == "whole"):
            raise ValueError("blended values: without filters, biases, values taken from the keys or a norm over the whole projection")
        # what the paged attention kernels see
        self.d = K.padded_head_dim(self.dk, self.dv) if self.wide else self.dk
        if self.wide:
            self.q_row_stride = self.nq * self.d
        self.qk_norm_eps = qk_norm_eps
        self.window = int(window) if window else None
        self.scale = float(scale) if scale is not None else 1.0 / math.sqrt(self.dk)
        if self.filtered and (self.dk % 2 or self.dv % 2 or (self.rotation is not None and not self.rotation[1])):
            raise ValueError("the filtered attention input takes even head sizes and turns pairs (2i, 2i + 1)")
        self.qkv_bias, self.o_bias = bool(qkv_bias), bool(o_bias)
        self.w_qkv = self.w_o = self.q_norm = self.k_norm = self.b_qkv = self.b_o = self.sinks = None

    # ---- declarations
    @property
    def replayable(self) -> bool:
        """The kernels take positions, lengths and tables from the device; the host plan of a
        captured step (how many blocks share a request's keys) is made for the upper bound of
        the context lengths and is right for every shorter one."""
        return all(part is None or is_replayable(part) for part in (self.position, self.value_position))

    def tensors(self) -> dict:
        t = {
            "q_proj.weight": TensorSpec((self.nq * self.dk, self.hidden_size)),
            "k_proj.weight": TensorSpec((self.nkv * self.dk, self.hidden_size)),
            "v_proj.weight": TensorSpec((self.nkv * self.dv, self.hidden_size)),
            "o_proj.weight": TensorSpec((self.hidden_size, self.nq * self.dv)),
        }
        if self.values_are_keys:
            del t["v_proj.weight"]
        if self.qk_norm_eps is not None and self.qk_norm_weight:
            whole = self.qk_norm == "whole"
            t["q_norm.weight"] = TensorSpec((self.nq * self.dk if whole else self.dk,), role="vector", init="norm")
            t["k_norm.weight"] = TensorSpec((self.nkv * self.dk if whole else self.dk,), role="vector", init="norm")
        if self.qkv_bias:
            t["q_proj.bias"] = TensorSpec((self.nq * self.dk,), role="vector")
            t["k_proj.bias"] = TensorSpec((self.nkv * self.dk,), role="vector")
            t["v_proj.bias"] = TensorSpec((self.nkv * self.dv,), role="vector")
        if self.o_bias:
            t["o_proj.bias"] = TensorSpec((self.hidden_size,), role="vector")
        if self.output_gate:
            t["gate.weight"] = TensorSpec((self.nq * self.dv, self.hidden_size))
        if self.learned_sinks:
            t["sinks"] = TensorSpec((self.nq,), role="vector", init="small")
        if self.value_blend is not None:      # stored in every blending layer, the first one's has no effect
            t["value_blend"] = TensorSpec((), role="vector", init="fraction")
        if self.taps:
            t["q_filter.weight"] = TensorSpec((self.nq * self.dk, self.taps), role="vector")
            t["k_filter.weight"] = TensorSpec((self.nkv * self.dk, self.taps), role="vector")
            t["v_filter.weight"] = TensorSpec((self.nkv * self.dv, self.taps), role="vector")
        return t

    def cache_spec(self) -> Optional[PagedCacheSpec]:
        return kv_cache_spec(self.nkv, self.d, self.window, self.chunk, self.keep_first)

    def state_spec(self):
        if not self.taps:
            return None
        return StateSpec((self.taps - 1, self.nq * self.dk + self.nkv * (self.dk + self.dv)), "float32", "filter")

    def bind(self, tensors: dict, dtype: torch.dtype) -> None:
        self.dtype = dtype
        # one product for everything that reads the input: q, k, v and, behind them, the gate's rows
        blocks = [tensors["q_proj.weight"], tensors["k_proj.weight"]]
        if not self.values_are_keys:
            blocks.append(tensors["v_proj.weight"])
        if self.output_gate:
            blocks.append(tensors["gate.weight"])
        rows = sum(b.shape[0] for b in blocks)
        if self.wide and rows % 8:      # rows of the product stay 16-byte aligned for the kernels that read heads out of them
            blocks.append(blocks[0].new_zeros((8 - rows % 8, self.hidden_size)))
        self.w_qkv = torch.cat(blocks, dim=0).contiguous()
        self.filters = (torch.cat([tensors[f"{s}_filter.weight"] for s in "qkv"], dim=0).t().contiguous()
                        if self.taps else None)       # [taps, channels]
        self.sinks = torch.zeros((self.nq,), dtype=torch.float32, device=self.w_qkv.device) if self.plus_one else None
        if self.learned_sinks:
            self.sinks = tensors["sinks"].contiguous()
        self.blend = float(tensors["value_blend"].reshape(())) if self.value_blend is not None else 0.0
        self.qkv_width = self.nq * self.dk + self.nkv * (self.dk + (0 if self.values_are_keys else self.dv))
        self.w_o = tensors["o_proj.weight"]
        if self.wide and self.d != self.dv:
            # the attention's result has heads of the padded size (zeros behind the values): zero columns there
            w = self.w_o.new_zeros((self.hidden_size, self.nq, self.d))
            w[:, :, :self.dv] = self.w_o.view(self.hidden_size, self.nq, self.dv)
            self.w_o = w.view(self.hidden_size, self.nq * self.d).contiguous()
        if self.qk_norm_eps is not None and self.qk_norm_weight:
            self.q_norm, self.k_norm = tensors["q_norm.weight"], tensors["k_norm.weight"]
        elif self.qk_norm_eps is not None:
            self.q_norm = self.k_norm = torch.ones((self.dk,), dtype=torch.float32, device=self.w_qkv.device)
        if self.qkv_bias:
            self.b_qkv = torch.cat([tensors["q_proj.bias"], tensors["k_proj.bias"], tensors["v_proj.bias"]]).contiguous()
        if self.o_bias:
            self.b_o = tensors["o_proj.bias"].contiguous()
        if self.position is not None:
            self.position.bind({}, dtype, self.w_o.device)
        if self.value_position is not None:
            self.value_position.bind({}, dtype, self.w_o.device)

    def _qkv_parts_ok(self) -> bool:
        """Whether the kernel behind the qkv product (norm, rotation, page write) adds float partial
        products itself: decided by sizes and the declared rotation alone, so the same answer holds
        when the norm before asks and when the product runs."""
        if self.wide:
            return False
        rotary_dim, interleaved = self.rotation if self.rotation is not None else (0, False)
        return K.rope_takes_parts(self.dtype, self.d, interleaved, rotary_dim, self.rotation is not None)

    def takes_unscaled_rows(self, n_rows: int) -> bool:
        """x goes into the qkv product and nowhere else: the norm before may leave its scale to that product."""
        return K.linear_takes_unscaled_rows(n_rows, self.w_qkv, partial_ok=self._qkv_parts_ok(), partial_max_width=None)

    # ---- one product with what else reads the same input (``parts/recurrent.py: ParallelMixer``)
    def input_weight(self):
        """The matrix of the one product this mixer begins with, or None where it has to make that product itself."""
        return self.w_qkv if self.wide and not self.filtered else None

    def share_input(self, weight: torch.Tensor) -> None:
        self.w_qkv = weight

    def forward_projected(self, proj, at: int, ctx: StepContext, mem: LayerMemory) -> torch.Tensor:
        """The rest of the mixer behind its input product, whose columns begin at ``at`` (0: the heads are read from the
        rows' beginning)."""
        if at:
            raise ValueError("the attention's heads begin its rows")
        return self._forward_wide(proj, ctx, mem)

    # ---- one step
    def forward(self, x, ctx: StepContext, mem: LayerMemory) -> torch.Tensor:
        n = x.shape[0]
        if self.wide and not self.filtered:
            return self._forward_wide(K.linear(x, self.w_qkv), ctx, mem)
        rotary_dim, interleaved = self.rotation if self.rotation is not None else (0, False)
        cos_sin = self.position.rotation_table(ctx) if self.rotation is not None else None
        # at few rows the projection may come as float partial products, which the next kernel adds
        qkv = K.linear(x, self.w_qkv, partial_max_width=None,       # the rotation kernel adds parts of any width
                       partial_ok=self._qkv_parts_ok())
        if self.filtered:
            return self._forward_filtered(qkv, ctx, mem, cos_sin, rotary_dim)
        if self.b_qkv is not None:
            K.add_bias(qkv, self.b_qkv)
        parts = None
        if qkv.dim() == 3:
            parts, qkv = qkv, torch.empty(qkv.shape[1:], dtype=x.dtype, device=x.device)
        writes = mem.writes
        K.qk_norm_rope_write(
            qkv, ctx.slot_mappings[mem.group] if writes else None, self.q_norm, self.k_norm,
            self.qk_norm_eps or 0.0, cos_sin, rotary_dim, interleaved,
            mem.pages["k"] if writes else None, mem.pages["v"] if writes else None, ctx.page_size,
            self.nq, self.nkv, self.d, parts=parts,
        )
        out = torch.empty((n, self.nq * self.d), dtype=x.dtype, device=x.device)
        from . import attention_backend

        attention_backend.run(self, out, qkv, ctx, mem)
        y = K.linear(out, self.w_o, partial_ok=True)      # the next norm adds the partial products
        if self.b_o is not None:
            K.add_bias(y, self.b_o)
        return y


    def _forward_filtered(self, qkv, ctx: StepContext, mem: LayerMemory, cos_sin, rotary_dim: int):
        if not mem.writes:
            raise ValueError("filtered heads write the cache they declare")
        v_turn = self.value_position.rotation_table(ctx) if self.value_position is not None else None
        q = K.attn_prepare_filtered(
            qkv, self.filters, mem.states.get("filter"), ctx.slot_ids, ctx.cu_seqlens, ctx.context_lens, ctx.max_q_len, cos_sin,
            rotary_dim, v_turn, ctx.slot_mappings[mem.group], mem.pages["k"], mem.pages["v"], ctx.page_size, self.nq, self.nkv,
            self.dk, self.dv, self.d)
        out = torch.empty((qkv.shape[0], self.nq * self.d), dtype=qkv.dtype, device=qkv.device)
        from . import attention_backend

        attention_backend.run(self, out, q, ctx, mem)
        gate = qkv[:, self.qkv_width:self.qkv_width + self.nq * self.dv] if self.output_gate else None
        if v_turn is not None or gate is not None:
            K.rotate_back_gate(out, gate, v_turn, self.nq, self.dv, self.d)
        y = K.linear(out, self.w_o, partial_ok=True)
        if self.b_o is not None:
            K.add_bias(y, self.b_o)
        return y

    def _forward_wide(self, qkv, ctx: StepContext, mem: LayerMemory):
        rotary_dim, interleaved = self.rotation if self.rotation is not None else (0, False)
        cos_sin = self.position.rotation_table(ctx) if self.rotation is not None else None
        if interleaved:
            raise ValueError("heads of two sizes and a norm over the whole projection rotate half-split pairs only")
        writes = mem.writes
        values = None
        if self.value_blend is not None:
            at = (self.nq + self.nkv) * self.dk
            own = qkv[:, at:at + self.nkv * self.dv]
            if self.value_blend == "first":
                ctx.extras[FIRST_VALUES] = own
            else:
                values = ctx.extras.get(FIRST_VALUES)
                if values is None:
                    raise ValueError("values are blended with those of an earlier layer, and none kept them")
        q = K.attn_prepare_wide(
            qkv, self.b_qkv, self.q_norm, self.k_norm, self.qk_norm_eps or 0.0, cos_sin, rotary_dim,
            ctx.slot_mappings[mem.group] if writes else None, mem.pages["k"] if writes else None,
            mem.pages["v"] if writes else None, ctx.page_size, self.nq, self.nkv, self.dk, self.dv, self.d, self.v_scale,
            norm_per_head=self.qk_norm == "head", values_are_keys=self.values_are_keys,
            positions=ctx.positions if self.q_temperature is not None else None, q_temperature=self.q_temperature,
            v_first=values, v_mix=self.blend)
        out = torch.empty((qkv.shape[0], self.nq * self.d), dtype=qkv.dtype, device=qkv.device)
        from . import attention_backend

        attention_backend.run(self, out, q, ctx, mem)
        if self.output_gate:
            K.sigmoid_gate_heads(out, qkv[:, self.qkv_width:self.qkv_width + self.nq * self.dv], self.nq, self.dv, self.d)
        y = K.linear(out, self.w_o, partial_ok=True)
        if self.b_o is not None:
            K.add_bias(y, self.b_o)
        return y


register_part("mixer", "gqa_attention", GroupedQueryAttention)
