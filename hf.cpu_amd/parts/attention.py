"""Softmax attention over a paged key/value cache, with grouped heads and an
optional window."""
import math

import torch

from .. import memory

from ..registry import make_part, register_part
from ..status import EINVAL, fail
from .base import FixedState, PagedKV, ParamSpec, Part


@register_part("mixer", "attention")
class Attention(Part):
    """``q = Wq h + bq`` etc. (src/model.c:581-585); position encoding on q and k;
    for query head ``h`` the key/value head is ``h / (heads / kv_heads)``; scores
    ``dot(q, k) * scale`` over the visible keys, softmax in fp32, weighted sum of
    values (src/model.c:499-528); ``x += Wo att`` (src/model.c:606-609).

    A key at ``pk`` is visible to a query at ``pq`` iff ``0 <= pq - pk`` and, when
    ``window > 0``, ``pq - pk < window``, and, when ``mask_chunk > 0``, ``pq // mask_chunk == pk // mask_chunk``
    (runs of ``mask_chunk`` positions counted from the start of the sequence, wherever a prompt was cut).

    ``own_kv=False``: the mixer has no key and value projections and no cache of its own; the plan's schedule lets
    its entry read an earlier entry's cache (``ScheduleEntry.cache_of``), with its own queries, scale and mask.

    ``names`` gives the tensors' names after ``prefix`` (keys q, k, v, o, and q_bias, k_bias, v_bias, o_bias).

    A position encoding that enters the scores instead of the queries and keys has an
    attribute ``score_slopes`` (fp32 on the device, one per query head): the score then is
    ``dot(q, k) * scale + score_slopes[h] * (pk - pq)``.

    ``qk_norm`` = eps: queries and keys are RMS-normed over the whole projection (all heads at once) with the weights
    ``q_norm`` and ``k_norm`` (names in ``names``), before the rotation. ``sink``: the softmax has one more term of score 0
    that has no value, ``p_j = exp(s_j) / (1 + sum exp(s_i))``. ``v_mix``: ``"first"``: this layer's values, as projected,
    are kept for the step; ``"blend"``: ``v <- (1 - l) v + l v_first`` with the scalar tensor ``v_mix`` (name in
    ``names``) and the kept values of the same token; the blended values are what is cached. A ``"first"`` layer holds the
    scalar too, unused.

    ``conv_taps`` K >= 1: q, k and v pass a causal convolution over the last K tokens per channel straight after the
    projection (tensors ``q_conv``, ``k_conv``, ``v_conv`` in ``names``, [channels, K], the last column the current token's, no
    bias, zeros before a sequence's start); the last K - 1 projected rows of a request are part of its state, so the mixer
    then needs ``{"kv": PagedKV, "conv": FixedState}`` (one tap is a factor per channel and needs no state). ``head_norm`` = eps: queries and keys are RMS-normed head by head over
    ``head_dim`` with weights of that size which all heads share (``q_norm``, ``k_norm``). ``talk``: the heads' softmax weights
    are mixed after the softmax, ``weight_h <- sum_g talk[h, g] weight_g`` (tensor ``talk`` [heads, heads]), and head h applies
    its mixed weights to the values of its own group. ``out_gate``: the concatenated heads are multiplied by
    ``sigmoid(Wg h)`` (tensor ``g``) before the output projection. Any of the first three takes the mixer through a path of its
    own (``_forward_shaped``), which knows no ``own_kv=False``, no ``qk_norm`` and no ``v_mix``, and with a convolution or mixed heads
    neither rotation nor sinks; an output gate alone goes with every other option (its rows ride in the q/k/v product).
    ``forward(..., accumulate=False)`` writes ``x = ...`` instead of adding.

    ``softcap`` c > 0: a score becomes ``c tanh(score / c)`` after the scale. ``weights="sigmoid"``: no softmax; a visible key
    weighs ``sigmoid(score + b_h)`` with one number a head (the tensor ``head_bias`` in ``names``, [heads]), and the weights are
    not normalised over the keys. ``sink="learned"``: the extra term's score is one number a head (the tensor ``sink``) instead of
    0. ``distance``: after scale and cap a score is lowered by ``a_h ln(1 + b_h (i - j))`` with two numbers a head (the tensors
    ``dist_scale`` and ``dist_rate``).

    Options that take the same path of their own as ``head_norm`` and go with each other, with a rotation, biases, windows, chunks,
    caps and sinks: ``head_norm_weight=False``: the per-head norm has no weight. ``norm_after``: it comes after the rotation, not before.
    ``out_gate="head"``: one gate a head (tensor ``g`` [heads, width]) multiplies the head's whole output. ``rel_bias`` = dict(rows=B,
    reach=R): after scale and cap a number of the tensor ``rel`` ([B, heads]) is added to the score, its row chosen by the distance
    (``distance_bucket``); rows 0: as many as the tensor has. ``keep_first`` n: under a window the first n keys of a sequence stay visible (their rows are kept in the
    cache for good). ``maps=2`` with ``diff`` d: differential attention: a query head and a key head are two of ``head_dim`` values
    ([map 1, map 2]) over the same values; with ``f = exp(lq1 . lk1) - exp(lq2 . lk2) + d`` (tensors ``lq1`` .. ``lk2``, [head_dim]) the
    head's output is ``a = map 1 - f map 2``, divided by its root mean square (``head_norm``'s eps) and multiplied by ``1 - d``.
    ``joins_heads`` (an attribute): ``heads(...)`` gives what the output projection reads, times ``out_scale``.
    """
    graph_safe = True
    lazy_input_ok = True
    can_overwrite = True


    def __init__(self, hidden_size, n_heads, n_kv_heads, head_dim, qkv_bias, window, position,
                 scale=None, out_bias=False, v_head_dim=None, prefix="", mask_chunk=0, own_kv=True, names=None,
                 qk_norm=None, sink=False, v_mix=None, conv_taps=0, head_norm=None, talk=False, out_gate=False,
                 softcap=None, weights="softmax", distance=False, head_norm_weight=True, norm_after=False, rel_bias=None,
                 keep_first=0, maps=1, diff=0.0):
        """``v_head_dim``: the size of a value head where it is not ``head_dim`` (key rows of the cache are
        then ``n_kv_heads * head_dim`` wide, value rows ``n_kv_heads * v_head_dim``, and the output
        projection reads ``n_heads * v_head_dim`` columns; such a mixer runs the plain kernels)."""
        super().__init__(prefix)
        if n_heads % n_kv_heads:
            fail(EINVAL, f"attention: {n_heads} heads are not a multiple of {n_kv_heads} key/value heads")
        self.E, self.H, self.G, self.D = hidden_size, n_heads, n_kv_heads, head_dim
        self.Dv = head_dim if v_head_dim is None else int(v_head_dim)
        self.maps, self.diff = int(maps), float(diff)
        self.HQ, self.GK = n_heads * self.maps, n_kv_heads * self.maps       # query and key heads as attention counts them
        self.QD, self.KD = self.HQ * head_dim, self.GK * head_dim
        self.VD, self.OD = n_kv_heads * self.Dv, n_heads * self.Dv
        self.qkv_bias = bool(qkv_bias)
        self.out_bias = bool(out_bias)
        self.window = int(window)
        self.mask_chunk = int(mask_chunk)
        self.own_kv = bool(own_kv)
        self.names = {n: f"{n}_proj.weight" for n in "qkvo"}
        self.names.update({f"{n}_bias": f"{n}_proj.bias" for n in "qkvo"})
        self.names.update(q_norm="q_norm.weight", k_norm="k_norm.weight", v_mix="v_mix", talk="talk", g="g_proj.weight",
                          q_conv="q_conv.weight", k_conv="k_conv.weight", v_conv="v_conv.weight", head_bias="head_bias",
                          sink="sink", dist_scale="dist_scale", dist_rate="dist_rate", rel="rel", lq1="lq1", lk1="lk1", lq2="lq2", lk2="lk2")
        self.names.update(names or {})
        self.conv_taps = int(conv_taps)
        self.head_norm = None if head_norm is None else float(head_norm)
        self.head_norm_weight, self.norm_after = bool(head_norm_weight), bool(norm_after)
        self.talk, self.out_gate, self.head_gate = bool(talk), bool(out_gate), out_gate == "head"
        self.gate_rows = 0 if not out_gate else n_heads if self.head_gate else self.OD
        self.rel_bias = None if rel_bias is None else (int(rel_bias["rows"]), float(rel_bias["reach"]))
        self.keep_first = int(keep_first)
        # what needs the path with per-head norms but neither a convolution nor mixed heads
        self.masked = self.head_gate or self.rel_bias is not None or self.keep_first > 0 or self.maps > 1 or self.norm_after \
            or (head_norm is not None and not (self.conv_taps >= 1 or self.talk) and (position.kind != "none" or qkv_bias or window or mask_chunk
                                                                                   or sink or softcap or distance))
        self.shaped = self.conv_taps >= 1 or self.head_norm is not None or self.talk or self.masked
        self.rel_table = self.map_factor = None
        self.out_scale = 1.0
        if self.maps not in (1, 2) or (self.maps == 2 and self.head_norm is None) or self.keep_first < 0:
            fail(EINVAL, f"attention: {self.maps} maps (two need head_norm's eps), {self.keep_first} kept keys")
        self.softcap = float(softcap or 0.0)
        if weights not in ("softmax", "sigmoid") or self.softcap < 0.0 or (weights == "sigmoid" and sink):
            fail(EINVAL, f"attention: weights '{weights}' (softmax, or sigmoid without a sink term) and a soft cap of {softcap}")
        self.weights = weights
        self.head_bias = None
        self.distance, self.learned_sink = bool(distance), sink == "learned"
        if self.distance and weights != "softmax":
            fail(EINVAL, "attention: a distance term goes with softmax weights")
        self.dist_w = self.sink_w = None
        if self.out_gate and not own_kv:
            fail(EINVAL, "attention: an output gate goes with a mixer that has projections of its own")
        if self.shaped and (not own_kv or qk_norm is not None or v_mix or weights != "softmax" or (self.out_gate and self.masked and not self.head_gate)):
            fail(EINVAL, "attention: per-head norms and what goes with them need projections of the mixer's own and a softmax, and know "
                         "gates of whole heads")
        if (self.conv_taps >= 1 or self.talk) and (position.kind != "none" or sink or qkv_bias or window or mask_chunk or self.softcap or distance
                                                   or self.masked):
            fail(EINVAL, "attention: a convolution and mixed heads go without rotation, biases, windows and the other options")
        if not 0 <= self.conv_taps <= 8:
            fail(EINVAL, f"attention: a convolution over {self.conv_taps} tokens (at most 8)")
        self.taps = self.talk_w = self.no_state = None
        self.qk_norm = None if qk_norm is None else float(qk_norm)
        self.sink = bool(sink)
        if v_mix not in (None, "first", "blend") or (v_mix and not own_kv):
            fail(EINVAL, f"attention: v_mix '{v_mix}' is neither first nor blend, or the layer has no values of its own")
        self.v_mix = v_mix
        self.q_norm_w = self.k_norm_w = self.v_blend = None
        if self.window < 0 or self.mask_chunk < 0:
            fail(EINVAL, "attention: a window and a masking chunk are counted in tokens, 0 for none")
        self.scale = float(scale) if scale is not None else 1.0 / math.sqrt(head_dim)   # src/model.c:507
        self.position = make_part("position", position)
        if self.masked and (getattr(self.position, "pairing", "split_half") != "split_half" or self.position.kind not in ("none", "rotary")):
            fail(EINVAL, "attention: per-head norms go with a rotation of split halves, or none")
        self.joins_heads = self.shaped and self.conv_taps == 0 and not self.talk and not (self.out_gate and not self.head_gate) and not out_bias
        self.w_qkv = self.b_qkv = self.w_o = self.b_o = None

    def sub_parts(self):
        return [self.position]

    @staticmethod
    def distance_bucket(n, rows, reach):
        """The row of a table of ``rows`` rows for a key n positions back: one row a distance in the lower half, logarithmic from there
        to ``reach``, the last row beyond."""
        half = rows // 2
        if n < half:
            return n
        return min(rows - 1, half + math.floor(math.log(n / half) / math.log(reach / half) * (rows - half)))

    def param_specs(self):
        p, nm = self.prefix, self.names
        widths = {"q": self.QD, "k": self.KD, "v": self.VD}
        specs = [ParamSpec(p + nm[n], (widths[n], self.E)) for n in self._projections()]
        specs.append(ParamSpec(p + nm["o"], (self.E, self.OD)))
        if self.qkv_bias:
            specs += [ParamSpec(p + nm[n + "_bias"], (widths[n],), "vector") for n in self._projections()]
        if self.out_bias:
            specs.append(ParamSpec(p + nm["o_bias"], (self.E,), "vector"))
        if self.qk_norm is not None:
            specs.append(ParamSpec(p + nm["q_norm"], (self.QD,), "vector", ("one_plus_normal", 0.1)))
            if self.own_kv:
                specs.append(ParamSpec(p + nm["k_norm"], (self.KD,), "vector", ("one_plus_normal", 0.1)))
        if self.v_mix:
            specs.append(ParamSpec(p + nm["v_mix"], (), "vector", ("normal", 0.3), optional=self.v_mix == "first"))
        if self.conv_taps >= 1:
            specs += [ParamSpec(p + nm[n + "_conv"], (widths[n], self.conv_taps), "vector", ("normal", 0.3)) for n in "qkv"]
        if self.head_norm is not None and self.head_norm_weight:
            specs += [ParamSpec(p + nm[n], (self.D,), "vector", ("one_plus_normal", 0.1)) for n in ("q_norm", "k_norm")]
        if self.talk:
            specs.append(ParamSpec(p + nm["talk"], (self.H, self.H), "vector", ("normal", 0.3)))
        if self.out_gate:
            specs.append(ParamSpec(p + nm["g"], (self.gate_rows, self.E)))
        if self.rel_bias is not None:
            specs.append(ParamSpec(p + nm["rel"], (self.rel_bias[0], self.H), "vector", ("normal", 0.5)))
        if self.maps == 2:
            specs += [ParamSpec(p + nm[n], (self.D,), "vector", ("normal", 0.1)) for n in ("lq1", "lk1", "lq2", "lk2")]
        if self.weights == "sigmoid":
            specs.append(ParamSpec(p + nm["head_bias"], (self.H,), "vector", ("normal", 0.5)))
        if self.learned_sink:
            specs.append(ParamSpec(p + nm["sink"], (self.H,), "vector", ("normal", 0.5)))
        if self.distance:
            specs += [ParamSpec(p + nm[n], (self.H,), "vector", ("one_plus_normal", 0.1)) for n in ("dist_scale", "dist_rate")]
        return specs

    def _projections(self):
        return "qkv" if self.own_kv else "q"

    def cache_need(self):
        if not self.own_kv:
            fail(EINVAL, f"attention '{self.prefix}' has no keys and values of its own: its schedule entry must read "
                         "another entry's cache")
        kv = PagedKV(self.KD, self.VD, self.window, self.mask_chunk, keep_first=self.keep_first)
        if self.conv_taps > 1:
            return {"kv": kv, "conv": FixedState((self.conv_taps - 1) * (self.QD + self.KD + self.VD))}
        return kv

    def reads_cache(self, need):
        """``need`` of the mixer whose storage this one reads, widened by what this one sees of it."""
        return PagedKV(need.k_width, need.v_width, need.window, need.mask_chunk, need.readers + ((self.window, self.mask_chunk),),
                       max(need.keep_first, self.keep_first))

    def bind(self, params, ops):
        p, nm = self.prefix, self.names
        # One matrix for the three projections that share an input: rows of q, then k, then v.
        mats = [params[p + nm[n]] for n in self._projections()]
        if self.maps == 2:
            mats[0] = self._maps_apart(mats[0])
        if self.out_gate:
            mats.append(params[p + nm["g"]])             # the gate reads the same input: one product for all four
        dt = torch.float32 if any(m.dtype == torch.float32 for m in mats) else mats[0].dtype
        self.w_qkv = memory.cat([m.to(dt) for m in mats], 0, f"{p}q, k and v in one matrix")
        if self.qkv_bias:
            biases = [params[p + nm[n + "_bias"]] for n in self._projections()]
            if self.maps == 2:
                biases[0] = self._maps_apart(biases[0])
            if self.out_gate:                            # the gate's rows have none
                biases.append(torch.zeros(self.gate_rows, dtype=biases[0].dtype, device=biases[0].device))
            self.b_qkv = memory.cat(biases, 0, f"{p}q, k and v biases in one vector")
        if self.weights == "sigmoid":
            self.head_bias = params[p + nm["head_bias"]].contiguous()
        if self.learned_sink:
            self.sink_w = params[p + nm["sink"]].contiguous()
        if self.distance:
            self.dist_w = tuple(params[p + nm[n]].contiguous() for n in ("dist_scale", "dist_rate"))
        self.w_o = params[p + nm["o"]]
        self.short_request_rows = ops.prompt_rows     # where the attention kernels for decoded tokens and for prompt portions part
        if self.out_bias:
            self.b_o = params[p + nm["o_bias"]]
        if self.qk_norm is not None:
            self.q_norm_w = params[p + nm["q_norm"]]
            self.k_norm_w = params[p + nm["k_norm"]] if self.own_kv else None
        if self.v_mix == "blend":
            self.v_blend = params[p + nm["v_mix"]].reshape(1)
        if self.conv_taps >= 1:
            self.no_state = memory.zeros((1, 1), torch.float32, ops.device, f"{p}a convolution's state that is never read")
            self.taps = memory.cat([params[p + nm[n + "_conv"]] for n in "qkv"], 0, f"{p}taps of q, k and v in one matrix").contiguous()
        if self.rel_bias is not None:
            # the table by distance: up to the one from which the last row holds, or the farthest that the mask shows
            rows, reach = int(params[p + nm["rel"]].shape[0]), self.rel_bias[1]
            if rows < 2 or not reach > rows // 2:
                fail(EINVAL, f"attention '{p}': a table of {rows} distance terms that reaches {reach:g} positions back")
            ids, seen = [], self.mask_chunk or self.window or 1 << 30
            while len(ids) < seen and (not ids or ids[-1] < rows - 1):
                ids.append(self.distance_bucket(len(ids), rows, reach))
            table = params[p + nm["rel"]].index_select(0, torch.tensor(ids, dtype=torch.int64, device=params[p + nm["rel"]].device))
            self.rel_table = memory.to_device(table.t().contiguous(), ops.device, f"{p}distance terms")
        if self.maps == 2:
            a, b, c, d = (params[p + nm[n]].double() for n in ("lq1", "lk1", "lq2", "lk2"))
            self.map_factor = memory.to_device((torch.exp((a * b).sum()) - torch.exp((c * d).sum()) + self.diff).float().reshape(1),
                                               ops.device, f"{p}factor of the second map")
        if self.head_norm is not None and self.head_norm_weight:
            self.q_norm_w, self.k_norm_w = params[p + nm["q_norm"]].contiguous(), params[p + nm["k_norm"]].contiguous()
        if self.talk:
            self.talk_w = params[p + nm["talk"]].contiguous()
        elif self.out_gate and self.shaped and not self.masked:              # the gate rides in the kernel that mixes heads: an identity mix
            self.talk_w = memory.to_device(torch.eye(self.H, dtype=torch.float32), ops.device, f"{p}identity mix of heads")

    def _maps_apart(self, rows):
        """Rows of queries head by head, [map 1, map 2] each, in the order attention counts its heads in: for every key head the
        first map's queries of its group, then the second's."""
        R = self.H // self.G
        return rows.reshape(self.G, R, 2, self.D, -1).transpose(1, 2).reshape(rows.shape)

    def heads(self, ops, step, h, cache, out, write_cache=True):
        """The concatenated heads before the output projection, times ``out_scale``, into ``out`` ([T, heads * v_head_dim], rows may lie
        apart): projections, norms, rotation and store, attention."""
        if not write_cache:
            fail(EINVAL, f"attention '{self.prefix}': this mixer cannot read another entry's cache")
        T = h.shape[0]
        proj = ops.scratch("qkv", (T, self.w_qkv.shape[0]), ops.act_dtype)
        with ops.section("qkv"):                # (sums of a product that split K, or of few rows, are finished by the next kernel)
            ops.gemm(h, self.w_qkv, proj, bias=self.b_qkv, defer=True)
        pos = self.position
        with ops.section("qkv_prepare"):
            q = ops.scratch("q_normed", (T, self.QD), ops.act_dtype)
            gate = ops.head_norm_store(proj, self.HQ, self.GK, self.D, self.Dv, self.q_norm_w, self.k_norm_w, self.head_norm or 0.0, q, cache,
                                step.group(cache.group).slot_map, n_v_heads=self.G, norm=self.head_norm is not None, after=self.norm_after,
                                positions=step.positions, inv_freq=getattr(pos, "inv_freq", None), rot_dim=getattr(pos, "rot_dim", 0),
                                extra="head_gate" if self.head_gate else None)
        att = out if self.maps == 1 else ops.scratch("att_maps", (T, self.HQ * self.Dv), torch.float32)
        with ops.section("attn"):
            ops.paged_attention(q, self.HQ, self.GK, self.D, cache, step, self.window, self.scale, att, v_head_dim=self.Dv,
                                mask_chunk=self.mask_chunk, sink=self.sink, softcap=self.softcap, sink_scores=self.sink_w,
                                distance=self.dist_w, v_share=self.maps, keep_first=self.keep_first, rel=self.rel_table,
                                gate=gate, out_scale=self.out_scale if self.maps == 1 else 1.0)
            if self.maps == 2:
                ops.diff_mix(att, self.map_factor, (1.0 - self.diff) * self.out_scale, self.head_norm, self.H, self.G, self.Dv, out)

    def _forward_shaped(self, ops, step, h, cache, x, accumulate):
        """The path of a mixer with a convolution, per-head norms, mixed heads or an output gate (see the class)."""
        T = h.shape[0]
        att = ops.scratch("att", (T, self.OD), ops.act_dtype)
        if self.joins_heads:
            self.heads(ops, step, h, cache, att)
            with ops.section("wo"):
                ops.gemm(att, self.w_o, x, accumulate=accumulate, defer=True)
            return
        C = self.QD + self.KD + self.VD
        kv = cache["kv"] if isinstance(cache, dict) else cache
        proj = ops.scratch("qkv", (T, self.w_qkv.shape[0]), ops.act_dtype)
        with ops.section("qkv"):
            ops.gemm(h, self.w_qkv, proj)
        rows = proj[:, :C]
        with ops.section("qkv_prepare"):
            if self.conv_taps >= 1:
                rows = ops.scratch("qkv_conv", (T, C), torch.float32)
                ops.causal_conv(proj[:, :C], self.taps, None, cache["conv"].state if self.conv_taps > 1 else self.no_state, step, rows)
            q = ops.scratch("q_normed", (T, self.QD), ops.act_dtype)
            ops.head_norm_store(rows, self.H, self.G, self.D, self.Dv, self.q_norm_w, self.k_norm_w, self.head_norm or 0.0, q, kv,
                                step.group(kv.group).slot_map)
        with ops.section("attn"):
            cross = ops.scratch("att_cross", (T, self.G * self.OD), ops.act_dtype)
            ops.paged_attention(q, self.H, self.G, self.D, kv, step, 0, self.scale, cross if self.talk_w is not None else att,
                                v_head_dim=self.Dv, cross_values=self.talk_w is not None)
            if self.talk_w is not None:
                ops.talk_mix(cross, self.talk_w, self.H, self.G, self.Dv, att, gate=proj[:, C:] if self.out_gate else None)
        with ops.section("wo"):
            ops.gemm(att, self.w_o, x, accumulate=accumulate, defer=True)

    def forward(self, ops, step, h, cache, x, write_cache=True, accumulate=True):
        if self.shaped:
            if not write_cache:
                fail(EINVAL, f"attention '{self.prefix}': this mixer cannot read another entry's cache")
            return self._forward_shaped(ops, step, h, cache, x, accumulate)
        T = h.shape[0]
        if write_cache and not self.own_kv:
            fail(EINVAL, f"attention '{self.prefix}' has no keys and values to write")
        width = self.QD + self.KD + self.VD if write_cache else self.QD
        gate = None
        if self.out_gate:                       # [q | k | v | gate] from one product; a layer that only reads takes them apart
            if write_cache:
                rows = ops.scratch("qkv", (T, width + self.OD), ops.act_dtype)
                with ops.section("qkv"):
                    ops.gemm(h, self.w_qkv, rows, bias=self.b_qkv)
                qkv, gate = rows[:, :width], rows[:, width:]
            else:
                qkv = ops.scratch("qkv", (T, width), ops.act_dtype)
                gate = ops.scratch("att_gate", (T, self.OD), ops.act_dtype)
                with ops.section("qkv"):
                    ops.gemm(h, self.w_qkv[:width], qkv, bias=None if self.b_qkv is None else self.b_qkv[:width])
                    ops.gemm(h, self.w_qkv[self.w_qkv.shape[0] - self.OD:], gate)
        else:
            qkv = ops.scratch("qkv", (T, width), ops.act_dtype)
            # a product that split K is added up inside the next kernel (position.store, the next norm)
            with ops.section("qkv"):
                ops.gemm(h, self.w_qkv[:width], qkv, bias=None if self.b_qkv is None else self.b_qkv[:width], defer=True)
        prepare = {}
        if self.qk_norm is not None:
            prepare.update(q_norm=self.q_norm_w, k_norm=self.k_norm_w if write_cache else None, eps=self.qk_norm)
        if self.v_mix and write_cache:
            # the first mixing layer's values of this step's tokens wait in a work buffer for the layers that blend
            kept = ops.scratch("v_first", (T, self.VD), ops.act_dtype)
            prepare.update(dict(v_keep=kept) if self.v_mix == "first" else dict(v_blend=self.v_blend, v_other=kept))
        if prepare:
            self.position.store(ops, step, qkv, self.H, self.G if write_cache else 0, cache, write_cache, v_head_dim=self.Dv,
                                prepare=prepare)
        elif self.Dv == self.D:
            self.position.store(ops, step, qkv, self.H, self.G if write_cache else 0, cache, write_cache)
        else:                                   # only a position part that knows of value heads of another size can serve
            self.position.store(ops, step, qkv, self.H, self.G if write_cache else 0, cache, write_cache, v_head_dim=self.Dv)
        att = ops.scratch("att", (T, self.OD), ops.act_dtype)
        with ops.section("attn"):
            ops.paged_attention(qkv, self.H, self.G, self.D, cache, step, self.window, self.scale, att,
                                slopes=getattr(self.position, "score_slopes", None), v_head_dim=self.Dv,
                                mask_chunk=self.mask_chunk, sink=self.sink, softcap=self.softcap, weights=self.weights,
                                head_bias=self.head_bias, sink_scores=self.sink_w, distance=self.dist_w)
            if gate is not None:
                ops.gate_mul(att, gate, att, "sigmoid")
        with ops.section("wo"):
            ops.gemm(att, self.w_o, x, bias=self.b_o, accumulate=accumulate, defer=True)


@register_part("mixer", "latent_attention")
class LatentAttention(Part):
    """Causal softmax attention whose keys and values (and, optionally, queries) come through latents. With H = ``n_heads``, D =
    ``head_dim`` (the unrotated dimensions of a query/key head), R = ``rot_dim`` (the rotated ones), Dv = ``v_head_dim``, C = ``kv_rank``:

    * ``q = Wuq (rmsnorm(Wdq h) * q_norm)``, or ``q = Wq h`` (``q_latent`` False); head by head ``[D unrotated | R rotated]``;
    * ``Wdkv h`` has ``C + R`` rows: the first C, RMS-normed with ``kv_norm``, are the latent ``c``; the last R are one key part
      that all heads share and that is rotated like the queries' R parts (``position``: a rotary PartSpec over R dimensions);
    * per head ``k = [Wuk c | rotated part]``, ``v = Wuv c``; ``score = q . k * scale``; softmax over the keys ``j <= i``, with
      ``window > 0`` over the last ``window`` of them; ``sink``: a head's denominator has one more term ``exp(sink_h)`` (the tensor
      ``sink``, [heads]) that has no value;
    * the concatenated heads are multiplied by ``sigmoid(Wg h)`` (``out_gate``) and projected by ``Wo``.

    The cache holds one row a token: the rotated part and the latent as the key of one shared head, the latent as its value. The
    keys' expansion is folded into the queries, ``q' = Wuk_h^T q_h`` (``score = q' . c + q_rot . k_rot``), and the values' is
    applied after the weighted sum, ``o_h = Wuv_h (sum_j p_j c_j)``: attention itself is the engine's, with H query heads on one
    key/value head of ``R + C`` key and ``C`` value dimensions. The latents' norms are fp32 over the 32-bit sums of their products.
    ``names``: the tensors' names after ``prefix`` (keys dq, q_norm, uq or q; dkv, kv_norm, uk, uv, g, o, sink).
    ``forward(..., accumulate=False)`` writes ``x = ...`` instead of adding.

    The products that read the mixer's input are held as one matrix (queries or their latent first, then ``Wdkv``, then the gate):
    a step of few rows runs it as one product with 32-bit sums, from which the heads' products (``Ops.head_rows``) and the store
    read; a prompt portion runs its parts with the output type that each wants."""
    graph_safe = True
    can_overwrite = True

    FEW_ROWS = 64                # rows up to which the heads' products run as one launch without a plan

    def __init__(self, hidden_size, n_heads, head_dim, rot_dim, v_head_dim, kv_rank, position, scale=None, q_rank=None, eps=1e-6,
                 out_gate=True, prefix="", names=None, q_latent=True, window=0, sink=False):
        """``q_rank`` None: the query latent's size is the tensors'."""
        super().__init__(prefix)
        self.E, self.H, self.D, self.R, self.Dv, self.C = hidden_size, n_heads, head_dim, rot_dim, v_head_dim, kv_rank
        self.q_latent = bool(q_latent)
        self.q_rank = (q_rank or None) if self.q_latent else None
        self.eps = float(eps)
        self.window, self.sink = int(window), bool(sink)
        if self.window < 0:
            fail(EINVAL, "latent_attention: a window is counted in tokens, 0 for none")
        self.scale = float(scale) if scale is not None else 1.0 / math.sqrt(head_dim + rot_dim)
        self.out_gate = bool(out_gate)
        self.position = make_part("position", position)
        if getattr(self.position, "score_slopes", None) is not None or getattr(self.position, "rot_dim", 0) > rot_dim:
            fail(EINVAL, f"latent_attention: the position part turns at most the {rot_dim} rotated dimensions")
        self.names = dict(dq="dq", q_norm="dq.norm", uq="uq", q="q", dkv="dkv", kv_norm="dkv.norm", uk="uk", uv="uv", g="g", o="o", sink="sink")
        self.names.update(names or {})
        self.HD = rot_dim + kv_rank                          # a head as attention sees it: [rotated part | latent]
        self.w_in = self.w_uq = self.w_uk_t = self.w_uv = self.w_o = self.q_norm_w = self.kv_norm_w = self.sink_w = None
        self.q_cols, self.few_ok = 0, False

    def sub_parts(self):
        return [self.position]

    def param_specs(self):
        p, nm = self.prefix, self.names
        rq = self.q_rank or 0                                # 0: any size (the loader takes the tensor's)
        q_rows = self.H * (self.D + self.R)
        if self.q_latent:
            specs = [ParamSpec(p + nm["dq"], (rq, self.E)), ParamSpec(p + nm["q_norm"], (rq,), "vector", ("one_plus_normal", 0.1)),
                     ParamSpec(p + nm["uq"], (q_rows, rq), "matrix", ("normal", 0.1))]
        else:
            specs = [ParamSpec(p + nm["q"], (q_rows, self.E))]
        specs += [ParamSpec(p + nm["dkv"], (self.C + self.R, self.E)),
                  ParamSpec(p + nm["kv_norm"], (self.C,), "vector", ("one_plus_normal", 0.1)),
                  ParamSpec(p + nm["uk"], (self.H * self.D, self.C), "matrix", ("normal", 0.1)),
                  ParamSpec(p + nm["uv"], (self.H * self.Dv, self.C), "matrix", ("normal", 0.1)),
                  ParamSpec(p + nm["o"], (self.E, self.H * self.Dv))]
        if self.out_gate:
            specs.append(ParamSpec(p + nm["g"], (self.H * self.Dv, self.E)))
        if self.sink:
            specs.append(ParamSpec(p + nm["sink"], (self.H,), "vector", ("normal", 0.5)))
        return specs

    def cache_need(self):
        return PagedKV(self.HD, self.C, self.window)

    def bind(self, params, ops):
        p, nm = self.prefix, self.names
        mats = [params[p + nm["dq" if self.q_latent else "q"]], params[p + nm["dkv"]]]
        if self.out_gate:
            mats.append(params[p + nm["g"]])
        dt = torch.float32 if any(m.dtype == torch.float32 for m in mats) else mats[0].dtype
        self.w_in = memory.cat([m.to(dt) for m in mats], 0, f"{p}the products that read the mixer's input in one matrix")
        self.q_cols = mats[0].shape[0]                       # of the queries, or of their latent
        self.w_uv, self.w_o = params[p + nm["uv"]].view(self.H, self.Dv, self.C), params[p + nm["o"]]
        if self.q_latent:
            self.w_uq, self.q_norm_w = params[p + nm["uq"]], params[p + nm["q_norm"]].contiguous()
            self.q_rank = self.q_cols
            if self.w_uq.shape[1] != self.q_rank or self.q_norm_w.numel() != self.q_rank:
                fail(EINVAL, f"latent_attention '{p}': the query latent's sizes do not match")
        # q' = Wuk_h^T q_h: the product reads Wuk_h [D, C] as [C, D] rows
        uk = params[p + nm["uk"]]
        self.w_uk_t = memory.to_device(uk.reshape(self.H, self.D, self.C).transpose(1, 2), ops.device,
                                       f"{p}the keys' expansion, transposed head by head")
        self.kv_norm_w = params[p + nm["kv_norm"]].contiguous()
        if self.sink:
            self.sink_w = params[p + nm["sink"]].contiguous()
        self.short_request_rows = ops.prompt_rows
        # whether the one-launch products take these sizes and types (16-byte reads of operands, 8-byte stores of results)
        self.few_ok = (ops.act_dtype == torch.bfloat16 and all(m.dtype == torch.bfloat16 for m in (self.w_in, self.w_uk_t, self.w_uv))
                       and self.D % 16 == 0 and self.C % 32 == 0 and self.Dv % 32 == 0 and self.R % 8 == 0)

    def forward(self, ops, step, h, cache, x, write_cache=True, accumulate=True):
        if not write_cache:
            fail(EINVAL, f"latent_attention '{self.prefix}': this mixer cannot read another entry's cache")
        T, H, D, R, C, Dv, HD = h.shape[0], self.H, self.D, self.R, self.C, self.Dv, self.HD
        Q, CR = self.q_cols, C + R
        few = self.few_ok and T <= self.FEW_ROWS and not ops.force_plain_gemm
        gate = None
        with ops.section("latent_down"):
            if few:                                          # one product: 32-bit rows [queries or their latent | dkv | gate]
                rows = ops.scratch("latent_rows", (T, self.w_in.shape[0]), torch.float32)
                ops.gemm(h, self.w_in, rows)
                q, down = rows[:, :Q], rows[:, Q:Q + CR]
                if self.out_gate:
                    gate = rows[:, Q + CR:]
            else:
                if self.q_latent:
                    rows = ops.scratch("latent_rows", (T, Q + CR), torch.float32)
                    ops.gemm(h, self.w_in[:Q + CR], rows)
                    q, down = rows[:, :Q], rows[:, Q:]
                else:
                    q = ops.scratch("latent_q_up", (T, Q), ops.act_dtype)
                    down = ops.scratch("latent_rows", (T, CR), torch.float32)
                    ops.gemm(h, self.w_in[:Q], q)
                    ops.gemm(h, self.w_in[Q:Q + CR], down)
                if self.out_gate:
                    gate = ops.scratch("att_gate", (T, H * Dv), ops.act_dtype)
                    ops.gemm(h, self.w_in[Q + CR:], gate)
        if self.q_latent:
            cq = ops.scratch("latent_q", (T, Q), ops.act_dtype)
            up = ops.scratch("latent_q_up", (T, H * (D + R)), ops.act_dtype)
            with ops.section("latent_q"):
                ops.group_rmsnorm(q, self.q_norm_w, self.eps, 1, cq)
                ops.gemm(cq, self.w_uq, up)
            q = up
        # a head's query as attention sees it: [rotated part | the keys' expansion folded in]
        folded = ops.scratch("latent_queries", (T, H * HD), ops.act_dtype)
        with ops.section("latent_pack"):
            if not few:
                ops.head_products(q.view(T * H, D + R), self.w_uk_t, folded.view(T * H, HD)[:, R:], H)
            pos = self.position
            ops.latent_store(down, q, self.kv_norm_w, self.eps, step.positions, getattr(pos, "inv_freq", None), getattr(pos, "rot_dim", 0),
                             getattr(pos, "pairing", "split_half"), folded, cache, step.group(cache.group).slot_map, H, D, R, C,
                             fold=self.w_uk_t if few else None)
        att = ops.scratch("latent_att", (T, H * C), ops.act_dtype)
        with ops.section("latent_attn"):
            ops.paged_attention(folded, H, 1, HD, cache, step, self.window, self.scale, att, v_head_dim=C, sink=self.sink, sink_scores=self.sink_w)
        heads = ops.scratch("att", (T, H * Dv), ops.act_dtype)
        with ops.section("latent_v"):
            # the values' expansion of each head's weighted sum of latents
            if few:
                ops.head_rows(att, self.w_uv, heads, C, Dv, gate=gate)
            else:
                ops.head_products(att.view(T * H, C), self.w_uv, heads.view(T * H, Dv), H)
                if gate is not None:
                    ops.gate_mul(heads, gate, heads, "sigmoid")
        with ops.section("latent_wo"):
            ops.gemm(heads, self.w_o, x, accumulate=accumulate, defer=True)
