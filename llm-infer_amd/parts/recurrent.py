from __future__ import annotations

import math

import torch

from ..cache.specs import StateSpec
from ..kernels import ops
from ..registry import register_mixer
from ..weights.loader import ParamSpec
from .base import Part


def _segments(part, ctx, waves_a_token: int):
    """The segments in which a 16-bit model walks a step's long prompts side by side (None: in order, as a float32 model
    and every decode step do, which gives the same bits however a prompt is cut): short enough that some
    ``ops.SSM_WAVES`` waves run, between 16 and ``ops.SSM_SEGMENT`` tokens."""
    if part.dtype == torch.float32 or ctx.is_decode or not getattr(ctx, "host_qlens", None):
        return None
    length = max(16, min(ops.SSM_SEGMENT, 1 << max(0, (ctx.n_tokens * waves_a_token // ops.SSM_WAVES).bit_length() - 1)))
    return ops.ssm_segments(ctx, length) if max(ctx.host_qlens) > length else None


def _in_chunks(part, ctx) -> bool:
    """True where a recurrence runs a chunk of tokens at a time: the prompts of a 16-bit model.  (A float32 model and every
    decode step go token by token, which gives the same bits however a prompt is cut.)"""
    return part.dtype != torch.float32 and not ctx.is_decode and bool(getattr(ctx, "host_qlens", None))


def _own_state(owns_cache, what):
    if not owns_cache:
        raise ValueError(f"{what} keeps a state of its own in every run")


@register_mixer("gated_delta")
class GatedDelta(Part):
    """The gated delta rule.  q and k (``n_kv_heads`` heads of ``head_dim`` d) and v (``n_heads`` heads of ``v_head_dim`` dv)
    are projections, each behind a causal convolution over time per channel (``conv_taps``, no bias) and silu; q and k
    become unit vectors per head, x / sqrt(sum x^2 + 1e-6), q times d^(-1/2).  Head h reads q/k head h // (n_heads /
    n_kv_heads); with beta = sigmoid(W_b x)_h and g = exp(-exp(A_log_h) softplus((W_a x)_h + dt_bias_h)) per head

        S <- g S;   u = beta (v - S^T k);   S <- S + k u^T;   o = S^T q

    Every head's o is divided by its root mean square (``norm_eps``), multiplied by a weight [dv] that the heads share and
    by silu(W_g x), and projected.  S (float32 [n_heads, d, dv]) and the convolution's last taps - 1 inputs are state of
    every sequence.  Unit norms, gates, decays and the recurrence are float32 whatever the matrices' type.  The prompts of a
    16-bit model run 32 tokens at a time on the matrix cores, with q, k and v in bfloat16 behind the convolution.  The input
    products are one product against [W_q; W_k; W_v; W_g; W_b; W_a], which ``ParallelMixers`` may share with the mixer
    beside this one.  ``names``: local tensor names."""

    NAMES = {"q": "q_proj.weight", "k": "k_proj.weight", "v": "v_proj.weight", "g": "g_proj.weight", "b": "b_proj.weight",
             "a": "a_proj.weight", "q_conv": "q_conv.weight", "k_conv": "k_conv.weight", "v_conv": "v_conv.weight",
             "a_log": "A_log", "dt_bias": "dt_bias", "norm": "norm.weight", "o": "o_proj.weight"}
    writes_rows = True

    def __init__(self, *, hidden_size, n_heads, n_kv_heads, head_dim, v_head_dim, conv_taps, norm_eps, names=None, position=None,
                 prefix, dtype, device):
        if n_heads % n_kv_heads != 0:
            raise ValueError("gated delta: n_heads must be a multiple of n_kv_heads")
        if not (1 <= head_dim <= 256 and v_head_dim >= 1):
            raise ValueError(f"gated delta: head sizes {head_dim} / {v_head_dim} (keys up to 256 wide)")
        if not 1 <= conv_taps <= 16:
            raise ValueError(f"gated delta: a convolution over {conv_taps} tokens (1 to 16)")
        self.hidden_size, self.n_heads, self.n_kv_heads = hidden_size, n_heads, n_kv_heads
        self.head_dim, self.v_head_dim, self.conv_taps, self.norm_eps = head_dim, v_head_dim, int(conv_taps), float(norm_eps)
        self.names = {**self.NAMES, **(names or {})}
        self.prefix, self.dtype, self.device = prefix, dtype, device
        self.channels = 2 * n_kv_heads * head_dim + n_heads * v_head_dim
        self.g_col = self.channels                                  # the columns of the input product: q | k | v | g | b | a
        self.b_col = self.g_col + n_heads * v_head_dim
        self.a_col = self.b_col + n_heads
        self.w_in = self.wo = None

    def params(self):
        H, G, d, dv, w, n, taps = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim, self.hidden_size, self.names, self.conv_taps
        return {n["q"]: ParamSpec((G * d, w)), n["k"]: ParamSpec((G * d, w)), n["v"]: ParamSpec((H * dv, w)),
                n["g"]: ParamSpec((H * dv, w)), n["b"]: ParamSpec((H, w)), n["a"]: ParamSpec((H, w)),
                n["q_conv"]: ParamSpec((G * d, taps), "vector", "wide"), n["k_conv"]: ParamSpec((G * d, taps), "vector", "wide"),
                n["v_conv"]: ParamSpec((H * dv, taps), "vector", "wide"), n["a_log"]: ParamSpec((H,), "vector", "small"),
                n["dt_bias"]: ParamSpec((H,), "vector", "small"), n["norm"]: ParamSpec((dv,), "vector", "ones"),
                n["o"]: ParamSpec((w, H * dv))}

    def bind(self, tensors):
        n = self.names
        self.w_in = ops.prepare_weight(torch.cat([tensors[n[k]] for k in ("q", "k", "v", "g", "b", "a")], 0).contiguous())
        self.conv = torch.cat([tensors[n[k]].as_subclass(torch.Tensor).float() for k in ("q_conv", "k_conv", "v_conv")], 0).contiguous()
        self.wo = ops.prepare_weight(tensors[n["o"]])
        self.a_log, self.dt_bias, self.norm = tensors[n["a_log"]], tensors[n["dt_bias"]], tensors[n["norm"]]

    def in_rows(self) -> int:
        return self.a_col + self.n_heads

    def cache_specs(self):
        return [StateSpec((self.n_heads, self.head_dim, self.v_head_dim), "float32"),
                StateSpec((max(self.conv_taps - 1, 1), self.channels), "float32")]

    def _heads(self, h, ctx, views, owns_cache, proj, col0):
        _own_state(owns_cache, "the delta rule")
        H, G, d, dv = self.n_heads, self.n_kv_heads, self.head_dim, self.v_head_dim
        if proj is None:
            proj, col0 = ops.linear(h, self.w_in, out_dtype=torch.float32), 0
        chunked = _in_chunks(self, ctx)
        rows = ops.delta_prepare(proj, col0, col0 + self.b_col, col0 + self.a_col, self.conv, views[1].state, self.a_log,
                                 self.dt_bias, ctx, H, G, d, dv, chunked)
        if not chunked and dv <= ops.SCAN_HEAD_LIMIT:      # the norm and gate behind it in the same kernel
            return ops.delta_scan(*rows, views[0].state, ctx, H, G, d, dv, (self.norm, proj, col0 + self.g_col, self.norm_eps, self.dtype))
        o = (ops.delta_chunks if chunked else ops.delta_scan)(*rows, views[0].state, ctx, H, G, d, dv)
        return ops.gated_head_norm(o, self.norm, proj, col0 + self.g_col, H, self.norm_eps, self.dtype, gate_silu=True)

    def addends(self, h, ctx, views, owns_cache=True, proj=None, col0=0):
        """``proj`` (float32 [T, n]) with this mixer's columns from ``col0`` on: the input product is not run here."""
        return [(ops.linear(self._heads(h, ctx, views, owns_cache, proj, col0), self.wo, out_dtype=torch.float32), 1.0)]

    def forward_into(self, h, out, ctx, views, owns_cache=True):
        ops.linear(self._heads(h, ctx, views, owns_cache, None, 0), self.wo, out=out)
        return None

    def forward(self, h, ctx, views, residual, owns_cache=True):
        ops.linear(self._heads(h, ctx, views, owns_cache, None, 0), self.wo, ops.EPI_ADD, out=residual)


@register_mixer("selective_scan")
class SelectiveScan(Part):
    """The selective state-space mixer with a decay for every channel and state.  The input product yields [x: inner | z:
    inner]; x passes a causal convolution over time per channel (``conv_taps``, with a bias) and silu; W_x x is [dt:
    ``dt_rank`` | B: ``n_state`` | C: ``n_state``]; per channel c and state i, with A = -exp(A_log) [inner, n_state],

        dt_c = softplus(W_dt dt + bias)_c;   S[c, i] <- exp(dt_c A[c, i]) S[c, i] + dt_c x_c B_i
        y_c = sum over i of S[c, i] C_i + D_c x_c

    and the output product reads y silu(z).  S (float32, kept as [n_state, inner]) and the convolution's last taps - 1 inputs
    are state of every sequence.  Step sizes, decays and the recurrence are float32 whatever the matrices' type.  A is kept
    as A log2(e), so that a decay is one 2^x.  ``names``: local tensor names."""

    NAMES = {"in": "in_proj.weight", "conv": "conv1d.weight", "conv_bias": "conv1d.bias", "x": "x_proj.weight", "dt": "dt_proj.weight",
             "dt_bias": "dt_proj.bias", "a_log": "A_log", "d": "D", "o": "out_proj.weight"}
    writes_rows = True

    def __init__(self, *, hidden_size, inner, n_state, dt_rank, conv_taps, names=None, position=None, prefix, dtype, device):
        if not (1 <= n_state <= 256 and inner >= 1 and dt_rank >= 1):
            raise ValueError(f"selective scan: {inner} channels with {n_state} states (up to 256), step sizes of rank {dt_rank}")
        if not 1 <= conv_taps <= 16:
            raise ValueError(f"selective scan: a convolution over {conv_taps} tokens (1 to 16)")
        self.hidden_size, self.inner, self.n_state, self.dt_rank, self.conv_taps = hidden_size, inner, n_state, dt_rank, int(conv_taps)
        self.names = {**self.NAMES, **(names or {})}
        self.prefix, self.dtype, self.device = prefix, dtype, device
        self.w_in = self.w_x = self.w_dt = self.wo = None

    def params(self):
        c, s, r, w, n = self.inner, self.n_state, self.dt_rank, self.hidden_size, self.names
        return {n["in"]: ParamSpec((2 * c, w)), n["conv"]: ParamSpec((c, self.conv_taps), "vector", "wide"),
                n["conv_bias"]: ParamSpec((c,), "vector", "small"), n["x"]: ParamSpec((r + 2 * s, c)), n["dt"]: ParamSpec((c, r)),
                n["dt_bias"]: ParamSpec((c,), "vector", "small"), n["a_log"]: ParamSpec((c, s), "vector", "small"),
                n["d"]: ParamSpec((c,), "vector", "ones"), n["o"]: ParamSpec((w, c))}

    def bind(self, tensors):
        n = self.names
        self.w_in, self.wo, self.w_x = (ops.prepare_weight(tensors[n[k]]) for k in ("in", "o", "x"))
        self.w_dt = ops.prepare_weight(tensors[n["dt"]])
        self.conv, self.conv_bias, self.dt_bias, self.d_skip = (tensors[n[k]] for k in ("conv", "conv_bias", "dt_bias", "d"))
        a_log = tensors[n["a_log"]].as_subclass(torch.Tensor).double()
        self.a2 = (-torch.exp(a_log) / math.log(2.0)).T.to(torch.float32).contiguous()

    def cache_specs(self):
        return [StateSpec((self.n_state, self.inner), "float32"), StateSpec((max(self.conv_taps - 1, 1), self.inner), "float32")]

    def _rows(self, h, ctx, views, owns_cache):
        _own_state(owns_cache, "a selective scan")
        c, s, r = self.inner, self.n_state, self.dt_rank
        xz = ops.linear(h, self.w_in, out_dtype=torch.float32)
        x = ops.conv_silu(xz, 0, c, self.conv, self.conv_bias, views[1].state, ctx, self.dtype)
        dbc = ops.linear(x, self.w_x, out_dtype=torch.float32)
        raw = ops.linear(ops.cast_columns(dbc, 0, r, self.dtype), self.w_dt, out_dtype=torch.float32)
        return ops.selective_scan(x, raw, self.dt_bias, dbc, r, r + s, xz, c, self.a2, self.d_skip, views[0].state, ctx,
                                  _segments(self, ctx, (c + 63) // 64))

    def forward_into(self, h, out, ctx, views, owns_cache=True):
        ops.linear(self._rows(h, ctx, views, owns_cache), self.wo, out=out)
        return None

    def forward(self, h, ctx, views, residual, owns_cache=True):
        ops.linear(self._rows(h, ctx, views, owns_cache), self.wo, ops.EPI_ADD, out=residual)


@register_mixer("wkv")
class TimeMixing(Part):
    """Time mixing of the RWKV family with a decay for every key channel that depends on the token.  With x' the
    previous token's input (zeros for a sequence's first), each of r, k, v, g, w reads its own mix x + (x' - x) mu_s; r, k, v
    (``n_heads`` heads of ``head_dim`` d) are projections of their mixes; the decay is w = exp(-exp(W_2 tanh(W_1 mix_w) +
    w_0)) per head and key channel, through a rank that the checkpoint's tensors say (``decay_rank``: what random
    weights take).  Per head

        o = (S + diag(u) k v^T)^T r   (the bonus u counts the current token only),      S <- diag(w) S + k v^T

    Every head's o is divided by its root mean square (``norm_eps``); the heads side by side are multiplied by a weight
    [n_heads d] and by silu(W_g mix_g), and projected.  S (float32 [n_heads, d, d]) and the previous token's input are
    state of every sequence.  The part reads its rows in float32 (``reads_float32``); decays and the recurrence are float32
    whatever the matrices' type.  The prompts of a 16-bit model run 32 tokens at a time on the matrix cores, with v in
    bfloat16.  ``names``: local tensor names."""

    NAMES = {"mu": "mu_{}", "r": "r_proj.weight", "k": "k_proj.weight", "v": "v_proj.weight", "g": "g_proj.weight", "w1": "w1", "w2": "w2",
             "w0": "w0", "u": "u", "norm": "norm.weight", "o": "o_proj.weight"}
    MIXES = "rkvgw"
    reads_float32 = True
    writes_rows = True

    def __init__(self, *, hidden_size, n_heads, head_dim, norm_eps, decay_rank=64, names=None, position=None, prefix, dtype, device):
        if not (1 <= head_dim <= 256 and n_heads >= 1 and decay_rank >= 1):
            raise ValueError(f"wkv: {n_heads} heads of {head_dim} (up to 256 wide)")
        self.hidden_size, self.n_heads, self.head_dim, self.norm_eps = hidden_size, n_heads, head_dim, float(norm_eps)
        self.decay_rank = int(decay_rank)
        self.names = {**self.NAMES, **(names or {})}
        self.prefix, self.dtype, self.device = prefix, dtype, device
        self.w = self.wo = None

    def params(self):
        w, n, c, r = self.hidden_size, self.names, self.n_heads * self.head_dim, self.decay_rank
        out = {n["mu"].format(s): ParamSpec((w,), "vector", "half") for s in self.MIXES}
        out.update({n[s]: ParamSpec((c, w)) for s in "rkvg"})
        out.update({n["w1"]: ParamSpec((r, w), free=(0,)), n["w2"]: ParamSpec((c, r), free=(1,)), n["w0"]: ParamSpec((c,), "vector", "small"),
                    n["u"]: ParamSpec((self.n_heads, self.head_dim), "vector", "wide"), n["norm"]: ParamSpec((c,), "vector", "ones"),
                    n["o"]: ParamSpec((w, c))})
        return out

    def bind(self, tensors):
        n = self.names
        if tensors[n["w1"]].shape[0] != tensors[n["w2"]].shape[1]:
            raise ValueError(f"{self.prefix}: the decay's two matrices have ranks {tensors[n['w1']].shape[0]} and {tensors[n['w2']].shape[1]}")
        self.decay_rank = tensors[n["w1"]].shape[0]
        self.mu = torch.stack([tensors[n["mu"].format(s)].as_subclass(torch.Tensor).float() for s in self.MIXES]).contiguous()
        rows, keys = self.n_heads * self.head_dim, ("r", "k", "v", "g", "w1")
        self.w_all = None
        if rows % 32 == 0 and ops.can_tile(tensors[n["r"]]) and len({tensors[n[s]].dtype for s in keys}) == 1:
            # one matrix, cut where the mixes change: a decode step's five products are one launch over it
            self.w_all = ops.prepare_weight(torch.cat([tensors[n[s]] for s in keys], 0).contiguous())
            self.w = {s: self.w_all.rows_from(i * rows, rows if s != "w1" else self.decay_rank) for i, s in enumerate(keys)}
        else:
            self.w = {s: ops.prepare_weight(tensors[n[s]]) for s in keys}
        self.w["w2"] = ops.prepare_weight(tensors[n["w2"]])
        self.w0 = ops.glu_params(tensors[n["w0"]].as_subclass(torch.Tensor).float().contiguous())
        self.bonus, self.norm, self.wo = tensors[n["u"]], tensors[n["norm"]], ops.prepare_weight(tensors[n["o"]])

    def cache_specs(self):
        return [StateSpec((self.n_heads, self.head_dim, self.head_dim), "float32"), StateSpec((self.hidden_size,), "float32")]

    def _rows(self, h, ctx, views, owns_cache):
        _own_state(owns_cache, "time mixing")
        if h.dtype != torch.float32:
            raise ValueError("time mixing reads float32 rows")
        H, d = self.n_heads, self.head_dim
        c, m, chunked = H * d, h.shape[0], _in_chunks(self, ctx)
        mixes = ops.token_shift(h, self.mu, views[1].state, ctx.pos, ctx.tok_slot, self.dtype, single=ctx.n_tokens == ctx.n_seqs)
        if self.w_all is not None and ctx.is_decode and m <= 16:
            gate = ops.linear_groups(mixes, self.w_all, c)                     # r | k | v | g | w1, float32
            r, k, v = (gate[:, i * c:(i + 1) * c] for i in range(3))
            gate_col, low = 3 * c, ops.cast_columns(gate, 4 * c, self.decay_rank, self.dtype, tanh=True)
        else:
            mix = dict(zip(self.MIXES, mixes))
            # (values in bfloat16, whichever 16-bit type the matrices have, where the recurrence runs in chunks)
            r, k, v = (ops.linear(mix[s], self.w[s], out_dtype=torch.bfloat16 if chunked and s == "v" else torch.float32) for s in "rkv")
            gate, gate_col = ops.linear(mix["g"], self.w["g"], out_dtype=torch.float32), 0
            low = ops.linear(mix["w"], self.w["w1"], ops.EPI_BIAS, out_dtype=self.dtype, params=ops.glu_params(act="tanh"))
        raw = ops.linear(low, self.w["w2"], ops.EPI_BIAS, out_dtype=torch.float32, params=self.w0)
        if not chunked and d <= ops.SCAN_HEAD_LIMIT:       # the norm and gate behind it in the same kernel
            return ops.wkv_scan(r, k, v, raw, self.bonus, views[0].state, ctx, H, d, (self.norm, gate, gate_col, self.norm_eps, self.dtype))
        o = (ops.wkv_chunks if chunked else ops.wkv_scan)(r, k, v, raw, self.bonus, views[0].state, ctx, H, d)
        return ops.gated_head_norm(o, self.norm, gate, gate_col, H, self.norm_eps, self.dtype, gate_silu=True)

    def forward_into(self, h, out, ctx, views, owns_cache=True):
        ops.linear(self._rows(h, ctx, views, owns_cache), self.wo, out=out)
        return None

    def forward(self, h, ctx, views, residual, owns_cache=True):
        ops.linear(self._rows(h, ctx, views, owns_cache), self.wo, ops.EPI_ADD, out=residual)
