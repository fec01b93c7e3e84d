"""Mixers that carry a state of fixed size from token to token, and the mixer that runs two mixers side by side.

State is laid out by position, as all per-request state of the engine is: the token at position p reads place
(p - 1) & 1 of two and writes place p & 1 (position 0 reads nothing, whatever a slot's former holder left), and the
inputs of a convolution of `taps` taps lie at place p mod taps of `taps`. A step of single tokens that is recorded
and run again reads what it read the first time.
"""
from typing import Dict, List, Optional

import torch

from .base import MIXERS, POSITIONS, CacheNeed, Mixer, OffersRows, joined_rows, register_mixer
from .spec import ParamDecl, PartSpec


class _BesideAnother:
    """What a mixer offers so that `side_by_side` can run it beside another: the input of its output product goes
    into a slice of a buffer the two share (`inner_into`, times a factor, before the one rounding), and its
    output matrix is handed over (`out_matrix`) instead of being kept."""

    defer_out = False

    def _keep_out(self, ops, w):
        if self.defer_out:
            self.w_out_raw, self.w_out = w, None
        else:
            self.w_out = ops.prepare_weight(w)

    def out_matrix(self):
        w, self.w_out_raw = self.w_out_raw, None
        return w


@register_mixer("min_gru")
class MinimalGatedRecurrence(_BesideAnother, Mixer):
    """A gated recurrence whose gates read the current token only (minGRU):

        z = sigmoid(W_z h + b_z),  u = W_x h + b_x,  c = u + 1/2 where u >= 0, sigmoid(u) below
        S_t = (1 - z) S_(t-1) + z c      element by element, S = 0 before the first token
        result = W_o (S_t * silu(W_g h))

    The three input matrices are one product; gates, candidate and state are float32."""

    recordable = True

    def __init__(self, width: int, inner: int, names, weight_suffix: str = "", bias_suffix: str = ".b"):
        """`names`: the checkpoint's names of W_z, W_x, W_g and W_o; W_z and W_x have a bias."""
        self.width, self.inner = width, inner
        self.names, self.weight_suffix, self.bias_suffix = tuple(names), weight_suffix, bias_suffix
        if len(self.names) != 4:
            raise ValueError("names: W_z, W_x, W_g and W_o, four names")

    def cache_need(self) -> Optional[CacheNeed]:
        return CacheNeed("state", state_shapes=(("carried", (2, self.inner)),))

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        z, x, g, o = (prefix + n for n in self.names)
        ws, bs = self.weight_suffix, self.bias_suffix
        return [ParamDecl(z + ws, (self.inner, self.width)), ParamDecl(z + bs, (self.inner,), "vector"),
                ParamDecl(x + ws, (self.inner, self.width)), ParamDecl(x + bs, (self.inner,), "vector"),
                ParamDecl(g + ws, (self.inner, self.width)), ParamDecl(o + ws, (self.width, self.inner))]

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        z, x, g, o = (prefix + n for n in self.names)
        ws, bs = self.weight_suffix, self.bias_suffix
        self.w_in = ops.prepare_weight(torch.cat([tensors[z + ws], tensors[x + ws], tensors[g + ws]], dim=0).contiguous())
        self.b_in = torch.cat([tensors[z + bs], tensors[x + bs], torch.zeros_like(tensors[z + bs])]).contiguous()
        self._keep_out(ops, tensors[o + ws])

    def flops_per_token(self, keys: float = 0.0) -> float:
        return super().flops_per_token(keys) + 6.0 * self.inner

    def inner_width(self) -> int:
        return self.inner

    def inner_into(self, h, ctx, cache, out, scale: float):
        proj = self.ops.linear(h, self.w_in, self.b_in, out_f32=True, f32_by_library=True)
        return self.ops.min_gru(proj, self.inner, ctx, cache.state["carried"], out=out, out_scale=scale)

    def forward(self, h, ctx, cache, residual):
        y = self.inner_into(h, ctx, cache, None, 1.0)
        return self.ops.linear(y, self.w_out, None, residual=residual, out_f32=True, f32_by_library=residual is None)


@register_mixer("rglru")
class GatedLinearRecurrence(_BesideAnother, Mixer):
    """Griffin's recurrent block around a real-gated linear recurrent unit. With `inner` channels in `blocks`
    equal parts:

        y = gelu_tanh(W_y h + b_y),   u = conv(W_x h + b_x) + b_conv     (a causal convolution of `taps` taps a channel)
        r = sigmoid(A_b u_b + a_b),   i = sigmoid(I_b u_b + i_b)         (part b of u through square matrices of its own)
        log a = -8 r softplus(lam),   S_t = a S_(t-1) + sqrt(1 - a^2) (i u),   S = 0 before the first token
        result = W_o (S_t * y)

    The first token has no special case. The two input matrices are one product and the two gates' matrices of a
    part are one. Gates, decay and state are float32; the state also keeps the convolution's last `taps - 1`
    inputs."""

    recordable = True

    def __init__(self, width: int, inner: int, blocks: int, taps: int, names, weight_suffix: str = "",
                 bias_suffix: str = ".b"):
        """`names`: the checkpoint's names of W_y, W_x, the convolution `[inner, taps]`, the two gates' matrices
        `[blocks, inner / blocks, inner / blocks]`, lam and W_o; all but lam and W_o have a bias."""
        if inner % blocks or taps < 1:
            raise ValueError(f"a recurrence of {inner} channels in {blocks} parts with {taps} taps")
        self.width, self.inner, self.blocks, self.taps = width, inner, blocks, taps
        self.names, self.weight_suffix, self.bias_suffix = tuple(names), weight_suffix, bias_suffix
        if len(self.names) != 7:
            raise ValueError("names: W_y, W_x, the convolution, the two gates, lam and W_o, seven names")

    def cache_need(self) -> Optional[CacheNeed]:
        shapes = (("carried", (2, self.inner)),)
        if self.taps > 1:
            shapes += (("inputs", (self.taps, self.inner)),)
        return CacheNeed("state", state_shapes=shapes)

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        y, x, conv, ra, ri, lam, o = (prefix + n for n in self.names)
        ws, bs = self.weight_suffix, self.bias_suffix
        c, b = self.inner, self.blocks
        return [ParamDecl(y + ws, (c, self.width)), ParamDecl(y + bs, (c,), "vector"),
                ParamDecl(x + ws, (c, self.width)), ParamDecl(x + bs, (c,), "vector"),
                ParamDecl(conv, (c, self.taps), "vector"), ParamDecl(conv + bs, (c,), "vector"),
                ParamDecl(ra + ws, (b, c // b, c // b)), ParamDecl(ra + bs, (b, c // b), "vector"),
                ParamDecl(ri + ws, (b, c // b, c // b)), ParamDecl(ri + bs, (b, c // b), "vector"),
                ParamDecl(lam, (c,), "vector"), ParamDecl(o + ws, (self.width, c))]

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        y, x, conv, ra, ri, lam, o = (prefix + n for n in self.names)
        ws, bs = self.weight_suffix, self.bias_suffix
        self.w_in = ops.prepare_weight(torch.cat([tensors[y + ws], tensors[x + ws]], dim=0).contiguous())
        self.b_in = torch.cat([tensors[y + bs], tensors[x + bs]]).contiguous()
        self.conv_w, self.conv_b = tensors[conv], tensors[conv + bs]
        # a part's two gates through one product: the rows of A_b, then those of I_b
        self.w_gates = torch.cat([tensors[ra + ws], tensors[ri + ws]], dim=1).contiguous()
        self.b_gates = torch.cat([tensors[ra + bs], tensors[ri + bs]], dim=1).contiguous()
        # log a = r * rate, rate = -8 softplus(lam), made once in float32
        self.rate = (-8.0 * torch.nn.functional.softplus(tensors[lam].float())).contiguous()
        self._keep_out(ops, tensors[o + ws])

    def flops_per_token(self, keys: float = 0.0) -> float:
        return super().flops_per_token(keys) + 2.0 * self.inner * self.taps + 10.0 * self.inner

    def inner_width(self) -> int:
        return self.inner

    def inner_into(self, h, ctx, cache, out, scale: float):
        ops, c = self.ops, self.inner
        proj = ops.linear(h, self.w_in, self.b_in, out_f32=True, f32_by_library=True)
        u, u_compute = ops.channel_conv(proj[:, c:], self.conv_w, self.conv_b, ctx, cache.state.get("inputs"))
        gates = ops.batched_linear(u_compute.view(-1, self.blocks, c // self.blocks), self.w_gates, out_f32=True)
        return ops.gated_linear_recurrence(gates, self.b_gates, u, proj[:, :c], self.rate, ctx, cache.state["carried"],
                                           out=out, out_scale=scale)

    def forward(self, h, ctx, cache, residual):
        y = self.inner_into(h, ctx, cache, None, 1.0)
        return self.ops.linear(y, self.w_out, None, residual=residual, out_f32=True, f32_by_library=residual is None)


class _LinearMemory(Mixer):
    """What the mixers around a linear memory share: a matrix S `[n, v]` a head that is carried from token to token,

        S_t = S' + k w^T,  S' = e^g S_(t-1),  o = S_t^T q,      w = write * val   or   w = write * (val - S'^T k)  (`delta`),

    whose queries, keys and values come out of a short causal convolution over time (`taps` a channel) and silu. Queries
    and keys have `groups` heads, head h takes number floor(h / (heads / groups)). One product makes everything that is
    read of a token, one kernel the convolution, its activation, unit norms, decays and write weights, one walks the
    memory, one makes what the output product reads. Everything between the two products is float32; the state is S and
    the convolution's last `taps - 1` inputs."""

    recordable = True
    delta = False

    def _sizes(self, width, heads, groups, head_size, value_size, taps, eps):
        if heads % groups or taps < 1:
            raise ValueError(f"a linear memory of {heads} heads over {groups} query/key heads with {taps} taps")
        if head_size > 256:
            raise ValueError(f"a linear memory's queries and keys have up to 256 elements a head, got {head_size}")
        self.width, self.heads, self.groups, self.taps, self.eps = width, heads, groups, taps, float(eps)
        self.n, self.v = head_size, value_size
        self.inner = heads * value_size
        self.channels = 2 * groups * head_size + self.inner

    def cache_need(self) -> Optional[CacheNeed]:
        # (a column's rows side by side: what a lane of the kernel holds are neighbours in memory)
        shapes = (("memory", (2, self.heads, self.v, self.n)),)
        if self.taps > 1:
            shapes += (("inputs", (self.taps, self.channels)),)
        return CacheNeed("state", state_shapes=shapes)

    def step_planners(self):
        from ..kernels.memory_plan import memory_plan
        return {"memory": memory_plan}

    def _load_in(self, tensors, names, ops):
        """The rows of the input matrices one under the other, filled up with zero rows to a multiple of 16."""
        w = torch.cat([tensors[n] for n in names], dim=0)
        return ops.prepare_weight(torch.nn.functional.pad(w, (0, 0, 0, -w.shape[0] % 16)).contiguous())

    def flops_per_token(self, keys: float = 0.0) -> float:
        # the memory's update and its product with the query, a head (with `delta` its product with the key too)
        return (super().flops_per_token(keys) + 2.0 * self.channels * self.taps
                + (6.0 if self.delta else 4.0) * self.heads * self.n * self.v)

    def forward(self, h, ctx, cache, residual):
        y = self._inner(self.ops.linear(h, self.w_in, None, out_f32=True, f32_by_library=True), ctx, cache.state)
        return self.ops.linear(y, self.w_out, None, residual=residual, out_f32=True, f32_by_library=residual is None)


@register_mixer("gated_delta")
class GatedDeltaRule(_LinearMemory):
    """The gated delta rule (gated DeltaNet). With q, k of `groups` heads of n elements and val of `heads` heads of v,
    each through a convolution over time and silu, q and k made unit vectors a head and q times n^(-1/2):

        beta = sigmoid(W_b h),   g = -exp(A_log) softplus(W_a h + dt_bias)                     (a number a head each)
        S_t = S' + k_t w_t^T,   S' = e^g S_(t-1),   w_t = beta_t (val_t - S'^T k_t),   o_t = S_t^T q_t

    A head's o at unit root mean square, times `norm` (v elements, the same for all heads), times silu(W_g h);
    W_o on the heads side by side."""

    delta = True

    def __init__(self, width: int, heads: int, groups: int, head_size: int, value_size: int, taps: int, eps: float, names,
                 conv_suffix: str = ".conv", weight_suffix: str = ""):
        """`names`: the checkpoint's names of W_q, W_k, W_v, W_g, W_a, W_b, W_o, A_log, dt_bias and the norm's weight; a
        convolution's weight `[channels, taps]` is its projection's name with `conv_suffix`."""
        self._sizes(width, heads, groups, head_size, value_size, taps, eps)
        self.names, self.conv_suffix, self.weight_suffix = tuple(names), conv_suffix, weight_suffix
        if len(self.names) != 10:
            raise ValueError("names: W_q, W_k, W_v, W_g, W_a, W_b, W_o, A_log, dt_bias and the norm, ten names")

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        q, k, v, g, a, b, o, a_log, dt_bias, norm = (prefix + n for n in self.names)
        ws, cs, h = self.weight_suffix, self.conv_suffix, self.heads
        qk = self.groups * self.n
        return [ParamDecl(q + ws, (qk, self.width)), ParamDecl(q + cs, (qk, self.taps), "vector"),
                ParamDecl(k + ws, (qk, self.width)), ParamDecl(k + cs, (qk, self.taps), "vector"),
                ParamDecl(v + ws, (self.inner, self.width)), ParamDecl(v + cs, (self.inner, self.taps), "vector"),
                ParamDecl(g + ws, (self.inner, self.width)), ParamDecl(a + ws, (h, self.width)),
                ParamDecl(b + ws, (h, self.width)), ParamDecl(o + ws, (self.width, self.inner)),
                ParamDecl(a_log, (h,), "vector"), ParamDecl(dt_bias, (h,), "vector"),
                ParamDecl(norm, (self.v,), "vector", "around_one")]

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        q, k, v, g, a, b, o, a_log, dt_bias, norm = (prefix + n for n in self.names)
        ws, cs = self.weight_suffix, self.conv_suffix
        self.w_in = self._load_in(tensors, [n + ws for n in (q, k, v, g, a, b)], ops)
        self.conv_w = torch.cat([tensors[n + cs] for n in (q, k, v)], dim=0).contiguous()
        self.rate = (-torch.exp(tensors[a_log].float())).contiguous()
        self.dt_bias = tensors[dt_bias]
        self.norm_weight = tensors[norm].repeat(self.heads).contiguous()
        self.w_out = ops.prepare_weight(tensors[o + ws])

    def _inner(self, proj, ctx, state):
        ops, qk, c, h = self.ops, self.groups * self.n, self.channels, self.heads
        at = c + self.inner                                     # the columns: q | k | v | gate | a | b
        u, decay, write = ops.memory_inputs(proj, 0, self.conv_w, None, ctx, state.get("inputs"), h, at, self.rate,
                                            self.dt_bias, write_at=at + h, unit=(self.n, 2 * qk, qk, self.n ** -0.5))
        o = ops.linear_memory(u, 0, qk, 2 * qk, h, self.groups, self.n, self.v, decay, write, ctx, state["memory"], True)
        return ops.gated_norm(o, proj[:, c:c + self.inner], self.norm_weight, self.eps, h, False)


@register_mixer("state_space")
class StateSpace(_LinearMemory):
    """A selective state space with one decay a head (Mamba-2). W_in h is laid out [z | x | B | C | dt]: z and x of
    `heads` heads of v elements, B and C of `groups` heads of n, dt a number a head. x, B and C together pass a convolution
    over time with a bias, and silu; dt <- softplus(dt + dt_bias):

        S <- exp(-exp(A_log) dt) S + dt B x^T,   y = S^T C + D x

    The heads' y side by side times silu(z), in `norm_groups` equal parts at unit root mean square, times `norm`; W_o."""

    def __init__(self, width: int, heads: int, groups: int, head_size: int, value_size: int, taps: int, norm_groups: int,
                 eps: float, names, bias_suffix: str = ".b", weight_suffix: str = ""):
        """`head_size`: n, the size of B and C. `names`: the checkpoint's names of W_in, the convolution (its bias: with
        `bias_suffix`), dt_bias, A_log, D, the norm's weight and W_o."""
        self._sizes(width, heads, groups, head_size, value_size, taps, eps)
        if self.inner % norm_groups:
            raise ValueError(f"{self.inner} elements do not divide into {norm_groups} equal parts")
        self.norm_groups, self.names = norm_groups, tuple(names)
        self.bias_suffix, self.weight_suffix = bias_suffix, weight_suffix
        if len(self.names) != 7:
            raise ValueError("names: W_in, the convolution, dt_bias, A_log, D, the norm and W_o, seven names")

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        w_in, conv, dt_bias, a_log, d, norm, o = (prefix + n for n in self.names)
        ws = self.weight_suffix
        return [ParamDecl(w_in + ws, (self.inner + self.channels + self.heads, self.width)),
                ParamDecl(conv, (self.channels, self.taps), "vector"),
                ParamDecl(conv + self.bias_suffix, (self.channels,), "vector"),
                ParamDecl(dt_bias, (self.heads,), "vector"), ParamDecl(a_log, (self.heads,), "vector"),
                ParamDecl(d, (self.heads,), "vector", "around_one"), ParamDecl(norm, (self.inner,), "vector", "around_one"),
                ParamDecl(o + ws, (self.width, self.inner))]

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        w_in, conv, dt_bias, a_log, d, norm, o = (prefix + n for n in self.names)
        self.w_in = self._load_in(tensors, [w_in + self.weight_suffix], ops)
        self.conv_w, self.conv_b = tensors[conv], tensors[conv + self.bias_suffix]
        self.rate = (-torch.exp(tensors[a_log].float())).contiguous()
        self.dt_bias, self.skip, self.norm_weight = tensors[dt_bias], tensors[d], tensors[norm]
        self.w_out = ops.prepare_weight(tensors[o + self.weight_suffix])

    def _inner(self, proj, ctx, state):
        ops, i, gn = self.ops, self.inner, self.groups * self.n
        u, decay, write = ops.memory_inputs(proj, i, self.conv_w, self.conv_b, ctx, state.get("inputs"), self.heads,
                                            i + self.channels, self.rate, self.dt_bias)
        o = ops.linear_memory(u, i + gn, i, 0, self.heads, self.groups, self.n, self.v, decay, write, ctx, state["memory"],
                              False)
        return ops.gated_norm(o, proj[:, :i], self.norm_weight, self.eps, self.norm_groups, True, skip=(self.skip, u[:, :i]))


class _PlainMemory(OffersRows, _BesideAnother, Mixer):
    """What the mixers around a linear memory without convolutions share: per head a matrix S `[n, v]` that is carried
    from token to token,

        S_t = diag(e^(g_t)) S_(t-1) + k_t v_t^T,   o_t = S_t^T q_t,   g_t a number a head or one a row of S,

    read straight off the float32 rows of one input product (queries, keys, values, gates, and what a mixer adds); each
    head's o at unit root mean square, times a weight or not, times silu(W_g h); W_o. The factor n^(-1/2) that the
    designs put on queries or keys scales every o of a head alike, and the norm takes it off again up to eps: it is not
    multiplied in anywhere, the norm's eps is n times as large instead. Everything between the two products is float32."""

    recordable = True

    def _sizes(self, width, heads, head_size, value_size, eps):
        if head_size > 256:
            raise ValueError(f"a linear memory's queries and keys have up to 256 elements a head, got {head_size}")
        self.width, self.heads, self.n, self.v, self.eps = width, heads, head_size, value_size, float(eps)
        self.qk, self.inner = heads * head_size, heads * value_size

    def cache_need(self) -> Optional[CacheNeed]:
        # (a column's rows side by side: what a lane of the kernel holds are neighbours in memory)
        return CacheNeed("state", state_shapes=(("memory", (2, self.heads, self.v, self.n)),))

    def step_planners(self):
        from ..kernels.memory_plan import memory_plan
        return {"memory": memory_plan}

    def _load_in(self, tensors, names, ops):
        """The rows of the input matrices one under the other, filled up with zero rows to a multiple of 16."""
        w = torch.cat([tensors[n] for n in names], dim=0)
        self._keep_in(ops, torch.nn.functional.pad(w, (0, 0, 0, -w.shape[0] % 16)).contiguous())

    def inner_width(self) -> int:
        return self.inner

    def _decays(self, proj, ctx):
        """The decays' logarithms as `ops.linear_memory` takes them, after anything else that is done to `proj`."""
        raise NotImplementedError

    def inner_into(self, h, ctx, cache, out, scale: float, rows=None):
        ops, qk = self.ops, self.qk
        proj = self._rows(h, rows)
        decay = self._decays(proj, ctx)
        at = 2 * qk + self.inner                                # the columns: q | k | v | gate | ...
        o = ops.linear_memory(proj[:, :at], 0, qk, 2 * qk, self.heads, self.heads, self.n, self.v, decay, None, ctx,
                              cache.state["memory"], False)
        return ops.gated_norm(o, proj[:, at:at + self.inner], self.norm_weight, self.eps * self.n, self.heads, False,
                              out=out, out_scale=scale)

    def forward(self, h, ctx, cache, residual, rows=None):
        y = self.inner_into(h, ctx, cache, None, 1.0, rows)
        return self.ops.linear(y, self.w_out, None, residual=residual, out_f32=True, f32_by_library=residual is None)


@register_mixer("gated_linear_attention")
class GatedLinearAttention(_PlainMemory):
    """Gated linear attention: queries W_q h n^(-1/2), keys W_k h and values W_v h of `heads` heads, and a decay for every
    row of S, e^g = sigmoid(z)^(1/tau) with z = W_a2 (W_a1 h) + b. Each head's o is normed with a weight of v elements
    that all heads share. The inner size of the two small matrices (`rank`) is the checkpoint's if not given."""

    def __init__(self, width: int, heads: int, head_size: int, value_size: int, tau: float, eps: float, names,
                 rank: Optional[int] = None, weight_suffix: str = "", bias_suffix: str = ".b"):
        """`names`: the checkpoint's names of W_q, W_k, W_v, W_g, W_o, W_a1, W_a2 (its bias: with `bias_suffix`) and the
        norm's weight."""
        self._sizes(width, heads, head_size, value_size, eps)
        self.tau, self.rank = float(tau), rank
        if not self.tau > 0:
            raise ValueError(f"gated linear attention: tau must be positive, got {tau}")
        self.names, self.weight_suffix, self.bias_suffix = tuple(names), weight_suffix, bias_suffix
        if len(self.names) != 8:
            raise ValueError("names: W_q, W_k, W_v, W_g, W_o, W_a1, W_a2 and the norm, eight names")

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        q, k, v, g, o, a1, a2, norm = (prefix + n for n in self.names)
        ws = self.weight_suffix
        return [ParamDecl(q + ws, (self.qk, self.width)), ParamDecl(k + ws, (self.qk, self.width)),
                ParamDecl(v + ws, (self.inner, self.width)), ParamDecl(g + ws, (self.inner, self.width)),
                ParamDecl(o + ws, (self.width, self.inner)), ParamDecl(a1 + ws, (self.rank, self.width)),
                ParamDecl(a2 + ws, (self.qk, self.rank)), ParamDecl(a2 + self.bias_suffix, (self.qk,), "vector"),
                ParamDecl(norm, (self.v,), "vector", "around_one")]

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        q, k, v, g, o, a1, a2, norm = (prefix + n for n in self.names)
        ws = self.weight_suffix
        self.rank = tensors[a1 + ws].shape[0]
        if tuple(tensors[a2 + ws].shape) != (self.qk, self.rank):
            raise ValueError(f"{a2}{ws} is {tuple(tensors[a2 + ws].shape)}, behind a matrix of {self.rank} rows it must be "
                             f"{(self.qk, self.rank)}")
        self._load_in(tensors, [n + ws for n in (q, k, v, g, a1)], ops)
        self.w_decay, self.b_decay = tensors[a2 + ws].contiguous(), tensors[a2 + self.bias_suffix]
        self.norm_weight = tensors[norm].repeat(self.heads).contiguous()
        self._keep_out(ops, tensors[o + ws])

    def flops_per_token(self, keys: float = 0.0) -> float:
        rank = self.rank or 0
        return (2.0 * self.width * (2 * self.qk + 3 * self.inner + rank) + 2.0 * self.qk * rank
                + 4.0 * self.heads * self.n * self.v)

    def _decays(self, proj, ctx):
        at = 2 * (self.qk + self.inner)
        return self.ops.channel_decays(proj[:, at:at + self.rank], self.w_decay, self.b_decay, self.tau)


@register_mixer("retention")
class Retention(_PlainMemory):
    """Retention: queries and keys turned by the position, keys times n^(-1/2), a decay a head that does not depend on the
    token, no weight behind the norm."""

    def __init__(self, width: int, heads: int, head_size: int, value_size: int, decay, eps: float, names, rotation=None,
                 weight_suffix: str = ""):
        """`decay`: a number a head, the factor itself. `names`: the checkpoint's names of W_q, W_k, W_v, W_g and W_o;
        `rotation`: a position encoding that gives `frequencies()`, or None."""
        self._sizes(width, heads, head_size, value_size, eps)
        self.decay = tuple(float(x) for x in decay)
        if len(self.decay) != heads or not all(0 < x <= 1 for x in self.decay):
            raise ValueError(f"retention: {heads} decays in (0, 1], got {self.decay}")
        self.rotation = POSITIONS.build(rotation) if rotation is not None else None
        if self.rotation is not None and (not hasattr(self.rotation, "frequencies") or self.rotation.dims > head_size):
            raise ValueError("retention turns its heads by a rotation that gives `frequencies()` for no more than their elements")
        self.names, self.weight_suffix = tuple(names), weight_suffix
        if len(self.names) != 5:
            raise ValueError("names: W_q, W_k, W_v, W_g and W_o, five names")

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        q, k, v, g, o = (prefix + n + self.weight_suffix for n in self.names)
        return [ParamDecl(q, (self.qk, self.width)), ParamDecl(k, (self.qk, self.width)),
                ParamDecl(v, (self.inner, self.width)), ParamDecl(g, (self.inner, self.width)),
                ParamDecl(o, (self.width, self.inner))]

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        q, k, v, g, o = (prefix + n + self.weight_suffix for n in self.names)
        self._load_in(tensors, [q, k, v, g], ops)
        # (logarithms made in float64 and rounded once)
        self.log_decay = torch.log(torch.tensor(self.decay, dtype=torch.float64)).float().to(tensors[q].device)
        self.freqs = None
        if self.rotation is not None and self.rotation.dims > 0:
            self.rotation.load(tensors, prefix + "rotation", ops, dtype)
            self.freqs = self.rotation.frequencies()
        self.norm_weight = None
        self._keep_out(ops, tensors[o])

    def flops_per_token(self, keys: float = 0.0) -> float:
        return super().flops_per_token(keys) + 4.0 * self.heads * self.n * self.v

    def _decays(self, proj, ctx):
        if self.freqs is not None:
            self.ops.turn_heads(proj, 0, 2 * self.heads, self.n, self.freqs, self.rotation.interleaved, ctx)
        return self.log_decay


class _SubCache:
    """The part of a call's cache that one of two mixers side by side sees: the pages as they are, and of the
    state the tensors under its own prefix, named as the mixer names them."""

    def __init__(self, cache, prefix: str):
        self.cache_id, self.group, self.writes, self.pages = cache.cache_id, cache.group, cache.writes, cache.pages
        self.state = {k[len(prefix):]: v for k, v in cache.state.items() if k.startswith(prefix)}

    k_pages = property(lambda self: self.pages.get("k"))
    v_pages = property(lambda self: self.pages.get("v"))


@register_mixer("side_by_side")
class SideBySide(OffersRows, Mixer):
    """Two mixers that read the same input, `left_scale * left(h) + right_scale * right(h)`.

    Both end in an output product; the two are made one: each mixer writes what its output matrix reads, times
    its factor, into its own columns of one buffer (`inner_into`), and the product of that buffer with the two
    output matrices side by side is the weighted sum, added up in float32. At most one of the two keeps pages;
    the state of both lives in the one cache of the call, under the prefixes `left.` and `right.`. Where both offer the
    rows of their input product (`OffersRows`), the two input products are one as well.

    With `out_norms` = {eps, left, right} each of the two results is first scaled to unit root mean square over the
    width and weighted (the tensors `left` and `right`, names under the mixer's prefix): each mixer then keeps its own
    output product, and the norms and the sum are the arrangement's (`results`) or, in `forward`, a launch a norm."""

    def __init__(self, left: PartSpec, right: PartSpec, left_name: str = "left.", right_name: str = "right.",
                 left_scale: float = 1.0, right_scale: float = 1.0, out_norms=None):
        self.left, self.right = MIXERS.build(left), MIXERS.build(right)
        self.out_norms = dict(out_norms) if out_norms else None
        for m in (self.left, self.right) if self.out_norms is None else ():
            if not hasattr(m, "inner_into"):
                raise ValueError(f"mixer {m.kind!r} cannot run beside another: it has no `inner_into`")
            m.defer_out = True
        if self.offers_rows:
            self.left.defer_in = self.right.defer_in = True
        self.left_name, self.right_name = left_name, right_name
        self.left_scale, self.right_scale = float(left_scale), float(right_scale)
        self.recordable = bool(getattr(self.left, "recordable", False) and getattr(self.right, "recordable", False))
        self._subs = {}

    @property
    def offers_rows(self) -> bool:
        return self.out_norms is None and all(getattr(m, "offers_rows", False) for m in (self.left, self.right))

    def cache_need(self) -> Optional[CacheNeed]:
        needs = [(m.cache_need(), p) for m, p in ((self.left, "left."), (self.right, "right."))]
        paged = [n for n, _ in needs if n is not None and n.kind == "paged"]
        if len(paged) > 1:
            raise ValueError("of two mixers side by side at most one keeps pages")
        state = tuple((p + name, shape) for n, p in needs if n is not None for name, shape in n.state_shapes)
        if paged:
            n = paged[0]
            return CacheNeed("paged", n.kv_heads, n.head_size, n.window, state, "float32", n.page_tensors)
        return CacheNeed("state", state_shapes=state) if state else None

    def param_decls(self, prefix: str) -> List[ParamDecl]:
        d = self.left.param_decls(prefix + self.left_name) + self.right.param_decls(prefix + self.right_name)
        if self.out_norms:
            d += [ParamDecl(prefix + self.out_norms[side], (self.left.width,), "vector", "around_one")
                  for side in ("left", "right")]
        return d

    def load(self, tensors: Dict, prefix: str, ops, dtype) -> None:
        super().load(tensors, prefix, ops, dtype)
        self.left.load(tensors, prefix + self.left_name, ops, dtype)
        self.right.load(tensors, prefix + self.right_name, ops, dtype)
        if self.out_norms:
            self.norm_weights = [tensors[prefix + self.out_norms[side]] for side in ("left", "right")]
            return
        if self.offers_rows:
            w, bias, self.places = joined_rows((self.left, self.right))
            self._keep_in(ops, w, bias)
        self.split = self.left.inner_width()
        self.w_out = ops.prepare_weight(torch.cat([self.left.out_matrix(), self.right.out_matrix()], dim=1).contiguous())

    def step_planners(self):
        return {**self.left.step_planners(), **self.right.step_planners()}

    def launch_shape(self, step):
        return (self.left.launch_shape(step), self.right.launch_shape(step))

    def flops_per_token(self, keys: float = 0.0) -> float:
        return self.left.flops_per_token(keys) + self.right.flops_per_token(keys)

    def _parts(self, cache):
        subs = self._subs.get(id(cache))
        if subs is None or subs[0] is not cache:
            subs = self._subs[id(cache)] = (cache, _SubCache(cache, "left."), _SubCache(cache, "right."))
        return subs

    def results(self, h, ctx, cache):
        if not self.out_norms:
            return super().results(h, ctx, cache)
        subs, eps = self._parts(cache), float(self.out_norms["eps"])
        return [(m.forward(h, ctx, sub, None), w, eps, scale) for m, sub, w, scale in
                zip((self.left, self.right), subs[1:], self.norm_weights, (self.left_scale, self.right_scale))]

    def forward(self, h, ctx, cache, residual, rows=None):
        if self.out_norms:
            x = residual
            for y, w, eps, scale in self.results(h, ctx, cache):
                x = self.ops.norm_add(y, w, None, eps, False, torch.zeros_like(y) if x is None else x, scale)
            return x
        subs = self._parts(cache)
        both = torch.empty(h.shape[0], self.split + self.right.inner_width(), dtype=self.dtype, device=self.ops.device)
        left, right = {}, {}
        if self.offers_rows:
            rows = self._rows(h, rows)
            left, right = ({"rows": rows[:, a:b]} for a, b in self.places)
        self.left.inner_into(h, ctx, subs[1], both[:, :self.split], self.left_scale, **left)
        self.right.inner_into(h, ctx, subs[2], both[:, self.split:], self.right_scale, **right)
        return self.ops.linear(both, self.w_out, None, residual=residual, out_f32=True, f32_by_library=residual is None)
