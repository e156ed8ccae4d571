"""Token mixers of a hybrid decoder: linear recurrences (decayed sum, gated delta rule, decays per head or key channel),
latent attention, grouped attention, and mixers side by side.

A mixer names the projections of its input that the layer computes in one product (``inputs``), and turns a row block of
them into its read-out, before the output projection.  Everything a design may choose is a constructor argument."""
from __future__ import annotations

import math

import torch
import torch.nn as nn

from . import _lib, mixer_ops as M
from .cache import GroupedCache, JoinedState, LatentCache, RecurrentState
from .model import rope_tables


class Workspace:
    """Scratch memory that grows to the largest request; one per model, used by one kernel chain at a time."""

    def __init__(self, device):
        self.device, self.buf = device, None

    def get(self, nbytes: int) -> torch.Tensor:
        if self.buf is None or self.buf.numel() < nbytes:
            self.buf = torch.empty(nbytes, dtype=torch.uint8, device=self.device)
        return self.buf


class Mixer(nn.Module):
    """inputs: (tensor name, rows) of the input projections, in the order they are stacked; width: of the read-out."""
    inputs: list
    width: int

    def fit(self, shapes: dict) -> None:
        """Sizes that only the checkpoint's tensors give (name -> shape)."""

    def weight_shapes(self, dim: int) -> dict:
        """Name -> shape of all tensors, the input and output projections included."""
        raise NotImplementedError

    def output(self, weights: dict) -> torch.Tensor:
        """Takes the projection of the read-out out of the tensors by name."""
        return weights.pop("o")

    def bind(self, weights: dict, offsets: dict, eps: float) -> None:
        """Tensors by name, and the column of every input projection in the stacked product."""
        raise NotImplementedError

    def new_state(self, max_seq: int, dtype, device):
        raise NotImplementedError

    def forward(self, proj, state, pos, start, out):
        """proj [rows, ld] -> out [rows, width] (its rows may be apart); pos: position of the first row on the device, start:
        the same on the host (None in a one-token step, which may be captured)."""
        raise NotImplementedError


class LinearRecurrence(Mixer):
    """S <- decay S + k v^T, or the gated delta rule behind short convolutions (``conv``).  Decays: constants per head
    (``decay``), per head from the input (the delta rule alone), or per head and key channel from a low-rank map of the input
    (``channel``): sigmoid(z)^(1 / tau), or exp(-exp(A_log) softplus(z)) where no tau is given.  The read-out is RMS-normed
    per head, or over all heads with constant decays, and gated (``gate``) by a projection of the input, or by a low-rank one
    (``low_rank_gate``)."""

    def __init__(self, heads: int, dim: int, vdim: int, workspace: Workspace, kv_heads=None, decay=None, conv: int = 0,
                 channel: bool = False, tau=None, gate: int = M.GATE_SILU, low_rank_gate: bool = False, out_scale: float = 1.0):
        super().__init__()
        self.heads, self.dim, self.vdim, self.kv_heads = heads, dim, vdim, kv_heads or heads
        self.delta, self.channel, self.tau, self.taps, self.workspace = conv > 0, channel, tau, conv, workspace
        if (decay is not None) + (channel or self.delta) != 1:
            raise ValueError("a recurrence has either constant decays, or decays per channel, or a convolution in front of a delta rule")
        if channel and self.delta == (tau is not None):
            raise ValueError("decays per channel take tau without the delta rule and A_log with it")
        if low_rank_gate and not channel:
            raise ValueError("a low-rank gate goes with decays per channel")
        if decay is not None and len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        if heads % self.kv_heads:
            raise ValueError(f"{heads} heads do not divide into {self.kv_heads} key heads")
        # a power of every distance inside a chunk, rounded once
        self.powers = None if decay is None else torch.tensor([[float(d) ** n for n in range(65)] for d in decay], dtype=torch.float64).float()
        self.width = heads * vdim
        # the read-out is normed over all heads together, or head by head with one shared weight
        self.groups, self.gate = (1 if decay is not None else heads), gate
        self.low_rank_gate, self.out_scale = low_rank_gate, out_scale
        self.rank_a = self.rank_g = dim                    # unless the tensors say otherwise

    def fit(self, shapes):
        rows = lambda n, default: shapes[n][0] if len(shapes.get(n, ())) == 2 else default
        self.rank_a, self.rank_g = rows("a1", self.rank_a), rows("g1", self.rank_g)

    @property
    def inputs(self):
        nqk = self.kv_heads * self.dim
        rows = [("q", nqk), ("k", nqk), ("v", self.width), ("g1", self.rank_g) if self.low_rank_gate else ("g", self.width)]
        rows += [("b", self.heads)] if self.delta else []
        return rows + ([("a1", self.rank_a)] if self.channel else [("a", self.heads)] if self.delta else [])

    def weight_shapes(self, dim):
        s = {n: (r, dim) for n, r in self.inputs}
        s["o"], s["norm"] = (dim, self.width), (self.width // self.groups,)
        nh, rows = self.heads * self.dim, dict(self.inputs)
        if self.delta:
            s.update({n + ".conv": (rows[n], self.taps) for n in "qkv"})
            s["A_log"], s["dt_bias"] = (self.heads,), (nh if self.channel else self.heads,)
        if self.channel:
            s["a2"] = (nh, self.rank_a)
            if not self.delta:
                s["a2.b"] = (nh,)
        if self.low_rank_gate:
            s["g2"] = (self.width, self.rank_g)
        return s

    def bind(self, weights, offsets, eps):
        self.eps, self.norm = eps, weights["norm"]
        self.fused = self.groups == self.heads and M.recurrence_step_fuses(self.dim, self.vdim)
        names = {"g1": "g", "a1": "a"}
        p = _lib.Recurrence(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, taps=max(self.taps, 1),
                            delta=int(self.delta), channel=int(self.channel), out_scale=self.out_scale,
                            **{"off_" + names.get(n, n): offsets[n] for n, _ in self.inputs})
        self.keep = [self.norm]

        def put(field, t):
            setattr(p, field, t.data_ptr())
            self.keep.append(t)
        if self.delta:
            for n in "qkv":
                put("conv_" + n, weights[n + ".conv"])
        if self.channel:
            p.rank_a, p.a_sign = self.rank_a, -1.0 if self.tau is not None else 1.0
            self.a2, self.g2 = weights["a2"], weights.get("g2")
            put("a2", self.a2)
            put("a_bias", weights["dt_bias" if self.delta else "a2.b"].float().contiguous())
            put("rate", weights["A_log"].float().exp() if self.delta else
                torch.full((self.heads,), 1.0 / self.tau, dtype=torch.float32, device=self.norm.device))
            if self.low_rank_gate:
                p.rank_g = self.rank_g
                put("g2", self.g2)
        elif self.delta:
            put("A_log", weights["A_log"])
            put("dt_bias", weights["dt_bias"])
        else:
            self.powers = self.powers.to(self.norm.device)
            put("decay", self.powers)
        self.params = p

    def new_state(self, max_seq, dtype, device):
        chans = 2 * self.kv_heads * self.dim + self.heads * self.vdim
        return RecurrentState(self.heads, self.dim, self.vdim, device, self.taps, chans, dtype)

    def forward(self, proj, state, pos, start, out):
        p, rows = self.params, proj.shape[0]
        p.proj, p.ld, p.pos, p.state = proj.data_ptr(), proj.shape[1], pos.data_ptr(), state.state.data_ptr()
        p.ring = state.ring.data_ptr() if state.ring is not None else None
        if rows == 1 and self.fused:
            M.recurrence_step(p, proj.dtype, out=out, norm_weight=self.norm, eps=self.eps, kind=self.gate)
            return
        o = torch.empty(rows, self.width, dtype=torch.float32, device=proj.device)
        if rows == 1:
            M.recurrence_step(p, proj.dtype, o=o)
        else:
            if self.channel:                               # every channel's decay before its softplus, in float32
                z = product_f32(proj[:, p.off_a:p.off_a + self.rank_a], self.a2)
                p.a = z.data_ptr()
            M.recurrence_rows(p, proj.dtype, o, self.workspace.get(M.recurrence_workspace(p, rows)), rows)
        gate, ld = proj[:, p.off_g:], p.ld
        if self.low_rank_gate:
            gate, ld = torch.empty(rows, self.width, dtype=proj.dtype, device=proj.device), self.width
            low = proj[:, p.off_g:p.off_g + self.rank_g]
            M.gemv(self.g2, low, gate) if rows == 1 else torch.mm(low, self.g2.t(), out=gate)
        M.group_norm_gate(o, gate, ld, self.norm, out, self.groups, self.eps, self.gate, self.out_scale)


def product_f32(x: torch.Tensor, w: torch.Tensor) -> torch.Tensor:
    """x @ w^T with a float32 result."""
    return torch.mm(x, w.t()) if x.dtype == torch.float32 else torch.mm(x, w.t(), out_dtype=torch.float32)


class LatentAttention(Mixer):
    """Causal attention whose keys and values are linear in one cached latent per token; a rotated key part is shared by
    the heads; a per-head sink may join the softmax's denominator."""

    def __init__(self, heads: int, dim: int, rot_dim: int, vdim: int, kv_rank: int, scale: float, rope_base: float,
                 workspace: Workspace, rope_dims=None, rope_scaling=None, sink: bool = True):
        super().__init__()
        self.heads, self.dim, self.rot, self.vdim, self.rank, self.scale = heads, dim, rot_dim, vdim, kv_rank, scale
        self.rope = dict(dims=rope_dims or rot_dim, base=rope_base, scaling=rope_scaling)
        self.sink, self.workspace = sink, workspace
        self.inputs = [("q", heads * (dim + rot_dim)), ("dkv", kv_rank + rot_dim)]
        self.width = heads * vdim

    def weight_shapes(self, dim):
        s = {n: (r, dim) for n, r in self.inputs}
        s.update({"dkv.norm": (self.rank,), "uk": (self.heads * self.dim, self.rank), "uv": (self.width, self.rank), "o": (dim, self.width)})
        if self.sink:
            s["sink"] = (self.heads,)
        return s

    def bind(self, weights, offsets, eps):
        self.uk, self.uv = weights["uk"], weights["uv"]
        self.keep = [weights["dkv.norm"], weights.get("sink")]
        self.params = _lib.Latent(off_q=offsets["q"], off_c=offsets["dkv"], heads=self.heads, dim=self.dim, rot=self.rot, vdim=self.vdim,
                                  rank=self.rank, eps=eps, scale=self.scale, norm=weights["dkv.norm"].data_ptr(), uk=self.uk.data_ptr(),
                                  uv=self.uv.data_ptr(), sink=weights["sink"].data_ptr() if self.sink else None)

    def new_state(self, max_seq, dtype, device):
        cache = LatentCache(max_seq, self.rank, self.rot, dtype, device)
        rows = cache.rows.shape[0]
        # angles and tables: one for all layer runs of this mixer
        if getattr(self, "tables", None) is None or self.tables[0].shape[0] != rows:
            self.tables = rope_tables(self.rot, rows, self.rope["base"], device, layout="pairs", dims=self.rope["dims"],
                                      scaling=self.rope["scaling"])
            self.params.cos_table, self.params.sin_table = (t.data_ptr() for t in self.tables)
            self.params.max_seq = rows
            self.step_space = torch.empty(M.latent_step_workspace(self.params), dtype=torch.uint8, device=device)
        return cache

    def forward(self, proj, state, pos, start, out):
        p, rows, dt = self.params, proj.shape[0], proj.dtype
        p.proj, p.ld, p.pos, p.cache = proj.data_ptr(), proj.shape[1], pos.data_ptr(), state.rows.data_ptr()
        if rows == 1:
            M.latent_step(p, dt, out, self.step_space)
            return
        q = torch.empty(rows, self.heads, self.dim + self.rot, dtype=dt, device=proj.device)
        M.latent_append(p, dt, q, rows)
        keys = start + rows
        # unrotated keys, and the values transposed (rows of the cache past the sequence are finite and never weighted)
        k = torch.mm(state.rows[:keys, :self.rank], self.uk.t())
        vt = torch.mm(self.uv, state.rows[:(keys + 63) // 64 * 64, :self.rank].t())
        M.latent_attention(p, dt, q, k, vt, out, start, rows)


class GroupedAttention(Mixer):
    """Causal attention whose query heads share key / value heads; queries and keys may be RMS-normed per head, the first
    ``rope_dims`` elements of a head turn, a valueless score may join the softmax's denominator (``sink``, None: none), and
    the read-out of every head may be gated by one projection of the input."""

    def __init__(self, heads: int, kv_heads: int, dim: int, vdim: int, scale: float, rope_base: float, rope_dims=None, rope_scaling=None,
                 qk_norm: bool = True, sink=None, gated: bool = True, out_scale: float = 1.0):
        super().__init__()
        if heads % kv_heads:
            raise ValueError(f"{heads} heads do not divide into {kv_heads} key heads")
        self.heads, self.kv_heads, self.dim, self.vdim, self.scale = heads, kv_heads, dim, vdim, scale
        self.rope = dict(dims=dim if rope_dims is None else rope_dims, base=rope_base, scaling=rope_scaling)
        self.qk_norm, self.sink, self.gated, self.out_scale = qk_norm, sink, gated, out_scale
        self.inputs = [("q", heads * dim), ("k", kv_heads * dim), ("v", kv_heads * vdim)] + ([("g", heads)] if gated else [])
        self.width = heads * vdim

    def weight_shapes(self, dim):
        s = {n: (r, dim) for n, r in self.inputs}
        s["o"] = (dim, self.width)
        if self.qk_norm:
            s["q.norm"] = s["k.norm"] = (self.dim,)
        return s

    def bind(self, weights, offsets, eps):
        self.keep = [weights.get("q.norm"), weights.get("k.norm")]
        ptr = lambda t: None if t is None else t.data_ptr()
        self.params = _lib.Grouped(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, rot=self.rope["dims"],
                                   gated=int(self.gated), eps=eps, scale=self.scale, sink=-math.inf if self.sink is None else self.sink,
                                   out_scale=self.out_scale, q_norm=ptr(self.keep[0]), k_norm=ptr(self.keep[1]),
                                   **{"off_" + n: offsets[n] for n, _ in self.inputs})

    def new_state(self, max_seq, dtype, device):
        cache = GroupedCache(max_seq, self.kv_heads, self.dim, self.vdim, dtype, device)
        # angles and scratch memory: one for all layer runs of this mixer
        if getattr(self, "tables", None) is None or self.tables[0].shape[0] != cache.positions:
            dims = self.rope["dims"]
            self.tables = rope_tables(dims, cache.positions, self.rope["base"], device, layout="pairs", scaling=self.rope["scaling"])
            self.params.cos_table, self.params.sin_table = (t.data_ptr() if dims else None for t in self.tables)
            self.params.max_seq = cache.positions
            self.step_space = torch.empty(M.grouped_step_workspace(self.params), dtype=torch.uint8, device=device)
        return cache

    def forward(self, proj, state, pos, start, out):
        p, rows, dt = self.params, proj.shape[0], proj.dtype
        p.proj, p.ld, p.pos, p.keys, p.values = proj.data_ptr(), proj.shape[1], pos.data_ptr(), state.keys.data_ptr(), state.values.data_ptr()
        if rows == 1:
            M.grouped_step(p, dt, out, self.step_space)
            return
        q = torch.empty(rows, self.heads, self.dim, dtype=dt, device=proj.device)
        M.grouped_append(p, dt, q, rows)
        M.grouped_attention(p, dt, q, out, start, rows)


class SideBySide(Mixer):
    """Mixers that read the same input, their results added (the mixers scale their own read-outs): tensors by 'side.name',
    the output projections side by side in one matrix."""

    def __init__(self, sides: dict):
        super().__init__()
        self.sides = nn.ModuleDict(sides)
        self.width = sum(m.width for m in sides.values())

    @staticmethod
    def _of(side, by_name):
        return {n[len(side) + 1:]: x for n, x in by_name.items() if n.startswith(side + ".")}

    def fit(self, shapes):
        for side, m in self.sides.items():
            m.fit(self._of(side, shapes))

    @property
    def inputs(self):
        return [(f"{side}.{n}", r) for side, m in self.sides.items() for n, r in m.inputs]

    def weight_shapes(self, dim):
        return {f"{side}.{n}": s for side, m in self.sides.items() for n, s in m.weight_shapes(dim).items()}

    def output(self, weights):
        return torch.cat([weights.pop(side + ".o") for side in self.sides], 1)

    def bind(self, weights, offsets, eps):
        for side, m in self.sides.items():
            m.bind(self._of(side, weights), self._of(side, offsets), eps)

    def new_state(self, max_seq, dtype, device):
        return JoinedState([m.new_state(max_seq, dtype, device) for m in self.sides.values()])

    def forward(self, proj, state, pos, start, out):
        at = 0
        for m, s in zip(self.sides.values(), state.parts):
            m(proj, s, pos, start, out[:, at:at + m.width])
            at += m.width


def lightning(cfg: dict, workspace: Workspace) -> LinearRecurrence:
    return LinearRecurrence(cfg["heads"], cfg["dim"], cfg["vdim"], workspace, decay=cfg["decay"], gate=M.GATE_SIGMOID)


def delta(cfg: dict, workspace: Workspace) -> LinearRecurrence:
    return LinearRecurrence(cfg["heads"], cfg["dim"], cfg["vdim"], workspace, kv_heads=cfg["kv_heads"], conv=cfg["conv"])


def channel_delta(cfg: dict, workspace: Workspace) -> LinearRecurrence:
    return LinearRecurrence(cfg["heads"], cfg["dim"], cfg["vdim"], workspace, kv_heads=cfg["kv_heads"], conv=cfg["conv"], channel=True,
                            gate=M.GATE_SIGMOID, low_rank_gate=True)


def latent_attention(cfg: dict, workspace: Workspace) -> LatentAttention:
    rot = cfg["rot"]
    return LatentAttention(cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"], cfg["scale"], rot["base"], workspace,
                           rope_dims=rot.get("dims"), rope_scaling=rot.get("scaling"))


def parallel(cfg: dict, workspace: Workspace) -> SideBySide:
    """Grouped attention with a sink of score 0 beside gated linear attention with decays per key channel."""
    l, r = cfg["left"], cfg["right"]
    left = GroupedAttention(l["heads"], l["kv_heads"], l["dim"], l["vdim"], l["scale"], l["rot"]["base"], rope_dims=l["rot"]["dims"],
                            sink=0.0, out_scale=cfg["left_scale"])
    right = LinearRecurrence(r["heads"], r["dim"], r["vdim"], workspace, channel=True, tau=r["tau"], out_scale=cfg["right_scale"])
    return SideBySide({"left": left, "right": right})


MIXER_TYPES = {"lightning": lightning, "delta": delta, "latent_attention": latent_attention, "parallel": parallel,
               "channel_delta": channel_delta}
