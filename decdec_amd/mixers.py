"""Token mixers of a hybrid decoder: linear recurrences (decayed sum, gated delta rule) and latent attention.

A mixer names the projections of its input that the layer computes in one product (``inputs``), and turns a row block of
them into its read-out, before the output projection.  Everything a design may choose is a constructor argument."""
from __future__ import annotations

import math

import torch
import torch.nn as nn

from . import _lib, mixer_ops as M
from .cache import LatentCache, RecurrentState
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

    def weight_shapes(self, dim: int) -> dict:
        """Name -> shape of all tensors, the input and output projections included."""
        raise NotImplementedError

    def bind(self, weights: dict, offsets: dict, eps: float) -> None:
        """Tensors by name, and the column of every input projection in the stacked product."""
        raise NotImplementedError

    def new_state(self, max_seq: int, dtype, device):
        raise NotImplementedError

    def forward(self, proj, state, pos, start, out):
        """proj [rows, ld] -> out [rows, width]; pos: position of the first row on the device, start: the same on the
        host (None in a one-token step, which may be captured)."""
        raise NotImplementedError


class LinearRecurrence(Mixer):
    """S <- decay S + k v^T (``decay``), or the gated delta rule behind short convolutions (``conv``)."""

    def __init__(self, heads: int, dim: int, vdim: int, workspace: Workspace, kv_heads=None, decay=None, conv: int = 0):
        super().__init__()
        self.heads, self.dim, self.vdim, self.kv_heads = heads, dim, vdim, kv_heads or heads
        self.delta, self.taps, self.workspace = decay is None, conv, workspace
        if self.delta == (conv == 0):
            raise ValueError("a recurrence has either constant decays or a convolution in front of a delta rule")
        if decay is not None and len(decay) != heads:
            raise ValueError(f"{len(decay)} decays for {heads} heads")
        if heads % self.kv_heads:
            raise ValueError(f"{heads} heads do not divide into {self.kv_heads} key heads")
        # a power of every distance inside a chunk, rounded once
        self.powers = None if decay is None else torch.tensor([[float(d) ** n for n in range(65)] for d in decay], dtype=torch.float64).float()
        nqk, nv = self.kv_heads * dim, heads * vdim
        self.inputs = [("q", nqk), ("k", nqk), ("v", nv), ("g", nv)] + ([("b", heads), ("a", heads)] if self.delta else [])
        self.width = nv
        # the read-out is normed over all heads together, or head by head with one shared weight
        self.groups, self.gate = (heads, M.GATE_SILU) if self.delta else (1, M.GATE_SIGMOID)

    def weight_shapes(self, dim):
        s = {n: (r, dim) for n, r in self.inputs}
        s["o"], s["norm"] = (dim, self.width), (self.width // self.groups,)
        if self.delta:
            rows = dict(self.inputs)
            s.update({n + ".conv": (rows[n], self.taps) for n in "qkv"})
            s["A_log"] = s["dt_bias"] = (self.heads,)
        return s

    def bind(self, weights, offsets, eps):
        self.eps, self.norm = eps, weights["norm"]
        self.fused = self.groups == self.heads and M.recurrence_step_fuses(self.dim, self.vdim)
        p = _lib.Recurrence(heads=self.heads, kv_heads=self.kv_heads, dim=self.dim, vdim=self.vdim, taps=max(self.taps, 1),
                            delta=int(self.delta), **{"off_" + n: offsets[n] for n, _ in self.inputs})
        self.keep = [self.norm]
        if self.delta:
            for field, name in (("conv_q", "q.conv"), ("conv_k", "k.conv"), ("conv_v", "v.conv"), ("A_log", "A_log"), ("dt_bias", "dt_bias")):
                setattr(p, field, weights[name].data_ptr())
                self.keep.append(weights[name])
        else:
            self.powers = self.powers.to(self.norm.device)
            p.decay = self.powers.data_ptr()
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
            M.recurrence_rows(p, proj.dtype, o, self.workspace.get(M.recurrence_workspace(p, rows)), rows)
        M.group_norm_gate(o, proj[:, p.off_g:], p.ld, self.norm, out, self.groups, self.eps, self.gate)


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


def lightning(cfg: dict, workspace: Workspace) -> LinearRecurrence:
    return LinearRecurrence(cfg["heads"], cfg["dim"], cfg["vdim"], workspace, decay=cfg["decay"])


def delta(cfg: dict, workspace: Workspace) -> LinearRecurrence:
    return LinearRecurrence(cfg["heads"], cfg["dim"], cfg["vdim"], workspace, kv_heads=cfg["kv_heads"], conv=cfg["conv"])


def latent_attention(cfg: dict, workspace: Workspace) -> LatentAttention:
    rot = cfg["rot"]
    return LatentAttention(cfg["heads"], cfg["dim"], cfg["rot_dim"], cfg["vdim"], cfg["kv_rank"], cfg["scale"], rot["base"], workspace,
                           rope_dims=rot.get("dims"), rope_scaling=rot.get("scaling"))


MIXER_TYPES = {"lightning": lightning, "delta": delta, "latent_attention": latent_attention}
