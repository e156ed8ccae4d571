"""Grouped attention (normed and partly rotated queries and keys, sink, one gate per head) against the plain oracle: whole
prompts, portions, token by token, keys at every tile edge, the first tokens, used caches; and mixers side by side."""
import math

import pytest
import torch

from oracle import hybrid_oracle as O
import hybrid_cases as cases
from mixer_bench import Bench, close as _close, portions as _portions

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]
G = cases.grouped
GROUPED = [G(6, 2, 32, 40, 16), G(4, 4, 22, 18, 10, base=500.0, scale=0.4), G(18, 1, 64, 24, 64), G(34, 2, 16, 32, 4), G(8, 2, 128, 128, 64, base=1e5),
           G(2, 1, 256, 200, 32), G(1, 1, 1, 1, 0), G(3, 1, 33, 7, 2), G(2, 2, 320, 256, 320), G(5, 5, 48, 130, 48, base=50.0),
           {**G(6, 3, 32, 32, 8), "sink": None}, {**G(4, 2, 24, 40, 8), "sink": 2.5, "qk_norm": False}, {**G(4, 1, 40, 24, 40), "gated": False},
           {**G(4, 2, 64, 64, 32), "out_scale": 0.3}]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", GROUPED)
def test_portions_and_token_by_token(m, dtype):
    T = 150
    b = Bench("grouped", m, dtype, T)
    want = b.want()
    for sizes in ((T,), (2,), (3, 64, 1, 2), (65, 63, 5), (1,), (130, 1)):
        _close(b.run(_portions(T, *sizes)), want, dtype, (m, sizes), factor=2.0)


def _plain(b):
    """Norm weights of one and an open gate, so that a read-out row is the attended value."""
    for n in ("q.norm", "k.norm"):
        b.w[n] = torch.ones_like(b.w[n])
    b.w["g"] = torch.zeros_like(b.w["g"])


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("max_seq", [700, 9000])
def test_a_query_finds_one_key_at_every_tile_edge(dtype, max_seq):
    """The last query of every head points at one key: its read-out is that token's value, wherever the key lies relative to
    the tiles of a prompt, to the passes of a decoding wave and to the shares of the workgroups."""
    T, H, KV, D, V, scale = 700, 4, 2, 32, 24, 4.0
    m = G(H, KV, D, V, 8, base=100.0, scale=scale)
    b = Bench("grouped", m, dtype, T, max_seq=max_seq, edit=_plain)
    off = b.mixer.params
    cols = lambda at, n: b.proj[:, at:at + n].double().cpu()
    k = O.rms_norm(cols(off.off_k, KV * D).view(T, KV, D), 1.0, b.eps).transpose(0, 1)
    kr = O.rotate(k, torch.arange(T), m["rot"])
    v = cols(off.off_v, KV * V).view(T, KV, V).transpose(0, 1)
    b.run([T - 1])
    for key in (0, 1, 15, 16, 31, 32, 62, 63, 64, 65, 127, 128, 255, 256, 257, 383, 384, 511, 512, 575, 576, 640, 697, 698, 699):
        q = torch.stack([O.rotate(k[h // 2, key:key + 1], torch.tensor([key - (T - 1)]), m["rot"])[0] for h in range(H)])
        b.proj[T - 1, off.off_q:off.off_q + H * D] = q.reshape(-1).to(dtype)
        qr = O.rotate(O.rms_norm(b.proj[T - 1, off.off_q:off.off_q + H * D].double().cpu().view(H, 1, D), 1.0, b.eps), torch.tensor([T - 1]), m["rot"])
        want = []
        for h in range(H):
            s = (kr[h // 2] @ qr[h, 0]) * scale
            assert int(s.argmax()) == key
            e = torch.exp(s - s.max())
            want.append((e / (e.sum() + torch.exp(-s.max()))) @ v[h // 2] * 0.5)
        want = torch.cat(want)
        assert float((want.view(H, V)[0] - 0.5 * v[0, key]).abs().max()) < 0.2
        one = b.run([1], T - 1)
        for name, got in (("one token", one[0]), ("portion of two", b.run([2], T - 2)[1]), ("portion", b.run([70], T - 70)[69])):
            _close(got, want, dtype, (name, key), factor=3.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sink", [None, 0.0, 40.0])
def test_sink_counts_once_whatever_the_number_of_workgroups(sink, dtype):
    """Scores spread over tens of units, so that a row may be all sink or none of it."""
    b = Bench("grouped", {**G(4, 2, 16, 24, 4, scale=1.5), "sink": sink}, dtype, 520)
    want = b.want()
    _close(b.run([520]), want, dtype, factor=4.0)
    _close(b.run([1] * 5), want[:5], dtype, factor=4.0)                 # the first tokens
    b.run([515])
    _close(b.run([1] * 5, 515), want[515:], dtype, factor=4.0)


def test_first_token_shares_its_weight_with_the_sink():
    """One key, score s: the read-out is v e^s / (1 + e^s)."""
    b = Bench("grouped", G(2, 1, 8, 8, 0, scale=0.5), torch.float32, 4, edit=_plain)
    off = b.mixer.params
    for q in (1.0, -1.0):                                               # the query along its key, and against it
        k = b.proj[0, off.off_k:off.off_k + 8]
        b.proj[0, off.off_q:off.off_q + 16] = torch.cat([k, k]) * q
        s = q * 8 * 0.5                                                 # both have a root mean square of one
        v = b.proj[0, off.off_v:off.off_v + 8].double().cpu()
        want = torch.cat([v, v]) * 0.5 / (1 + math.exp(-s))
        for sizes in ([1], [2], [4]):
            _close(b.run(sizes)[0], want, torch.float32, (q, sizes), factor=5.0)


def test_no_key_after_the_query_and_every_key_up_to_it():
    T = 300
    b = Bench("grouped", G(4, 2, 16, 24, 4), torch.float32, T)
    off, base = b.mixer.params, None
    base = b.run([T])
    for at in (0, 1, 63, 64, 127, 128, 255, 256, 299):
        keep = b.proj.clone()
        b.proj[at, off.off_k:off.off_k + 32] += 2.0
        b.proj[at, off.off_v:off.off_v + 48] += 2.0
        for sizes in ((T,), (70,), (1,)):
            diff = (b.run(_portions(T, *sizes)) - base).abs().amax(1)
            assert float(diff[:at].max() if at else 0.0) < 1e-5 and float(diff[at:].min()) > 1e-4, (at, sizes)
        b.proj.copy_(keep)


def test_a_cache_of_a_longer_sequence_before_is_not_seen():
    m = G(4, 2, 16, 24, 4)
    b = Bench("grouped", m, torch.float32, 600)
    b.run([600])
    short = Bench("grouped", m, torch.float32, 70, seed=9, max_seq=600)
    short.state = b.state                                                # full of the other sequence's rows
    want = short.want()
    _close(short.run([69]), want[:69], torch.float32)
    _close(short.run([1], 69), want[69:], torch.float32)
    _close(short.run([1] * 70), want, torch.float32)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", [cases.parallel(G(6, 2, 32, 40, 16), cases.gated_linear(3, 24, 32, 8.0), 0.6, 1.7),
                               cases.parallel(G(2, 1, 22, 9, 6), cases.gated_linear(2, 10, 11, 1.0), 1.0, 1.0)])
def test_mixers_side_by_side(m, dtype):
    T = 140
    b = Bench("parallel", m, dtype, T)
    want = b.want()
    n = m["left"]["heads"] * m["left"]["vdim"]
    for sizes in ((T,), (2,), (3, 64, 1, 2), (1,)):
        got = b.run(_portions(T, *sizes))
        _close(got[:, :n], want[:, :n], dtype, ("left", sizes), factor=2.0)
        _close(got[:, n:], want[:, n:], dtype, ("right", sizes), factor=4.0)
