"""Mixer kernels against the plain oracle, each mechanism alone: in one portion, in portions of several sizes and token by
token, in float32 (tight) and bfloat16."""
import pytest
import torch

from decdec_amd import mixer_ops as M
from oracle import hybrid_oracle as O
import hybrid_cases as cases
from mixer_bench import Bench, close as _close, portions as _portions, rand as _rand

pytestmark = pytest.mark.gpu
DTYPES = [torch.float32, torch.bfloat16]


# ---- rows --------------------------------------------------------------------------------------------------
@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,K,act", [(5, 3, 2), (64, 84, 0), (301, 200, 100), (4100, 96, 4100), (16400, 264, 8), (40, 2056, 1), (7, 1025, 3)])
def test_gemv_with_an_activation_on_its_first_rows(N, K, act, dtype):
    w, x, a = _rand(N, K, seed=N).to(dtype), _rand(K, seed=1).to(dtype), torch.tensor([0.7, -0.4]).to(dtype)
    out = torch.full((N,), 9.0, dtype=dtype, device="cuda")
    M.gemv(w.cuda(), x.cuda(), out, a.cuda() if act else None, act)
    y = w.double() @ x.double()
    y[:act] = O.xielu(y[:act], a[0].double(), a[1].double())
    _close(out, y, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("N,K", [(5, 3), (301, 200), (4100, 96)])
def test_gemv_with_gelu_and_a_scale(N, K, dtype):
    w, x = _rand(N, K, seed=N).to(dtype), _rand(K, seed=1).to(dtype)
    y = w.double() @ x.double()
    out = torch.empty(N, dtype=dtype, device="cuda")
    M.gemv(w.cuda(), x.cuda(), out, None, N, M.ACT_GELU_TANH)
    _close(out, O.gelu_tanh(y), dtype)
    M.gemv(w.cuda(), x.cuda(), out, scale=0.3)
    _close(out, 0.3 * y, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,dim", [(1, 84), (3, 33), (4, 4096), (2, 7001)])
def test_residual_and_embedding_behind_a_dynamic_tanh(rows, dim, dtype):
    x, y = _rand(rows, dim, seed=1, scale=3.0), _rand(rows, dim, seed=2).to(dtype)
    x[0, :7] = torch.tensor([0.0, 1e-6, -1e-4, 1e-2, 40.0, -40.0, 300.0])     # near zero and far past saturation
    a, w, b = torch.tensor(0.7).to(dtype), _rand(dim, seed=5).to(dtype), _rand(dim, seed=6).to(dtype)
    norm = tuple(t.cuda() for t in (a, w, b))
    want = lambda v: O.dynamic_tanh(v, a.double(), w.double(), b.double())
    xd, out = x.cuda(), torch.empty(rows, dim, dtype=dtype, device="cuda")
    M.residual_tanh(xd, None, norm, out)
    assert torch.equal(xd.cpu(), x)
    _close(out, want(x.double()), dtype)
    M.residual_tanh(xd, y.cuda(), norm, out)
    assert torch.equal(xd.cpu(), x + y.float())            # the residual stream is float32 whatever the storage type
    _close(out, want(x.double() + y.double()), dtype)
    no_bias = (norm[0], norm[1], torch.zeros_like(norm[2]))
    small = (_rand(rows, dim, seed=7) * 1e-4).cuda()       # tanh keeps its relative accuracy there
    M.residual_tanh(small, None, no_bias, out)
    _close(out, torch.tanh(a.double() * small.double().cpu()) * w.double(), dtype)
    table, toks = _rand(50, dim, seed=8).to(dtype).cuda(), torch.tensor([3, 49, 0, 3][:rows], device="cuda")
    M.embed(table, toks, xd, out, norm)
    assert torch.equal(xd, table[toks].float())
    _close(out, want(table[toks].double().cpu()), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("n,ld", [(52, 60), (7, 9), (5000, 5000)])
def test_gelu_rows(n, ld, dtype):
    inp = _rand(3, ld, seed=4, scale=3.0).to(dtype).cuda()
    want = O.gelu_tanh(inp[:, :n].double().cpu())
    out = inp if n == ld else torch.empty(3, n, dtype=dtype, device="cuda")   # in place where the rows are whole
    M.activation(inp, n, None, out, M.ACT_GELU_TANH)
    _close(out, want, dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,n", [(3, 36), (3, 128), (2, 256), (2, 201), (2, 1028), (1, 1030)])
@pytest.mark.parametrize("at,wide", [(0, 0), (8, 16), (3, 5)])
def test_group_norm_gate_into_columns_with_a_scale(groups, n, at, wide, dtype):
    o, g, w = _rand(3, groups * n, seed=1).cuda(), _rand(3, groups * n, seed=2).to(dtype).cuda(), _rand(n, seed=3).to(dtype).cuda()
    buf = torch.full((3, groups * n + wide), 7.0, dtype=dtype, device="cuda")
    out = buf[:, at:at + groups * n]
    M.group_norm_gate(o, g, groups * n, w, out, groups, 0.01, M.GATE_SILU, 0.3)
    want = 0.3 * O.rms_norm(o.double().view(3, groups, n), w.double(), 0.01).view(3, -1) * O.silu(g.double())
    _close(out, want, dtype)
    assert float((buf[:, :at] - 7).abs().sum() + (buf[:, at + groups * n:] - 7).abs().sum()) == 0


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rows,dim,gate,final", [(1, 84, True, True), (3, 84, True, False), (2, 33, True, True), (4, 4096, False, True),
                                                 (2, 7000, True, True), (1, 16384, True, False), (2, 20000, True, True)])
def test_gated_residual(rows, dim, gate, final, dtype):
    eps = 1e-3
    x, y = _rand(rows, dim, seed=1, scale=3.0), _rand(rows, dim, seed=2, scale=0.05).to(dtype)
    g, b, w, fw = _rand(rows, dim + 12, seed=3).to(dtype), _rand(dim, seed=4).to(dtype), _rand(dim, seed=5).to(dtype), _rand(dim, seed=6).to(dtype)
    xd, gd = x.cuda(), g.cuda()
    xe, fo = (torch.empty(rows, dim, dtype=dtype, device="cuda") for _ in range(2))
    M.gated_residual(xd, y.cuda(), gd[:, 8:] if gate else None, dim + 12, b.cuda() if gate else None, w.cuda(), xe, eps,
                     fw.cuda() if final else None, fo if final else None)
    y = y.double() * (O.sigmoid(g[:, 8:8 + dim].double() + b.double()) if gate else 1.0)
    want = x.double() + O.rms_norm(y, w.double(), eps)
    _close(xd, want, torch.float32)                     # the residual stream is float32 whatever the storage type
    _close(xe, want, dtype)
    if final:
        _close(fo, O.rms_norm(want, fw.double(), eps), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
def test_embed_norm_and_activation_rows(dtype):
    table = _rand(50, 21, seed=1).to(dtype).cuda()
    toks = torch.tensor([3, 49, 0, 3], device="cuda")
    x, xe = torch.empty(4, 21, device="cuda"), torch.empty(4, 21, dtype=dtype, device="cuda")
    M.embed(table, toks, x, xe)
    assert torch.equal(x, table[toks].float()) and torch.equal(xe, table[toks])
    M.embed(table, torch.tensor([50, -1, 2, 1], device="cuda"), x, None)          # ids outside the table read row 0
    assert torch.equal(x[:2], table[[0, 0]].float())
    for rows, dim in ((3, 21), (2, 5000)):
        v, w = _rand(rows, dim, seed=2).cuda(), _rand(dim, seed=3).to(dtype).cuda()
        out = torch.empty(rows, dim, dtype=dtype, device="cuda")
        M.rmsnorm(v, w, out, 0.1)
        _close(out, O.rms_norm(v.double(), w.double(), 0.1), dtype)
    for n, ld in ((52, 60), (7, 9), (5000, 5008)):
        inp, a = _rand(3, ld, seed=4, scale=2.0).to(dtype).cuda(), torch.tensor([-0.3, 1.2]).to(dtype).cuda()
        out = torch.empty(3, n, dtype=dtype, device="cuda")
        M.activation(inp, n, a, out)
        _close(out, O.xielu(inp[:, :n].double(), a[0].double(), a[1].double()), dtype)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("groups,n,kind", [(1, 140, M.GATE_SIGMOID), (3, 36, M.GATE_SILU), (2, 2048, M.GATE_SILU), (3, 128, M.GATE_SILU),
                                           (2, 256, M.GATE_SIGMOID), (2, 201, M.GATE_SILU), (1, 1030, M.GATE_SIGMOID)])
@pytest.mark.parametrize("off,pad", [(2, 5), (8, 16)])
def test_group_norm_gate(groups, n, kind, off, pad, dtype):
    o, g, w = _rand(3, groups * n, seed=1).cuda(), _rand(3, groups * n + pad, seed=2).to(dtype).cuda(), _rand(n, seed=3).to(dtype).cuda()
    out = torch.empty(3, groups * n, dtype=dtype, device="cuda")
    M.group_norm_gate(o, g[:, off:], groups * n + pad, w, out, groups, 0.01, kind)
    z = g[:, off:off + groups * n].double()
    want = O.rms_norm(o.double().view(3, groups, n), w.double(), 0.01).view(3, -1) * (O.silu(z) if kind == M.GATE_SILU else O.sigmoid(z))
    _close(out, want, dtype)


# ---- mixers ------------------------------------------------------------------------------------------------
RECURRENCES = [("lightning", cases.lightning(3, 32, 32)), ("lightning", cases.lightning(5, 12, 28, [0.0, 0.3, 0.95, 0.9999, 1.0])),
               ("lightning", cases.lightning(2, 128, 128)), ("lightning", cases.lightning(1, 200, 72, [0.98])), ("lightning", cases.lightning(2, 1, 1)),
               ("delta", cases.delta(4, 2, 48, 64, 4)), ("delta", cases.delta(3, 3, 20, 36, 3)), ("delta", cases.delta(4, 2, 128, 128, 4)),
               ("delta", cases.delta(2, 2, 64, 16, 1)), ("delta", cases.delta(6, 2, 9, 130, 2)), ("delta", cases.delta(1, 1, 256, 256, 7)),
               ("delta", cases.delta(2, 1, 16, 300, 5)),
               ("gated_linear", cases.gated_linear(3, 32, 32, 16.0)), ("gated_linear", cases.gated_linear(5, 12, 28, 1.0)),
               ("gated_linear", cases.gated_linear(2, 128, 128, 4.0)), ("gated_linear", cases.gated_linear(1, 200, 72, 0.5)),
               ("gated_linear", cases.gated_linear(2, 1, 1, 2.0)), ("gated_linear", cases.gated_linear(2, 48, 2000, 8.0)),
               ("channel_delta", cases.delta(4, 2, 48, 64, 4)), ("channel_delta", cases.delta(3, 3, 20, 36, 3)),
               ("channel_delta", cases.delta(4, 2, 128, 128, 4)), ("channel_delta", cases.delta(2, 2, 64, 16, 1)),
               ("channel_delta", cases.delta(6, 2, 9, 130, 2)), ("channel_delta", cases.delta(1, 1, 256, 256, 7)),
               ("channel_delta", cases.delta(2, 1, 16, 300, 9)), ("channel_delta", cases.delta(1, 1, 30, 1100, 4))]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind,m", RECURRENCES)
def test_recurrence_in_portions_and_token_by_token(kind, m, dtype):
    T = 150
    b = Bench(kind, m, dtype, T)
    want = b.want()
    for sizes in ((T,), (2,), (3, 64, 1, 2), (65, 63, 5), (1,), (130, 1)):
        # the state of the sequence before is left in place: position 0 starts afresh
        _close(b.run(_portions(T, *sizes)), want, dtype, (kind, m, sizes), factor=4.0)


@pytest.mark.parametrize("dtype", DTYPES)
def test_delta_rule_with_decays_that_forget_at_once_and_never(dtype):
    def edit(b):
        b.w["A_log"] = torch.tensor([5.0, -12.0, 2.0]).to(torch.bfloat16)
        b.w["dt_bias"] = torch.tensor([4.0, -6.0, 1.0]).to(torch.bfloat16)
    b = Bench("delta", cases.delta(3, 1, 24, 24, 4), dtype, 140, edit=edit)
    for sizes in ((140,), (37,), (1,)):
        _close(b.run(_portions(140, *sizes)), b.want(), dtype, sizes, factor=4.0)


@pytest.mark.parametrize("kind", ["delta", "channel_delta"])
def test_convolution_sees_exactly_its_taps_across_a_cut(kind):
    """One token's input is changed: the read-outs of a head without memory differ for `taps` tokens from there on, no
    more and no fewer, wherever the portions are cut."""
    taps, T = 4, 40

    def edit(b):                                           # a decay of e^-150: nothing but the convolution reaches back
        b.w["A_log"], b.w["dt_bias"] = torch.tensor([5.0]).to(torch.bfloat16), torch.full_like(b.w["dt_bias"], 4.0)
        a = "a" if kind == "delta" else "a1"
        b.w[a] = torch.zeros_like(b.w[a])
    b = Bench(kind, cases.delta(1, 1, 16, 16, taps), torch.float32, T, edit=edit)
    for sizes in ((T,), (1,), (2,), (7, 1)):
        base = b.run(_portions(T, *sizes))
        keep = b.proj.clone()
        for at in (0, 6, 7, 13):
            b.proj[at, :48] += 1.0                         # q, k and v of one token
            moved = (b.run(_portions(T, *sizes)) - base).abs().amax(1) > 1e-4
            assert moved.nonzero().view(-1).tolist() == list(range(at, at + taps)), (sizes, at)
            b.proj.copy_(keep)


def _channel_extremes(kind, H, D):
    """Per channel: forgetting at once, never, and everything between, side by side in a head."""
    def edit(b):
        g = torch.Generator().manual_seed(3)
        bias = torch.randn(H * D, generator=g) * 3.0
        bias[::5], bias[1::5] = -30.0, 30.0
        b.w["a2.b" if kind == "gated_linear" else "dt_bias"] = bias.to(torch.bfloat16)
        if kind == "channel_delta":
            b.w["A_log"] = torch.tensor([4.0, -9.0, 1.0][:H]).to(torch.bfloat16)
    return edit


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("kind", ["gated_linear", "channel_delta"])
def test_channel_decays_that_forget_at_once_and_never(kind, dtype):
    m = cases.gated_linear(3, 40, 24, 0.25) if kind == "gated_linear" else cases.delta(3, 1, 40, 24, 4)
    b = Bench(kind, m, dtype, 200, edit=_channel_extremes(kind, 3, 40))
    want = b.want()
    for sizes in ((200,), (37,), (1,)):
        _close(b.run(_portions(200, *sizes)), want, dtype, (kind, sizes), factor=4.0)


@pytest.mark.parametrize("kind", ["gated_linear", "channel_delta"])
def test_tokens_that_forget_everything_between_tokens_that_keep(kind):
    """Decays near one among decays of e^-160 and less: what is written after a token that forgets lasts, whatever the sums hold."""
    T, D, V = 140, 24, 16

    def edit(b):
        z = torch.full((T,), -6.0)
        z[[5, 6, 7, 8, 20, 63, 64, 100]] = 60.0
        b.h[:, 0] = (z if kind == "channel_delta" else -z).to(torch.bfloat16)
        for n in ("q", "k", "v", "b", "g", "g1"):
            if n in b.w:
                b.w[n][:, 0] = 0
        b.w["a1"].zero_(), b.w["a2"].zero_()
        b.w["a1"][0, 0] = 1
        b.w["a2"][:, 0] = 1
        if kind == "channel_delta":
            b.w["A_log"][:] = 1.0
        b.w["dt_bias" if kind == "channel_delta" else "a2.b"].mul_(0.1)
    m = cases.gated_linear(1, D, V, 0.35) if kind == "gated_linear" else cases.delta(1, 1, D, V, 2)
    b = Bench(kind, m, torch.float32, T, edit=edit)
    want = b.want()
    for sizes in ((T,), (1,), (50, 3)):
        _close(b.run(_portions(T, *sizes)), want, torch.float32, sizes, factor=2.0)


@pytest.mark.parametrize("kind", ["gated_linear", "channel_delta"])
def test_every_key_channel_has_its_own_decay(kind):
    """A head whose channels all forget at once but one: what a token wrote comes back through that channel alone, from any
    distance and over any cut."""
    T, D, V, keep = 150, 24, 16, 7
    m = cases.gated_linear(1, D, V, 1.0) if kind == "gated_linear" else cases.delta(1, 1, D, V, 1)

    def edit(b):
        forget = -60.0 if kind == "gated_linear" else 60.0                     # sigmoid(-60), or exp(-e softplus(60))
        bias = torch.full((D,), forget)
        bias[keep] = -forget
        b.w["a2.b" if kind == "gated_linear" else "dt_bias"] = bias.to(torch.bfloat16)
        b.w["a1"] = torch.zeros_like(b.w["a1"])
        if kind == "channel_delta":
            b.w["A_log"] = torch.tensor([1.0]).to(torch.bfloat16)
    b = Bench(kind, m, torch.float32, T, edit=edit)
    want = b.want()
    for sizes in ((T,), (1,), (50, 3), (65,)):
        base = b.run(_portions(T, *sizes))
        _close(base, want, torch.float32, sizes, factor=4.0)
    k = b.mixer.params.off_k
    saved = b.proj.clone()
    b.proj[3, k + keep] += 3.0                                                 # the lasting channel of an early key
    far = (b.run([T]) - base).abs().amax(1)
    assert float(far[100:].max()) > 1e-3 and float(far[:3].max()) < 1e-6
    if kind == "gated_linear":                                                 # (unit vectors couple the channels)
        b.proj.copy_(saved)
        b.proj[3, k + keep + 1] += 3.0
        moved = (b.run([T]) - base).abs().amax(1) > 1e-5
        assert moved.nonzero().view(-1).tolist() == [3]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("rank", [1, 7, 64, 200, 1024])
def test_low_rank_maps_of_any_rank(rank, dtype):
    def edit(b):
        g, H, D, V = torch.Generator().manual_seed(rank), 2, 16, 24
        put = lambda n, *s: b.w.__setitem__(n, (torch.randn(*s, generator=g) * 1.5 / s[1] ** 0.5).to(torch.bfloat16))
        put("a1", rank, 40), put("a2", H * D, rank), put("g1", rank, 40), put("g2", H * V, rank)
    b = Bench("channel_delta", cases.delta(2, 1, 16, 24, 4), dtype, 70, edit=edit)
    want = b.want()
    for sizes in ((70,), (1,)):
        _close(b.run(_portions(70, *sizes)), want, dtype, (rank, sizes), factor=4.0)


LATENTS = [cases.latent(3, 64, 32, 96, 80, scaling=cases.YARN), cases.latent(3, 22, 10, 18, 30, base=500.0), cases.latent(17, 16, 8, 24, 48, scale=0.4),
           cases.latent(2, 128, 64, 128, 512, base=10000.0), cases.latent(1, 200, 56, 200, 96), cases.latent(2, 32, 16, 40, 72, dims=8),
           cases.latent(1, 2, 2, 1, 1), cases.latent(2, 96, 64, 256, 136)]


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("m", LATENTS)
def test_latent_attention_in_portions_and_token_by_token(m, dtype):
    T = 150
    b = Bench("latent_attention", m, dtype, T)
    want = b.want()
    for sizes in ((T,), (2,), (3, 64, 1, 2), (65, 63, 5), (1,), (130, 1)):
        _close(b.run(_portions(T, *sizes)), want, dtype, (m, sizes), factor=2.0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("max_seq", [700, 8000])
def test_latent_attention_finds_one_key_at_every_tile_edge(dtype, max_seq):
    """A query is made to point at one key: its read-out is that token's value, wherever the key lies relative to the tiles
    of 64 keys and to the shares of the one-token kernel's workgroups."""
    T, m = 700, cases.latent(2, 32, 8, 32, 48, base=1e6, scale=1.0)
    b = Bench("latent_attention", m, dtype, T, max_seq=max_seq)
    H, D, R, V, C = 2, 32, 8, 32, 48
    c = O.rms_norm(b.proj[:, 80:80 + C].double().cpu(), b.w["dkv.norm"].double(), b.eps)
    kn = (c @ b.w["uk"].double().T).view(T, H, D)
    v = (c @ b.w["uv"].double().T).view(T, H * V)
    b.run([T - 1])
    tried = 0
    for key in (0, 1, 62, 63, 64, 65, 127, 128, 319, 320, 511, 512, 575, 576, 640, 697, 698):
        q = torch.zeros(H, D + R, dtype=torch.float64)
        for h in range(H):
            others = torch.cat((kn[:key, h], kn[key + 1:, h]))
            q[h, :D] = kn[key, h] * 60.0 / float(kn[key, h] @ kn[key, h] - (others @ kn[key, h]).max()).__abs__()
        b.proj[T - 1, :80] = q.view(-1).to(dtype)
        scores = torch.stack([kn[:, h] @ b.proj[T - 1].double().cpu()[:80].view(H, D + R)[h, :D] for h in range(H)])
        if (scores.argmax(1) != key).any():
            continue                                       # a longer key in the same direction wins
        tried += 1
        one = b.run([1], T - 1)
        for name, got in (("one token", one[0]), ("portion", b.run([3], T - 3)[2])):
            e = torch.exp(scores - scores.amax(1, keepdim=True))
            want = torch.cat([(e[h] / (e[h].sum() + torch.exp(b.w["sink"][h].double() - scores[h].max()))) @ v.view(T, H, V)[:, h] for h in range(H)])
            _close(got, want, dtype, (name, key), factor=3.0)
    assert tried >= 14


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("sink", [-30.0, 0.0, 12.0])
def test_sink_counts_once_whatever_the_number_of_workgroups(sink, dtype):
    def edit(b):
        b.w["sink"] = torch.tensor([sink, sink / 2]).to(torch.bfloat16)
    b = Bench("latent_attention", cases.latent(2, 16, 8, 16, 24), dtype, 520, edit=edit)
    want = b.want()
    _close(b.run([520]), want, dtype, factor=2.0)
    _close(b.run([1] * 5), want[:5], dtype, factor=2.0)                 # the first tokens
    b.run([515])
    _close(b.run([1] * 5, 515), want[515:], dtype, factor=2.0)


def test_no_key_after_the_query_and_every_key_up_to_it():
    """The last visible key is the query's own: changing a later token's input changes nothing, changing its own does."""
    T = 140
    b = Bench("latent_attention", cases.latent(2, 16, 8, 16, 24), torch.float32, T)
    base = b.run([T])
    for at in (0, 1, 63, 64, 127, 128, 139):
        keep = b.proj.clone()
        b.proj[at, 48:48 + 32] += 2.0                                    # latent and rotated key of one token
        for sizes in ((T,), (70,), (1,)):
            diff = (b.run(_portions(T, *sizes)) - base).abs().amax(1)
            assert float(diff[:at].max() if at else 0.0) < 1e-5 and float(diff[at]) > 1e-4, (at, sizes)
        b.proj.copy_(keep)


def test_a_cache_of_a_longer_sequence_before_is_not_seen():
    m = cases.latent(2, 16, 8, 16, 24)
    b = Bench("latent_attention", m, torch.float32, 300)
    b.run([300])
    short = Bench("latent_attention", m, torch.float32, 70, seed=9, max_seq=300)
    short.state = b.state                                                # full of the other sequence's rows
    want = short.want()
    _close(short.run([69]), want[:69], torch.float32)
    _close(short.run([1], 69), want[69:], torch.float32)
