"""Each kernel call that the Kelutar parts added or widened, alone, against the plain torch function of
the same name (tests/emulated_ops.py) or a float64 formula written here, in both activation types:
steps of several sequences of unequal length, some at their start in slots that hold another
request's leftovers (NaN here), some continuing; sizes that are no multiples of anything."""
import math
from types import SimpleNamespace

import pytest
import torch

from servelab_amd.kernels import KernelError
from servelab_amd.parts.base import RotaryTables
from test_vekanex_kernels_gpu import DEV, DTYPES, Q_LENS, SLOTS, STARTS, close, fake_batch, states, tables
from test_window_kernels_gpu import fill_pages, paged

pytestmark = pytest.mark.gpu

ONES = ([1, 1, 1, 1, 1], [0, 5, 0, 7, 300], SLOTS)          # one token a sequence


def batches(q_lens, starts, slots):
    out = [fake_batch(q_lens, starts, slots, d) for d in (DEV, "cpu")]
    for b in out:
        b.max_q_len = max(q_lens)
    return out


@pytest.mark.parametrize("dtype", DTYPES)
def test_embedding_with_learned_positions(dtype):
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(0)
    for T, H, V, P in ((1, 72, 11, 9), (33, 256, 300, 77), (5, 1000, 7, 2000)):
        table, pos_table = torch.randn(V, H, generator=g).to(dtype), torch.randn(P, H, generator=g).to(dtype)
        ids = torch.randint(0, V, (T,), generator=g, dtype=torch.int32)
        pos = torch.randint(0, P, (T,), generator=g, dtype=torch.int32)
        pos[-1] = P - 1
        for scale in (1.0, 17.5):
            got = hip.embed(ids.to(DEV), table.to(DEV), scale, pos.to(DEV), pos_table.to(DEV))
            close(got, emu.embed(ids, table, scale, pos, pos_table), 1e-6)
            close(got, table[ids.long()].double() * scale + pos_table[pos.long()].double(), 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 4, 7])
def test_convolution_over_the_stream(dtype, taps):
    """Prompts and portions (a launch of its own behind the normed add) and single tokens (one launch with
    it), with and without an output to add; rows, stream and kept inputs."""
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(taps)
    for H in (72, 256, 1030, 2064, 9000):
        w = 0.5 * torch.randn(taps, H, generator=g)
        gain = 1 + 0.3 * torch.randn(H, generator=g)
        for lens, starts, slots in ((Q_LENS, STARTS, SLOTS), ONES):
            T = sum(lens)
            bd, bh = batches(lens, starts, slots)
            resid, y = 3 * torch.randn(T, H, generator=g), torch.randn(T, H, generator=g).to(dtype)
            st = states(6, max(1, (taps - 1) * H) + 3, seed=4)
            for add in (False, True):
                for write in (True, False):
                    r1, r2, s1, s2 = resid.clone().to(DEV), resid.clone(), st.clone().to(DEV), st.clone()
                    kw1 = dict(y=y.to(DEV), y_weight=gain.to(DEV), y_eps=1e-5) if add else {}
                    kw2 = dict(y=y, y_weight=gain, y_eps=1e-5) if add else {}
                    o1 = hip.stream_conv(r1, w.to(DEV), s1, 0, bd, write, **kw1)
                    o2 = emu.stream_conv(r2, w, s2, 0, bh, write, **kw2)
                    close(r1, r2, 2e-6)
                    close(o1, o2, 3e-6 if dtype == torch.float32 else 8e-3)
                    n = (taps - 1) * H
                    if write and n:
                        close(s1[sorted(slots)][:, :n], s2[sorted(slots)][:, :n], 2e-6)
                    if not write:
                        assert torch.equal(torch.nan_to_num(s1.cpu(), 77.0), torch.nan_to_num(st, 77.0))
                    if not add:
                        assert torch.equal(r1.cpu(), resid)
            # the rows written out for a sequence that starts in the step
            a, b = sum(lens[:2]), sum(lens[:3])
            o = hip.stream_conv(resid.clone().to(DEV), w.to(DEV), st.clone().to(DEV), 0, bd, True)
            x = resid[a:b].double()
            for t in range(b - a):
                want = x[t] + sum(w[j].double() * x[t - taps + 1 + j] for j in range(taps) if t - taps + 1 + j >= 0)
                close(o[a + t], want, 3e-6 if dtype == torch.float32 else 8e-3)


def test_single_tokens_and_portions_give_the_same_bits():
    """A sequence's tokens one by one through the one-launch form and in one portion: rows, stream, slot."""
    hip, _ = tables(torch.bfloat16)
    g = torch.Generator().manual_seed(3)
    T, H, taps = 9, 520, 4
    resid, y = torch.randn(T, H, generator=g).to(DEV), torch.randn(T, H, generator=g).bfloat16().to(DEV)
    w, gain = torch.randn(taps, H, generator=g).to(DEV), torch.rand(H, generator=g).to(DEV)
    ra, sa = resid.clone(), torch.full((2, (taps - 1) * H), float("nan"), device=DEV)
    rows = hip.stream_conv(ra, w, sa, 0, batches([T], [0], [1])[0], True, y=y, y_weight=gain, y_eps=1e-5)
    sb, outs, rb = torch.full_like(sa, float("nan")), [], []
    for t in range(T):
        r = resid[t:t + 1].clone()
        outs.append(hip.stream_conv(r, w, sb, 0, batches([1], [t], [1])[0], True, y=y[t:t + 1].contiguous(), y_weight=gain,
                                    y_eps=1e-5))
        rb.append(r)
    close(torch.cat(rb), ra, 1e-6)
    close(torch.cat(outs), rows, 8e-3)
    close(sb[1], sa[1], 1e-6)


def test_postnorm_that_wants_no_rows():
    hip, emu = tables(torch.bfloat16)
    g = torch.Generator().manual_seed(1)
    resid, y, w = torch.randn(5, 300, generator=g), torch.randn(5, 300, generator=g).bfloat16(), torch.rand(300, generator=g)
    r1, r2 = resid.clone().to(DEV), resid.clone()
    assert hip.add_postnorm(r1, y.to(DEV), w.to(DEV), 1e-5, 0.7, want_rows=False) is None
    emu.add_postnorm(r2, y, w, 1e-5, 0.7)
    close(r1, r2, 1e-6)


@pytest.mark.parametrize("H,D,Dv", [(1, 1, 1), (3, 10, 14), (2, 48, 24), (4, 64, 96), (2, 128, 40), (1, 200, 33), (1, 512, 9)])
def test_forget_scan(H, D, Dv):
    hip, emu = tables(torch.float32)
    g = torch.Generator().manual_seed(D)
    width = 2 * H * D + H * Dv + 5
    for lens, starts, slots in ((Q_LENS, STARTS, SLOTS), ONES, ([200, 3], [0, 17], [3, 5])):
        T = sum(lens)
        buf = torch.randn(T, width, generator=g)
        f_col, v_col = 3 + H * D, 3 + 2 * H * D
        buf[:, f_col:f_col + H * D] = 3 * buf[:, f_col:f_col + H * D] + 2
        buf[::3, f_col] = 25.0                                # gates that stand open, and one that is shut
        buf[1::5, f_col] = -25.0
        lower = torch.rand(H * D, generator=g)
        lower[0] = 0.0
        bd, bh = batches(lens, starts, slots)
        st = torch.randn(6, H * D * Dv + 2, generator=g) * 0.3
        for s, a in zip(slots, starts):
            if a == 0:
                st[s] = float("nan")
        for write in (True, False):
            s1, s2 = st.clone().to(DEV), st.clone()
            o1 = hip.forget_scan(buf.to(DEV), 3, f_col, v_col, H, D, Dv, lower.to(DEV), s1, bd, write, q_scale=0.7)
            o2 = emu.forget_scan(buf, 3, f_col, v_col, H, D, Dv, lower, s2, bh, write, q_scale=0.7)
            close(o1, o2, 1e-5)
            if write:
                close(s1[sorted(slots)][:, :H * D * Dv], s2[sorted(slots)][:, :H * D * Dv], 1e-5)
            else:
                assert torch.equal(torch.nan_to_num(s1.cpu(), 77.0), torch.nan_to_num(st, 77.0))
    with pytest.raises(KernelError):
        hip.forget_scan(buf.to(DEV), 3, f_col, width, H, D, Dv, lower.to(DEV), st.to(DEV), bd, True)


@pytest.mark.parametrize("dtype", DTYPES)
def test_head_norm_without_a_gate(dtype):
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(6)
    for T, H, Dv in ((1, 3, 14), (40, 2, 128), (7, 1, 300)):
        o = torch.randn(T, H * Dv, generator=g)
        for per_head in (False, True):
            w = 1 + 0.3 * torch.randn(H * Dv if per_head else Dv, generator=g)
            got = hip.head_norm_gate(o.to(DEV), H, Dv, w.to(DEV), per_head, 1e-5)
            x = o.view(T, H, Dv).double()
            want = x / (x.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * (w.view(H, Dv) if per_head else w).double()
            close(got, want.reshape(T, -1), 3e-6 if dtype == torch.float32 else 8e-3)
            close(got, emu.head_norm_gate(o, H, Dv, w, per_head, 1e-5), 3e-6 if dtype == torch.float32 else 8e-3)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T", [3, 21, 600])
def test_norm_per_head_in_the_launch_that_turns_and_stores(dtype, T):
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(T)
    for H, G, D, rot, keys in ((4, 2, 16, 0, True), (6, 3, 10, 4, False), (1, 1, 150, 150, False), (8, 2, 64, 0, True),
                               (2, 1, 300, 0, True)):
        Dv = D if keys else 12
        buf = 2 * torch.randn(T, (H + G) * D + (0 if keys else G * Dv) + 3, generator=g)
        qg, kg = torch.randn(H * D, generator=g), torch.randn(G * D, generator=g)
        ang = torch.rand(T, max(1, rot // 2), generator=g) * 6
        tb = RotaryTables(torch.cos(ang), torch.sin(ang)) if rot else None
        tbd = RotaryTables(tb.cos.to(DEV), tb.sin.to(DEV)) if rot else None
        page = 16
        pages = -(-T // page) + 2
        slots = torch.randperm(pages * page, generator=g)[:T].to(torch.int32)
        kc2, vc2 = torch.zeros(pages, G, page, D).to(dtype), torch.zeros(pages, G, Dv, page).to(dtype)
        kd, vd = kc2.clone().to(DEV), vc2.clone().to(DEV)
        q1 = hip.projnorm_rope_store(buf.to(DEV), H, G, D, Dv, qg.to(DEV), kg.to(DEV), 1e-5, rot, tbd, slots.to(DEV), kd, vd,
                                     page, values_are_keys=keys, per_head=True)
        q2 = emu.projnorm_rope_store(buf, H, G, D, Dv, qg, kg, 1e-5, rot, tb, slots, kc2, vc2, page, values_are_keys=keys,
                                     per_head=True)
        tol = 3e-6 if dtype == torch.float32 else 8e-3
        close(q1, q2, tol)
        close(kd, kc2, tol)
        close(vd, vc2, tol)
        if not rot:
            x = buf[:, :H * D].view(T, H, D).double()
            want = x / (x.pow(2).mean(-1, keepdim=True) + 1e-5).sqrt() * qg.view(H, D).double()
            close(q1, want.reshape(T, -1), tol)


def test_norm_per_head_behind_a_convolution():
    hip, emu = tables(torch.float32)
    g = torch.Generator().manual_seed(9)
    H, G, D, taps, T = 3, 1, 20, 3, sum(Q_LENS)
    C = (H + 2 * G) * D
    bd, bh = batches(Q_LENS, STARTS, SLOTS)
    buf, w = torch.randn(T, C, generator=g), torch.randn(C, taps, generator=g)
    qg, kg = torch.randn(H * D, generator=g), torch.randn(G * D, generator=g)
    slots = torch.arange(T, dtype=torch.int32)
    st = states(6, (taps - 1) * C, seed=8)
    k1, v1 = torch.zeros(5, G, 16, D), torch.zeros(5, G, D, 16)
    kd, vd, s1 = k1.clone().to(DEV), v1.clone().to(DEV), st.clone().to(DEV)
    q1 = hip.projnorm_rope_store(buf.to(DEV), H, G, D, D, qg.to(DEV), kg.to(DEV), 1e-5, 0, None, slots.to(DEV), kd, vd, 16,
                                 conv=(w.to(DEV), s1, 0, bd, True), per_head=True)
    q2 = emu.projnorm_rope_store(buf, H, G, D, D, qg, kg, 1e-5, 0, None, slots, k1, v1, 16, conv=(w, st, 0, bh, True),
                                 per_head=True)
    close(q1, q2, 5e-6)
    close(kd, k1, 5e-6)
    close(vd, v1, 5e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,Dk,Dv", [(4, 2, 24, 16), (6, 1, 64, 64), (3, 3, 10, 10), (2, 1, 32, 48)])
def test_gate_on_every_channel(dtype, H, G, Dk, Dv):
    """Prompts, a portion deep in its sequence, portions of two tokens, single tokens (few keys, and enough
    for shares of the keys)."""
    hip, _ = tables(dtype)
    g = torch.Generator().manual_seed(H + Dk)
    page = 16
    seqs = [(0, 70), (45, 19), (0, 2), (61, 2), (0, 1), (16, 1), (700, 1), (31, 1)]
    lens = [a + b for a, b in seqs]
    for window in (None, 9):
        tbl, kc, vc = paged(lens, page, G, Dk, Dv, dtype, g)
        keys = [torch.randn(n, G, Dk, generator=g).to(dtype) for n in lens]
        values = [torch.randn(n, G, Dv, generator=g).to(dtype) for n in lens]
        fill_pages(tbl, kc, vc, keys, values, page)
        for part in (slice(0, 4), slice(4, 8)):
            sub = seqs[part]
            T = sum(b for _, b in sub)
            q = torch.randn(T, H * Dk, generator=g).to(dtype)
            gate = 2 * torch.randn(T, H * Dv + 7, generator=g)
            cu, pos, want = [0], [], []
            for s, (a, b) in enumerate(sub):
                k, v = keys[part.start + s], values[part.start + s]
                qs = q[cu[-1]:cu[-1] + b].view(b, H, Dk).double()
                kh, vh = k.repeat_interleave(H // G, 1).double(), v.repeat_interleave(H // G, 1).double()
                sc = torch.einsum("ihd,jhd->hij", qs, kh) * 0.4
                i, j = torch.arange(a, a + b)[:, None], torch.arange(a + b)[None, :]
                vis = (j <= i) & (i - j < (window or 10 ** 6))
                want.append(torch.einsum("hij,jhd->ihd", torch.softmax(sc.masked_fill(~vis[None], -math.inf), -1), vh))
                pos += list(range(a, a + b))
                cu.append(cu[-1] + b)
            b2 = SimpleNamespace(cu_q=torch.tensor(cu, dtype=torch.int32, device=DEV),
                                 positions=torch.tensor(pos, dtype=torch.int32, device=DEV), num_seqs=len(sub), num_tokens=T,
                                 max_q_len=max(b for _, b in sub), max_ctx_len=max(a + b for a, b in sub))
            args = (q.to(DEV), 0, H, G, Dk, Dv, kc.to(DEV), vc.to(DEV), page, tbl[part].contiguous().to(DEV), b2, 0.4, window)
            got = hip.window_attention(*args, channel_gate=gate.to(DEV), channel_gate_col=3)
            want = torch.cat(want).reshape(T, H * Dv)
            gated = want * torch.sigmoid(gate[:, 3:3 + H * Dv].double())
            close(got, gated, 2e-5 if dtype == torch.float32 else 2e-2)
            close(hip.window_attention(*args), want, 2e-5 if dtype == torch.float32 else 2e-2)
            with pytest.raises(KernelError, match="channel gates"):
                hip.window_attention(*args, channel_gate=gate.to(DEV), channel_gate_col=8)


@pytest.mark.parametrize("rows", [1, 2, 5, 8, 16, 17, 24, 64, 100, 200, 600])
def test_squared_relu_feed_forward_at_every_row_count(rows):
    """bfloat16: the row count decides which product kernel runs and where the activation is applied."""
    g = torch.Generator().manual_seed(2)
    for width, inter, activation in ((256, 1536, "relu2"), (72, 40, "relu2"), (96, 64, "silu"), (2048, 4096, "relu2")):
        up = torch.randn(inter, width, generator=g) * width ** -0.5
        down = torch.randn(width, inter, generator=g) * inter ** -0.5
        x = torch.randn(rows, width, generator=g)
        for dtype in DTYPES:
            hip, emu = tables(dtype)
            w_u, w_d = hip.prepare_weight(up.to(dtype).to(DEV)), hip.prepare_weight(down.to(dtype).to(DEV))
            h = hip.activated_linear(x.to(dtype).to(DEV), w_u, activation)
            close(h, emu.activated_linear(x.to(dtype), up.to(dtype), activation), 2e-5 if dtype == torch.float32 else 1.5e-2)
            want = emu.plain_mlp(x.to(dtype), up.to(dtype), down.to(dtype), activation)
            for defer in (False, True):
                got = hip.materialize(hip.plain_mlp(x.to(dtype).to(DEV), w_u, w_d, activation, defer=defer))
                close(got, want, 2e-5 if dtype == torch.float32 else 2e-2)
            z = x.to(dtype).double() @ up.to(dtype).double().T
            mid = torch.relu(z) ** 2 if activation == "relu2" else z * torch.sigmoid(z)
            close(got, mid @ down.to(dtype).double().T, 2e-5 if dtype == torch.float32 else 2.5e-2)
