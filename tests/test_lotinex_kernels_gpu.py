"""Each kernel call that the Lotinex parts added or widened, alone, against the plain torch function of
the same name (tests/emulated_ops.py) or a float64 formula written here, in both activation types:
steps of several sequences of unequal length, some at their start in slots that hold another
request's leftovers (NaN here), some continuing; sizes that are no multiples of anything."""
import math
from types import SimpleNamespace

import pytest
import torch

from servelab_amd.kernels import KernelError
from servelab_amd.parts.base import RotaryTables
from test_kelutar_kernels_gpu import ONES, batches
from test_vekanex_kernels_gpu import DEV, DTYPES, Q_LENS, SLOTS, STARTS, close, states, tables
from test_window_kernels_gpu import fill_pages, paged

pytestmark = pytest.mark.gpu
STEPS = ((Q_LENS, STARTS, SLOTS), ONES, ([200, 3], [0, 17], [3, 5]))


def dev(t):
    return None if t is None else t.to(DEV)


def fresh_is_nan(st, starts, slots):
    for s, a in zip(slots, starts):
        if a == 0:
            st[s] = float("nan")
    return st


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("S", [1, 2, 3, 4, 5, 8, 11, 16])
def test_streams_written_read_and_normed_in_one_call(dtype, S):
    """Nothing pending, one output, two with norms of their own; layer norm with and without a bias, RMS norm;
    every row in place, and listed rows that leave the copies alone."""
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(S)
    for T, H in ((1, 72), (9, 256), (3, 2056), (2, 1030), (2, 9000), (5, 37)):
        x = 2 * torch.randn(T, S, H, generator=g)
        ys = [torch.randn(T, H, generator=g).to(dtype) for _ in range(2)]
        gains = [1 + 0.3 * torch.randn(H, generator=g) for _ in range(2)]
        mix, out, read = torch.randn(S, S, generator=g) / S, torch.randn(S, generator=g), torch.randn(S, generator=g)
        w, b = 1 + 0.3 * torch.randn(H, generator=g), torch.randn(H, generator=g)
        rows = torch.tensor([T - 1, 0], dtype=torch.int32)
        for outputs in ([], [(ys[0], None, 0.0)], [(ys[0], gains[0], 1e-5), (ys[1], gains[1], 1e-4)],
                        [(ys[0], None, 0.0), (ys[1], gains[1], 1e-4)]):
            on = [(dev(y), dev(gn), e) for y, gn, e in outputs]
            for bias, center, rd in ((b, True, read), (None, False, read), (b, True, None)):
                for pick in (None, rows):
                    x1, x2 = x.clone().to(DEV), x.clone()
                    o1 = hip.streams_norm(x1, on, dev(mix), dev(out), dev(rd), dev(w), dev(bias), 1e-5, center=center,
                                          rows=dev(pick))
                    o2 = emu.streams_norm(x2, outputs, mix, out, rd, w, bias, 1e-5, center=center, rows=pick)
                    close(o1, o2, 1e-5 if dtype == torch.float32 else 1e-2)
                    close(x1, x2, 3e-6)
                    if pick is not None or not outputs:
                        assert torch.equal(x1.cpu(), x)
    x = torch.randn(2, S, 40, generator=g).double()           # the write, by its definition
    y = torch.randn(2, 40, generator=g).to(dtype)
    mix, out = torch.randn(S, S, generator=g), torch.randn(S, generator=g)
    x1 = x.float().to(DEV)
    hip.streams_norm(x1, [(dev(y), None, 0.0)], dev(mix), dev(out), dev(out), dev(torch.ones(40)), None, 1e-5)
    for t in range(S):
        want = sum(mix[s, t].double() * x[:, s] for s in range(S)) + out[t].double() * y.double()
        close(x1[:, t], want, 1e-5)
    with pytest.raises(KernelError):
        hip.streams_norm(x1, [(dev(y), None, 0.0)], dev(mix[:, :1].contiguous()) if S > 1 else dev(torch.ones(2, 2)), dev(out), None,
                         dev(torch.ones(40)), None, 1e-5)


@pytest.mark.parametrize("dtype", DTYPES)
def test_layer_norm_with_a_bias_and_an_embedding_in_copies(dtype):
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(2)
    for T, H in ((1, 72), (7, 1030), (4, 2048), (3, 17000)):
        x, d = torch.randn(T, H, generator=g) + 0.5, torch.randn(T, H, generator=g).to(dtype)
        w, b = torch.randn(H, generator=g), torch.randn(H, generator=g)
        x1, x2 = x.clone().to(DEV), x.clone()
        close(hip.add_layernorm(x1, dev(d), dev(w), 1e-5, bias=dev(b)), emu.add_layernorm(x2, d, w, 1e-5, bias=b),
              1e-5 if dtype == torch.float32 else 1e-2)
        v = (x + d.float()).double()
        want = (v - v.mean(-1, keepdim=True)) / (v.var(-1, unbiased=False, keepdim=True) + 1e-5).sqrt() * w + b
        close(hip.add_layernorm(x.clone().to(DEV), dev(d), dev(w), 1e-5, bias=dev(b),
                                rows=torch.tensor([T - 1], dtype=torch.int32, device=DEV)), want[T - 1:],
              1e-5 if dtype == torch.float32 else 1e-2)
    table = torch.randn(11, 72, generator=g).to(dtype)
    ids = torch.tensor([3, 10, 0], dtype=torch.int32)
    got = hip.embed(dev(ids), dev(table), 2.5, copies=3)
    assert got.shape == (3, 3, 72)
    for s in range(3):
        close(got[:, s], table[ids.long()].double() * 2.5, 1e-6)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("H,G,Dk,Dv", [(4, 2, 24, 16), (6, 1, 64, 32), (3, 3, 10, 12), (8, 2, 64, 80), (2, 1, 32, 48)])
def test_attention_in_chunks_with_a_sink(dtype, H, G, Dk, Dv):
    """Prompts, portions and single tokens; chunks that end inside the step, at page borders and at its first
    token, of one token and longer than everything; with a sink of score 0 and a cap; beside a window."""
    hip, _ = tables(dtype)
    g = torch.Generator().manual_seed(H + Dv)
    page = 16
    seqs = [(0, 70), (45, 19), (0, 2), (61, 2), (0, 1), (16, 1), (700, 1), (31, 1), (639, 1), (640, 1)]
    lens = [a + b for a, b in seqs]
    tbl, kc, vc = paged(lens, page, G, Dk, Dv, dtype, g)
    keys = [torch.randn(n, G, Dk, generator=g).to(dtype) for n in lens]
    values = [torch.randn(n, G, Dv, generator=g).to(dtype) for n in lens]
    fill_pages(tbl, kc, vc, keys, values, page)
    for chunk, window, cap, sink in ((9, None, None, None), (64, None, None, 0.0), (1, None, None, None), (320, None, 5.0, 0.0),
                                     (10 ** 6, None, None, None), (32, 20, None, 0.0), (None, 13, 2.0, 0.0), (None, None, None, 0.0)):
        for part in (slice(0, 4), slice(4, 10), slice(2, 6)):
            sub = seqs[part]
            T = sum(b for _, b in sub)
            q = torch.randn(T, H * Dk, generator=g).to(dtype)
            cu, pos, want = [0], [], []
            for s, (a, b) in enumerate(sub):
                qs = q[cu[-1]:cu[-1] + b].view(b, H, Dk).double()
                kh = keys[part.start + s].repeat_interleave(H // G, 1).double()
                vh = values[part.start + s].repeat_interleave(H // G, 1).double()
                sc = torch.einsum("ihd,jhd->hij", qs, kh) * 0.3
                if cap:
                    sc = cap * torch.tanh(sc / cap)
                i, j = torch.arange(a, a + b)[:, None], torch.arange(a + b)[None, :]
                vis = (j <= i) & (i - j < (window or 10 ** 6))
                if chunk:
                    vis &= i // chunk == j // chunk
                e = torch.exp(sc.masked_fill(~vis[None], -math.inf))
                p = e / (e.sum(-1, keepdim=True) + (1.0 if sink is not None else 0.0))
                want.append(torch.einsum("hij,jhd->ihd", p, vh))
                pos += list(range(a, a + b))
                cu.append(cu[-1] + b)
            b2 = SimpleNamespace(cu_q=torch.tensor(cu, dtype=torch.int32, device=DEV),
                                 positions=torch.tensor(pos, dtype=torch.int32, device=DEV), num_seqs=len(sub), num_tokens=T,
                                 max_q_len=max(b for _, b in sub), max_ctx_len=max(a + b for a, b in sub))
            got = hip.window_attention(dev(q), 0, H, G, Dk, Dv, dev(kc), dev(vc), page, dev(tbl[part].contiguous()), b2, 0.3,
                                       window, chunk=chunk, softcap=cap,
                                       sinks=None if sink is None else torch.zeros(H, device=DEV))
            close(got, torch.cat(want).reshape(T, H * Dv), 2e-5 if dtype == torch.float32 else 2e-2)


def test_released_pages_of_a_chunk_are_never_read():
    """Pages before the query's chunk hold NaN: what a later owner may have left there."""
    hip, _ = tables(torch.bfloat16)
    g = torch.Generator().manual_seed(3)
    H, G, Dk, Dv, page, chunk = 4, 2, 64, 32, 16, 40
    n = 130
    tbl, kc, vc = paged([n], page, G, Dk, Dv, torch.bfloat16, g)
    first = (n - 1) // chunk * chunk
    k, v = torch.randn(n, G, Dk, generator=g).bfloat16(), torch.randn(n, G, Dv, generator=g).bfloat16()
    k[:first], v[:first] = float("nan"), float("nan")
    fill_pages(tbl, kc, vc, [k], [v], page)
    tbl[0, :first // page] = 0
    q = torch.randn(1, H * Dk, generator=g).bfloat16()
    b = SimpleNamespace(cu_q=torch.tensor([0, 1], dtype=torch.int32, device=DEV),
                        positions=torch.tensor([n - 1], dtype=torch.int32, device=DEV), num_seqs=1, num_tokens=1, max_q_len=1,
                        max_ctx_len=n)
    for table in (hip, tables(torch.float32)[0]):
        cast = (lambda t: t.to(DEV)) if table is hip else (lambda t: t.float().to(DEV))
        got = table.window_attention(cast(q), 0, H, G, Dk, Dv, cast(kc), cast(vc), page, tbl.to(DEV), b, 0.2, None, chunk=chunk)
        s = torch.einsum("hd,jhd->hj", q.view(H, Dk).double(), k[first:].repeat_interleave(2, 1).double()) * 0.2
        want = torch.einsum("hj,jhd->hd", torch.softmax(s, -1), v[first:].repeat_interleave(2, 1).double())
        close(got, want.reshape(1, -1), 2e-2)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("per_head", [True, False])
def test_queries_alone_are_normed_and_turned(dtype, per_head):
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(4)
    for T, H, D, rot in ((3, 4, 16, 8), (33, 3, 10, 10), (600, 2, 96, 48), (2, 1, 30, 0)):
        buf, gain = torch.randn(T, H * D + 3, generator=g), torch.randn(H * D, generator=g)
        ang = torch.rand(T, max(1, rot // 2), generator=g) * 6
        tb = RotaryTables(torch.cos(ang), torch.sin(ang)) if rot else None
        tbd = RotaryTables(dev(tb.cos), dev(tb.sin)) if rot else None
        got = hip.projnorm_rope_store(dev(buf), H, 0, D, 12, dev(gain), None, 1e-5, rot, tbd, None, None, None, 16,
                                      per_head=per_head)
        want = emu.projnorm_rope_store(buf, H, 0, D, 12, gain, None, 1e-5, rot, tb, None, None, None, 16, per_head=per_head)
        close(got, want, 3e-6 if dtype == torch.float32 else 8e-3)
    with pytest.raises(KernelError):
        hip.projnorm_rope_store(dev(buf), H, 0, D, 12, dev(gain), None, 1e-5, 0, None,
                                torch.zeros(2, dtype=torch.int32, device=DEV), None, None, 16)


@pytest.mark.parametrize("H,G,D,Dv", [(1, 1, 1, 1), (4, 2, 12, 18), (6, 3, 9, 20), (4, 4, 64, 32), (2, 1, 128, 40), (1, 1, 200, 33)])
def test_delta_scan_with_one_decay_a_head(H, G, D, Dv):
    hip, emu = tables(torch.float32)
    g = torch.Generator().manual_seed(D)
    C = 2 * G * D + H * Dv
    for lens, starts, slots in STEPS:
        T = sum(lens)
        src, gates = torch.randn(T, C + 3, generator=g), 2 * torch.randn(T, 2 * H + 5, generator=g)
        qk = src[:, 2:2 + 2 * G * D].view(T, 2 * G, D)
        qk /= qk.norm(dim=-1, keepdim=True)
        gates[1::7, 2 + H:2 + 2 * H] = 30.0                     # a state that is wiped, and one that is kept
        gates[2::7, 2 + H:2 + 2 * H] = -30.0
        rates, bias = torch.randn(H, generator=g), torch.randn(H, generator=g) - 1
        bd, bh = batches(lens, starts, slots)
        st = fresh_is_nan(torch.randn(6, H * D * Dv + 2, generator=g) * 0.3, starts, slots)
        for write in (True, False):
            s1, s2 = st.clone().to(DEV), st.clone()
            args = (2, 2 + G * D, 2 + 2 * G * D, H, G, D, Dv)
            o1 = hip.head_delta_scan(dev(src), *args, dev(gates), 2, 2 + H, dev(rates), dev(bias), s1, bd, write)
            o2 = emu.head_delta_scan(src, *args, gates, 2, 2 + H, rates, bias, s2, bh, write)
            close(o1, o2, 2e-5)
            if write:
                close(s1[sorted(slots)][:, :H * D * Dv], s2[sorted(slots)][:, :H * D * Dv], 2e-5)
            else:
                assert torch.equal(torch.nan_to_num(s1.cpu(), 77.0), torch.nan_to_num(st, 77.0))
    with pytest.raises(KernelError):
        hip.head_delta_scan(dev(src), *args, dev(gates), 2, 2 * H + 5, dev(rates), dev(bias), st.to(DEV), bd, True)


@pytest.mark.parametrize("C,N,R", [(56, 6, 5), (24, 16, 1), (80, 24, 7), (512, 40, 40), (10, 70, 3), (300, 16, 33), (64, 8, 4),
                                   (130, 32, 9), (65, 64, 2), (5, 1, 1), (3, 300, 2), (70, 33, 130)])
@pytest.mark.parametrize("dtype", DTYPES)
def test_selective_scan(dtype, C, N, R):
    """One token a sequence (one launch), steps within a segment, and prompts of several segments."""
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(C + N)
    steps = STEPS + (([64, 65, 1, 128, 2], [0, 3, 0, 0, 9], SLOTS), ([64, 2], [5, 0], [1, 2]), ([1], [0], [2]))
    for lens, starts, slots in steps:
        T = sum(lens)
        u, proj = torch.randn(T, C, generator=g), torch.randn(T, R + 2 * N + 3, generator=g)
        gate = torch.randn(T, C + 6, generator=g)
        step, bias, skip = torch.randn(C, R, generator=g), 2 * torch.randn(C, generator=g) - 1, torch.randn(C, generator=g)
        rates = -torch.exp(torch.randn(N, C, generator=g))
        bd, bh = batches(lens, starts, slots)
        st = fresh_is_nan(torch.randn(6, N * C + 2, generator=g), starts, slots)
        for write in (True, False):
            s1, s2 = st.clone().to(DEV), st.clone()
            o1 = hip.selective_scan(dev(u), dev(proj), R, N, dev(step), dev(step.t().contiguous()), dev(bias), dev(rates), dev(skip),
                                    dev(gate), 4, s1, bd, write)
            o2 = emu.selective_scan(u, proj, R, N, step, step.t(), bias, rates, skip, gate, 4, s2, bh, write)
            close(o1, o2, 3e-5 if dtype == torch.float32 else 1e-2)
            if write:
                close(s1[sorted(slots)][:, :N * C], s2[sorted(slots)][:, :N * C], 3e-5)
                assert torch.equal(s1[:, N * C:].isnan().cpu(), st[:, N * C:].isnan())
            else:
                assert torch.equal(torch.nan_to_num(s1.cpu(), 77.0), torch.nan_to_num(st, 77.0))
    with pytest.raises(KernelError):
        hip.selective_scan(dev(u), dev(proj[:, :R + 2 * N - 1].contiguous()), R, N, dev(step), dev(step.t().contiguous()), dev(bias),
                           dev(rates), dev(skip), dev(gate), 4, st.to(DEV), bd, True)


def test_step_sizes_of_many_tokens_and_wide_ranks():
    """The tiled form of the low-rank expansion (many tokens, ranks of 24 and more) and its softplus."""
    hip, emu = tables(torch.float32)
    g = torch.Generator().manual_seed(5)
    for T, C, rank, heads in ((1, 40, 24, 1), (63, 64, 40, 4), (64, 64, 24, 2), (130, 200, 37, 5), (257, 130, 130, 1), (64, 3, 160, 3)):
        buf, w2 = torch.randn(T, rank + 9, generator=g), torch.randn(C, rank, generator=g) * rank ** -0.5
        b, rates = torch.randn(C, generator=g), torch.randn(heads, generator=g)
        for mode in ("softplus", "plain", "log_sigmoid", "rate_softplus") if C % heads == 0 else ("softplus", "plain"):
            for bias in (b, None):
                kw = dict(heads=heads, divisor=3.0, rates=rates) if mode == "rate_softplus" else dict(divisor=3.0)
                kd = {k: dev(v) if torch.is_tensor(v) else v for k, v in kw.items()}
                close(hip.lowrank_expand(dev(buf), 4, dev(w2), dev(bias), mode, **kd), emu.lowrank_expand(buf, 4, w2, bias, mode, **kw),
                      5e-6)
    z = torch.tensor([[-90.0], [-20.0], [0.0], [20.0], [90.0]])
    got = hip.lowrank_expand(dev(z), 0, torch.ones(1, 1, device=DEV), None, "softplus").cpu().double()
    want = torch.nn.functional.softplus(z.double())
    assert ((got - want).abs() <= 1e-6 * want + 1e-30).all()


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("taps", [1, 2, 3, 4, 6])
def test_short_convolution_of_single_tokens_moves_its_slot_on(dtype, taps):
    """Rows in both types; the state's last inputs after single tokens (one launch) and after portions (two)."""
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(taps)
    for C, heads, d in ((70, 0, 0), (300, 3, 20)):
        w, b = torch.randn(C, taps, generator=g), torch.randn(C, generator=g)
        for lens, starts, slots in STEPS[:2]:
            T = sum(lens)
            buf = torch.randn(T, C + 5, generator=g)
            bd, bh = batches(lens, starts, slots)
            st = states(6, (taps - 1) * C + 4, seed=8)
            for write in (True, False):
                s1, s2 = st.clone().to(DEV), st.clone()
                kw = dict(unit_heads=heads, unit_dim=d, scaled_heads=min(1, heads), scale=0.3)
                o1, r1 = hip.short_conv(dev(buf), 2, dev(w), s1, 3, bd, write, bias=dev(b), want_rows=True, **kw)
                o2, r2 = emu.short_conv(buf, 2, w, s2, 3, bh, write, bias=b, want_rows=True, **kw)
                close(o1, o2, 3e-6)
                close(r1, r2, 3e-6 if dtype == torch.float32 else 8e-3)
                assert torch.equal(r1.float(), o1.to(dtype).float())
                n = (taps - 1) * C
                if write and n:
                    close(s1[sorted(slots)][:, 3:3 + n], s2[sorted(slots)][:, 3:3 + n], 0)
                elif n:
                    assert torch.equal(torch.nan_to_num(s1.cpu(), 77.0), torch.nan_to_num(st, 77.0))
            # the same convolution in the launch that norms, turns and stores
            H, G, D = 3, 1, C // 5
            qg, kg = torch.randn(H * D, generator=g), torch.randn(G * D, generator=g)
            cs = slice(0, 5 * D)
            place = torch.arange(T, dtype=torch.int32)
            k2, v2 = torch.zeros(T // 16 + 1, G, 16, D).to(dtype), torch.zeros(T // 16 + 1, G, D, 16).to(dtype)
            k1, v1, s1, s2 = dev(k2.clone()), dev(v2.clone()), st.clone().to(DEV), st.clone()
            q1 = hip.projnorm_rope_store(dev(buf), H, G, D, D, dev(qg), dev(kg), 1e-5, 0, None, dev(place), k1, v1, 16,
                                         conv=(dev(w[cs].contiguous()), s1, 1, bd, True))
            q2 = emu.projnorm_rope_store(buf, H, G, D, D, qg, kg, 1e-5, 0, None, place, k2, v2, 16, conv=(w[cs], s2, 1, bh, True))
            for a, c in ((q1, q2), (k1, k2), (v1, v2)):
                close(a, c, 1e-5 if dtype == torch.float32 else 1e-2)
            if taps > 1:
                n = (taps - 1) * 5 * D
                close(s1[sorted(slots)][:, 1:1 + n], s2[sorted(slots)][:, 1:1 + n], 0)


@pytest.mark.parametrize("dtype", DTYPES)
@pytest.mark.parametrize("T,E,top,width,ff", [(1, 5, 2, 72, 24), (33, 7, 1, 64, 16), (9, 16, 16, 64, 48), (700, 8, 2, 256, 160),
                                              (1200, 12, 2, 128, 96), (64, 300, 3, 32, 32)])
def test_experts_weighted_on_their_inputs(dtype, T, E, top, width, ff):
    """16, 64 and 128 rows a tile, with and without the matrix cores; gated and ungated."""
    hip, emu = tables(dtype)
    g = torch.Generator().manual_seed(T)
    logits = 2 * torch.randn(T, E + 3, generator=g)
    x = torch.randn(T, width, generator=g).to(dtype)
    gu = (torch.randn(E, 2 * ff, width, generator=g) * width ** -0.5).to(dtype)
    down = (torch.randn(E, width, ff, generator=g) * ff ** -0.5).to(dtype)
    routing = hip.route_tokens(dev(logits), E, top, sigmoid=True)
    chosen, shares = emu.route_tokens(logits, E, top, sigmoid=True)
    assert torch.equal(routing.chosen.cpu(), chosen)
    close(routing.shares, shares, 1e-6)
    close(routing.shares, torch.sigmoid(torch.gather(logits.double(), 1, chosen.long())), 1e-6)
    tol = 2e-5 if dtype == torch.float32 else 2e-2
    for gated, act, w in ((True, "silu", gu), (False, "relu2", gu[:, :ff].contiguous())):
        mats = hip.prepare_expert_matrices(dev(w), gated=gated), hip.prepare_expert_matrices(dev(down))
        got = hip.routed_experts(dev(x), routing, *mats, activation=act, gated=gated, weigh_input=True)
        want = torch.zeros(T, width, dtype=torch.float64)
        for e in range(E):
            for k in range(top):
                rows = (chosen[:, k] == e).nonzero()[:, 0]
                z = (x[rows].double() * shares[rows, k:k + 1].double()) @ w[e].double().T
                mid = torch.nn.functional.silu(z[:, :ff]) * z[:, ff:] if gated else torch.relu(z) ** 2
                want[rows] += mid @ down[e].double().T
        close(got, want, tol)
        if T <= 33:
            close(got, emu.routed_experts(x, (chosen, shares), w, down, activation=act, gated=gated, weigh_input=True), tol)
