"""Each mechanism of the Derosun decoder alone, kernel by kernel: the norm behind the residual sum, the matrix memory with
exponential gates (chunks and single tokens), the rotations with scaled frequencies and with a magnitude on every path that
turns latent rows and queries, capped scores behind whole-row norms, and gated products with biases."""
import numpy as np
import pytest
import torch

import plain_derosun as P

pytestmark = pytest.mark.gpu

DEV = "cuda:0"
F64 = torch.float64
BF = torch.bfloat16


def rel(got, ref):
    return float((got.cpu().to(F64) - ref).abs().max()) / max(float(ref.abs().max()), 1e-30)


def workspace():
    from agave_amd.parts import Workspace
    return Workspace(torch.device(DEV))


def planner_for(key=None, slots=4, pages=60, dtype=torch.float32, context=4096):
    from agave_amd.cache import KVCache
    from agave_amd.engine.step import StepPlanner
    cache = KVCache({0: key} if key is not None else {}, {}, slots, {key: pages} if key is not None else {}, dtype, torch.device(DEV), context)
    return cache, StepPlanner(cache, 1000, torch.device(DEV))


# ---------------------------------------------------------------- the norm behind the residual sum
@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("n, e", [(1, 64), (5, 192), (300, 40), (70, 2560), (3, 6144), (2, 30), (9, 1), (4, 1023)])
@pytest.mark.parametrize("slices", [0, 1, 3, 11])
def test_norm_of_a_sum(dtype, n, e, slices):
    """h <- rms(alpha h + branch + bias) g with a branch in the activations' type or in 32-bit slices, with and without a
    bias; the rows handed on as they are, through a further norm, or not at all.  Rows that allow 16-byte accesses and not."""
    from agave_amd.ops import kernels
    g = torch.Generator().manual_seed(e + slices)
    alpha, eps, eps2 = 2.5, 3e-4, 1e-2
    h = torch.randn(n, e, generator=g)
    branch = torch.randn(slices, n, e, generator=g) if slices else torch.randn(n, e, generator=g).to(dtype)
    gain, gain2, bias = (1 + 0.3 * torch.randn(e, generator=g) for _ in range(3))
    whole = branch.to(F64).sum(0) if slices else branch.to(F64)
    tol = 3e-6 if dtype == torch.float32 else 5e-3
    for b in (None, bias):
        want = P.norm_of_sum(h.to(F64), whole + (b.to(F64) if b is not None else 0.0), gain.to(F64), alpha, eps)
        for pre in ("none", "rows", "norm"):
            hd, out = h.to(DEV), torch.full((n, e), 9.0, dtype=dtype, device=DEV)
            kernels.norm_of_sum(hd, branch.to(DEV), alpha, b.to(DEV) if b is not None else None, gain.to(DEV), eps,
                                None if pre == "none" else out, gain2.to(DEV) if pre == "norm" else None, eps2)
            assert rel(hd, want) < 3e-6, (pre, b is None)
            if pre == "rows":
                assert rel(out, want) < tol
            elif pre == "norm":
                assert rel(out, P.rms(want, eps2) * gain2.to(F64)) < tol


# ---------------------------------------------------------------- the matrix memory
class Memory:
    """Rows, state and plain results of a batch of sequences; ``run`` advances any of them by some tokens."""

    def __init__(self, heads, dk, dv, lens, seed, dtype=torch.float32, cap=6.0, f_bias=None, i_bias=None, slots=None):
        g = torch.Generator().manual_seed(seed)
        self.heads, self.dk, self.dv, self.lens, self.dtype = heads, dk, dv, lens, dtype
        self.cap, self.eps = cap, 2e-4
        self.width = (2 * heads * (dk + dv) + 2 * heads + 3) // 4 * 4
        self.rows = [torch.randn(t, self.width, generator=g) for t in lens]
        self.i_bias = i_bias if i_bias is not None else torch.randn(heads, generator=g)
        self.f_bias = f_bias if f_bias is not None else 2 + 2 * torch.randn(heads, generator=g)
        self.weight = 1 + 0.2 * torch.randn(heads * dv, generator=g)
        n_slots = slots or len(lens) + 1
        self.cache, self.planner = planner_for(slots=n_slots)
        self.slots = [self.cache.alloc_slot() for _ in lens]
        self.S = torch.zeros(n_slots, heads, dv, dk, device=DEV)
        self.n = torch.zeros(n_slots, heads, dk, device=DEV)
        self.m = torch.zeros(n_slots, heads, device=DEV)
        self.ws = workspace()

    def bounds(self):
        H, a, b = self.heads, self.heads * self.dk, self.heads * self.dv
        return [0, a, 2 * a, 2 * a + b, 2 * a + 2 * b, 2 * a + 2 * b + H, 2 * a + 2 * b + 2 * H]

    def run(self, which, counts, start):
        """The next ``counts[i]`` tokens, from ``start[i]`` on, of the sequences ``which``; their outputs."""
        from agave_amd.ops import mlstm as M
        step = self.planner.plan([self.slots[i] for i in which], [[0] * c for c in counts], "all")
        wide = torch.cat([self.rows[i][s:s + c] for i, c, s in zip(which, counts, start)]).to(DEV)
        cols = [wide[:, lo:hi] for lo, hi in zip(self.bounds()[:-1], self.bounds()[1:])]
        gates = M.Gates(self.i_bias.to(DEV), self.f_bias.to(DEV), self.cap, self.weight.to(DEV), self.eps, 1e-6, self.dk ** -0.5)
        out = torch.full((wide.shape[0], self.heads * self.dv), 9.0, dtype=self.dtype, device=DEV)
        M.mlstm(*cols, gates, out, self.S, self.n, self.m, step, self.heads, self.dk, self.dv, self.ws)
        self.planner.commit(step)
        return list(torch.split(out.cpu(), counts))

    def plain(self, i):
        """(outputs [T, heads * dv], per head (S, n, m)) of sequence i."""
        x, H, dk, dv = self.rows[i].to(F64), self.heads, self.dk, self.dv
        T, b = x.shape[0], self.bounds()
        q, k = x[:, b[0]:b[1]].view(T, H, dk) * dk ** -0.5, x[:, b[1]:b[2]].view(T, H, dk)
        v, gate = x[:, b[2]:b[3]].view(T, H, dv), x[:, b[3]:b[4]]
        li = P.capped(x[:, b[4]:b[5]] + self.i_bias.to(F64), self.cap)
        lf = torch.nn.functional.logsigmoid(P.capped(x[:, b[5]:b[6]] + self.f_bias.to(F64), self.cap))
        got = [P.matrix_memory(q[:, h], k[:, h], v[:, h], li[:, h], lf[:, h]) for h in range(H)]
        o = P.rms(torch.stack([x for x, _ in got], 1), self.eps).reshape(T, H * dv)
        return o * self.weight.to(F64) * torch.sigmoid(gate), [s for _, s in got]

    def check(self, got, i, what, states=True):
        want, ends = self.plain(i)
        # (a read-out that almost cancels is divided by something small, as in any 32-bit computation: one row in fifty may be
        # off by more than the rest)
        err = (got.to(F64) - want).abs().max(-1).values / float(want.abs().max())
        tol = 2e-5 if self.dtype == torch.float32 else 6e-3
        assert float(err.max()) < 20 * tol and int((err > tol).sum()) <= len(err) // 50, (what, float(err.max()), int(err.argmax()))
        if states:
            slot = self.slots[i]
            for h, (S, n, m) in enumerate(ends):
                # (m is rounded token by token, and S and n are relative to the rounded one)
                ahead = float(self.m[slot, h]) - m
                assert abs(ahead) < 1e-5 * max(1.0, abs(m)), (what, "m", h)
                off = rel(self.S[slot, h].double() * np.exp(ahead), S.T), rel(self.n[slot, h].double() * np.exp(ahead), n)
                assert max(off) < 2e-5, (what, h)


def cut(total, piece):
    return [min(piece, total - s) for s in range(0, total, piece)]


SIZES = [(3, 32, 80), (3, 20, 12), (1, 1, 1), (2, 10, 7), (4, 64, 48), (1, 128, 128), (2, 66, 130), (1, 256, 512), (1, 36, 600), (1, 300, 20),
         (1, 515, 40)]


@pytest.mark.parametrize("heads, dk, dv", SIZES)
def test_matrix_memory_in_every_cut(heads, dk, dv):
    """Whole (two chunks and a part), in pieces of 1, 2, 17, 128 and 129, and whole then token by token: outputs and final
    states.  Sizes in steps of four and not, of one, beyond a lane group and beyond four waves' columns."""
    T = 290 if dk * dv < 20000 else 150
    cuts = [[T], cut(T, 17), cut(T, 128), cut(T, 129), [T - 40] + [1] * 40]
    cuts += [cut(T, 1), cut(T, 2)] if dk * dv < 5000 else [cut(T, 32)]
    for c in cuts:
        M = Memory(heads, dk, dv, [T], seed=dk + dv)
        at, outs = 0, []
        for n in c:
            outs += M.run([0], [n], [at])
            at += n
        M.check(torch.cat(outs), 0, c[:3])


def test_matrix_memory_writes_bfloat16_rows():
    for n in ([200], [150] + [1] * 50):
        M = Memory(3, 48, 80, [200], seed=2, dtype=BF)
        at, outs = 0, []
        for c in n:
            outs += M.run([0], [c], [at])
            at += c
        M.check(torch.cat(outs), 0, n[:2])


def test_batches_of_unequal_sequences_and_slots_used_again():
    """Sequences of 1 to 400 tokens in one step, then token by token together, then others in the same slots (zeroed)."""
    lens = [300, 1, 64, 129, 128, 400, 2]
    M = Memory(2, 24, 40, lens, seed=8)
    first = [250, 1, 64, 100, 128, 257, 1]
    outs = [[o] for o in M.run(list(range(7)), first, [0] * 7)]
    used = list(first)
    while True:
        live = [i for i in range(7) if used[i] < lens[i]]
        if not live:
            break
        for i, o in zip(live, M.run(live, [1] * len(live), [used[i] for i in live])):
            outs[i].append(o)
            used[i] += 1
    for i in range(7):
        M.check(torch.cat(outs[i]), i, f"sequence {i}")
    N = Memory(2, 24, 40, [140, 30], seed=9, slots=8)
    N.S, N.n, N.m, N.slots = M.S, M.n, M.m, [M.slots[5], M.slots[0]]
    N.cache, N.planner = M.cache, M.planner
    for s in M.slots:
        M.cache.free_slot(s)
        for t in (M.S, M.n, M.m):
            t[s].zero_()
    N.slots = [N.cache.alloc_slot(), N.cache.alloc_slot()]
    for i, o in enumerate(N.run([0, 1], [140, 30], [0, 0])):
        N.check(o, i, "slots used again")


@pytest.mark.parametrize("f_bias, i_bias", [(-30.0, 0.0), (30.0, 0.0), (0.0, -30.0), (0.0, 30.0), (-30.0, -30.0), (30.0, 30.0), (1.0, 0.0)])
def test_gates_at_both_ends_of_their_cap(f_bias, i_bias):
    """Forget gates that keep everything or nothing, input gates far above and far below it: the running maximum stays at 0,
    falls, or follows the input gates, and the divisor's floor holds or does not."""
    for cap in (3.0, 15.0):
        M = Memory(2, 16, 24, [270], seed=4, cap=cap, f_bias=torch.full((2,), f_bias), i_bias=torch.full((2,), i_bias))
        a, b = M.run([0], [200], [0]), []
        for t in range(200, 270):
            b += M.run([0], [1], [t])
        M.check(torch.cat(a + b), 0, (cap, f_bias, i_bias))


def test_a_write_far_back():
    """One token writes with a gate that stands far above the others', 300 tokens before a query that looks for its key: a
    head that forgets slowly returns its value, one that forgets fast does not; across chunks, in prompts and token by token."""
    for run in ([330], [30, 300], [320] + [1] * 10, cut(330, 2)):
        M = Memory(2, 16, 8, [330], seed=6, cap=20.0, f_bias=torch.tensor([30.0, -1.0]), i_bias=torch.zeros(2))
        x, b = M.rows[0], M.bounds()
        x[:, b[4]:b[6]] = 0.0                                   # input gates of 1, forget gates of the biases
        x[:, b[0]:b[2]] *= 0.05
        x[5, b[4]:b[5]] = 9.0
        x[5, b[1]:b[2]] = 1.0
        x[5, b[2]:b[3]] = 40.0
        x[:, b[3]:b[4]] = 3.0
        x[329, b[0]:b[1]] = 2.0
        at, outs = 0, []
        for n in run:
            outs += M.run([0], [n], [at])
            at += n
        got = torch.cat(outs)
        M.check(got, 0, run[:2])
        y = got[-1].view(2, 8) / (M.weight.view(2, 8) * torch.sigmoid(torch.tensor(3.0)))
        assert float((y[0] - 1.0).abs().max()) < 0.02            # all of the written value: equal elements, normed to one
        assert float((y[1] - 1.0).abs().max()) > 0.3
        without = Memory(2, 16, 8, [330], seed=6, cap=20.0, f_bias=M.f_bias, i_bias=M.i_bias)
        without.rows[0] = x.clone()
        without.rows[0][5, b[2]:b[3]] = 0.0
        want, _ = without.plain(0)
        moved = (got[-1].to(F64) - want[-1]).view(2, 8).abs().max(-1).values
        assert float(moved[0]) > 0.3 and float(moved[1]) < 1e-5


# ---------------------------------------------------------------- rotations
@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("heads, dim, rot, kv_rank, q_rank", [(3, 12, 6, 40, 20), (5, 32, 16, 48, 64), (2, 1, 2, 1, 3), (16, 128, 64, 512, 96)])
def test_latent_rows_and_queries_turned_with_a_magnitude(dtype, heads, dim, rot, kv_rank, q_rank):
    """YaRN's frequencies with the magnitude on sine and cosine: the latent row, query rows turned apart and in place, and the
    trailing elements of the fold on both of its kernels and in a decode step's joint launch."""
    from agave_amd.cache import GroupKey
    from agave_amd.ops import latent as L
    eps, qd, kd = 2e-4, dim + rot, kv_rank + rot
    conf = {"base": 300.0, "dims": rot, "scaling": {"factor": 6.0, "original": 200, "fast": 16.0, "slow": 1.0}}
    freq, mag = P.yarn_frequencies(conf), P.yarn_magnitude(conf)
    turn = L.Turn(torch.tensor(freq, dtype=F64, device=DEV), True, mag)
    tol = 3e-6 if dtype == torch.float32 else 5e-3
    for n, decode in ((75, False), (9, True)):
        g = torch.Generator().manual_seed(dim + n)
        cache, planner = planner_for(GroupKey(None, 1, kd, v_head_dim=kv_rank, layout="rows_vt"), slots=9, dtype=dtype, pages=260)
        slots = [cache.alloc_slot() for _ in range(n if decode else 1)]
        planner.commit(planner.plan(slots, [[0] * (900 + 11 * i) for i in range(len(slots))], "all"))
        step = planner.plan(slots, [[0]] * n if decode else [[0] * n], "all")
        wide = torch.randn(n, (q_rank + kd + heads * qd + 3) // 4 * 4, generator=g) * 2
        w, wq = 1 + 0.3 * torch.randn(kv_rank, generator=g), 1 + 0.3 * torch.randn(q_rank, generator=g)
        dev, pos, x = wide.to(DEV), step.tok_pos.cpu().long(), wide.to(F64)
        q0 = heads * qd
        table, tbase = step.tables[0]
        kp, vp, packed = cache.pages_of(0)
        pages = L.CachePages(kp, vp, table, tbase, packed)
        cq, row = torch.empty(n, q_rank, dtype=dtype, device=DEV), torch.empty(n, kd, dtype=dtype, device=DEV)
        L.latent_prepare(step, eps, turn, rot, q_raw=dev[:, q0:q0 + q_rank], q_weight=wq.to(DEV), q_out=cq, kv_raw=dev[:, q0 + q_rank:q0 + q_rank + kd],
                         kv_weight=w.to(DEV), k_row=row, kv_rank=kv_rank, pages=pages)
        kv = x[:, q0 + q_rank:q0 + q_rank + kd]
        want_row = torch.cat([P.rms(kv[:, :kv_rank], eps) * w.to(F64), P.turn_neighbours(kv[:, None, kv_rank:], pos, freq, mag)[:, 0]], -1)
        assert rel(cq, P.rms(x[:, q0:q0 + q_rank], eps) * wq.to(F64)) < tol and rel(row, want_row) < tol
        q64 = x[:, :q0].view(n, heads, qd)
        want_q = torch.cat([q64[..., :dim], P.turn_neighbours(q64[..., dim:], pos, freq, mag)], -1).reshape(n, -1)
        typed = dev[:, :q0].to(dtype).contiguous()
        apart = torch.empty_like(typed)
        L.turn_queries(typed, apart, heads, dim, rot, turn, step.tok_pos)
        L.turn_queries(typed, typed, heads, dim, rot, turn, step.tok_pos)
        assert torch.equal(typed, apart) and rel(apart, want_q) < 3 * tol
        fold = (torch.randn(heads, kv_rank, dim, generator=g) * dim ** -0.5).to(dtype)
        tail = torch.cat([torch.einsum("thk,hck->thc", q64[..., :dim], fold.to(F64)), want_q.view(n, heads, qd)[..., dim:]], -1).reshape(n, -1)
        for plain in (True, False):
            y = torch.empty(n, heads * kd, dtype=dtype, device=DEV)
            L.heads_product(dev[:, :q0], fold.to(DEV), y, heads, qd, kd, tail=rot, turn=turn, tok_pos=step.tok_pos, force_plain=plain)
            assert rel(y, tail) < 3 * tol, plain
        if decode and dtype == BF and L.decode_rows_ok(dev[:, :q0], heads, dim, rot) and (q0 + q_rank) % 4 == 0:
            y2 = torch.empty_like(y)
            L.decode_rows(dev[:, :q0], fold.to(DEV), y2, heads, dim, rot, turn, dev[:, q0 + q_rank:q0 + q_rank + kd], w.to(DEV), kv_rank, pages, step, eps)
            assert torch.equal(y, y2)


@pytest.mark.parametrize("dtype", [torch.float32, BF])
@pytest.mark.parametrize("H, G, d, rot, vd", [(6, 3, 16, 8, 16), (4, 4, 32, 32, 48), (5, 1, 48, 20, 20), (6, 1, 128, 64, 96), (1, 1, 10, 2, 7)])
def test_attention_with_row_norms_banded_rotation_and_capped_scores(dtype, H, G, d, rot, vd):
    """Rows normed whole and turned, into pages, then the attention with a cap that the largest scores are far beyond: a
    prompt, and single rows behind it."""
    from agave_amd.cache import GroupKey
    from agave_amd.ops import attention_biased as A
    T, eps, scale, cap = 150, 1e-4, 2.0, 5.0
    conf = {"base": 800.0, "dims": rot, "scaling": {"factor": 4.0, "low": 1.0, "high": 4.0, "original": 60}}
    freq = P.banded_frequencies(conf)
    g = torch.Generator().manual_seed(d)
    cache, planner = planner_for(GroupKey(None, G, d, v_head_dim=vd, layout="rows_vt"), dtype=dtype)
    slot = cache.alloc_slot()
    wide = torch.randn(T, (H + G) * d + G * vd, generator=g)
    qw, kw = 1 + 0.2 * torch.randn(H * d, generator=g), 1 + 0.2 * torch.randn(G * d, generator=g)
    x, pos = wide.to(F64), torch.arange(T)
    q = P.turn_halves((P.rms(x[:, :H * d], eps) * qw.to(F64)).view(T, H, d), pos, freq)
    k = P.turn_halves((P.rms(x[:, H * d:(H + G) * d], eps) * kw.to(F64)).view(T, G, d), pos, freq)
    v = x[:, (H + G) * d:].view(T, G, vd)
    s = [q[:, n] @ k[:, n // (H // G)].T * scale for n in range(H)]
    assert max(float(z.abs().max()) for z in s) > 2 * cap
    want = torch.stack([P.softmax_seen(P.capped(s[n], cap)) @ v[:, n // (H // G)] for n in range(H)], 1).reshape(T, -1)
    kp, vp, packed = cache.pages_of(0)
    fr = torch.tensor(freq, dtype=F64, device=DEV)
    ws = workspace()
    got, at = [], 0
    for c in [120, 5] + [1] * 25:
        step = planner.plan([slot], [[0] * c], "all")
        table, base = step.tables[0]
        dev = wide[at:at + c].to(DEV)
        q_out, out = torch.empty(c, H * d, dtype=dtype, device=DEV), torch.empty(c, H * vd, dtype=dtype, device=DEV)
        A.row_norm_rope(dev[:, :H * d], dev[:, H * d:(H + G) * d], dev[:, (H + G) * d:], q_out, None, None, qw.to(DEV), kw.to(DEV), eps, eps, fr,
                        1.0, step, H, G, d, vd, pages=(kp, vp, table, base, 0, packed))
        A.attention(q_out, out, None, kp, vp, table, base, 0, step, H, G, d, vd, scale, None, 0, A.BIAS_NONE, None, None, packed, workspace=ws,
                    softcap=cap)
        planner.commit(step)
        got.append(out.cpu())
        at += c
    err = (torch.cat(got).to(F64) - want).abs().max() / want.abs().max()
    assert float(err) < (5e-6 if dtype == torch.float32 else 2e-2)


# ---------------------------------------------------------------- gated products with biases
@pytest.mark.parametrize("m", [1, 5, 40, 64, 65, 300])
@pytest.mark.parametrize("ff, k", [(24, 40), (200, 96), (513, 256), (7, 64)])
def test_gated_products_with_biases(m, ff, k):
    """Skinny and tiled products, every tile shape, and the product that makes its normalised row itself, for SiLU, GELU and
    the clamped swish; biases large enough that a neighbour's would show."""
    from agave_amd.ops import gemm_mfma as G
    g = torch.Generator().manual_seed(m + ff)
    w = (torch.randn(2 * ff, k, generator=g) * k ** -0.5).to(BF)
    x = torch.randn(m, k, generator=g).to(BF)
    gb, ub = torch.randn(ff, generator=g) * 2, torch.randn(ff, generator=g) * 2

    def forms(z):
        a, b = z[:, :ff] + gb.to(F64), z[:, ff:] + ub.to(F64)
        c = torch.clamp(a, max=1.3)
        return {"silu": a * torch.sigmoid(a) * b, "gelu_tanh": torch.nn.functional.gelu(a, approximate="tanh") * b,
                "swish_clamped": c * torch.sigmoid(1.702 * c) * (torch.clamp(b, -1.3, 1.3) + 1.0)}
    packed = G.pack_weight(w.to(DEV), interleave_ff=ff)
    for act, ref in forms(x.to(F64) @ w.to(F64).T).items():
        form = G.gate_form_of(act, 1.3, 1.702)._replace(gate_bias=gb.to(DEV), up_bias=ub.to(DEV))
        out = torch.empty(m, ff, dtype=BF, device=DEV)
        G.product(x.to(DEV), packed, out, ff, epilogue=1, form=form)
        assert rel(out, ref) < 5e-3, act
        if m > 64:
            for tile in range(4):
                out.fill_(9.0)
                G.tiled_as(x.to(DEV), packed, out, ff, tile, epilogue=1, form=form)
                assert rel(out, ref) < 5e-3, (act, tile)
        if m == 1:
            h, gain = torch.randn(1, k, generator=g), 1 + 0.2 * torch.randn(k, generator=g)
            G.row_normed(h.to(DEV), None, None, None, 0.0, gain.to(DEV), 1e-5, packed, out, ff, epilogue=1, form=form)
            xn = (P.rms(h.to(F64), 1e-5) * gain.to(F64)).to(BF).to(F64)
            assert rel(out, forms(xn @ w.to(F64).T)[act]) < 2e-2, act
    with pytest.raises(ValueError, match="neither"):
        G.product(x.to(DEV), packed, out, ff, epilogue=1, form=form._replace(up_bias=None))
    with pytest.raises(TypeError, match="bias"):
        G.product(x.to(DEV), packed, out, ff, epilogue=1, form=form._replace(up_bias=gb[:-1].to(DEV), gate_bias=gb[:-1].to(DEV)))


def test_biases_of_a_gated_product_in_two_launches():
    """More 256 x 256 tiles than compute units: the last rows run in a second launch, with the biases that are theirs."""
    from agave_amd.ops import gemm_mfma as G
    m, ff, k = 2048, 4224, 64
    g = torch.Generator().manual_seed(5)
    w, x = (torch.randn(2 * ff, k, generator=g) * k ** -0.5).to(BF), torch.randn(m, k, generator=g).to(BF)
    gb, ub = torch.randn(ff, generator=g) * 2, torch.randn(ff, generator=g) * 2
    z = (x.to(DEV).float() @ w.to(DEV).float().T).cpu()
    a, b = z[:, :ff] + gb, z[:, ff:] + ub
    out = torch.empty(m, ff, dtype=BF, device=DEV)
    form = G.gate_form_of("silu")._replace(gate_bias=gb.to(DEV), up_bias=ub.to(DEV))
    G.product(x.to(DEV), G.pack_weight(w.to(DEV), interleave_ff=ff), out, ff, epilogue=1, form=form)
    assert rel(out, (a * torch.sigmoid(a) * b).to(F64)) < 5e-3


# ---------------------------------------------------------------- one layer of each kind
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("layer", [
    P.attention_layer(4, 2, 16, 24, 8, mlp=None), P.latent_layer(3, 8, 6, 16, 24, 16, mlp=None), P.mlstm_layer(2, 12, 20, mlp=None),
    P.mlstm_layer(1, 8, 16, mlp=P.dense(40))], ids=["attention", "latent", "mlstm", "mlstm and feed-forward"])
def test_a_model_of_one_layer(dtype, layer):
    """First tokens alone, pieces of two and three, decoding across a page's border."""
    import engine_utils as U
    from agave_amd.engine import Engine
    cfg = P.config([layer], vocab=61, width=48, alpha=0.7, embed_scale=2.0)
    w = P.random_weights(cfg, 12)
    eng = Engine.from_tensors(cfg, {k: v.bfloat16() for k, v in w.items()}, dtype=dtype, max_slots=1, max_context=128)
    toks = U.random_tokens(70, 61, 3)
    ref = P.forward(cfg, w, toks)
    tol = (3e-5 if dtype == "float32" else 0.06) * float(ref.abs().max())
    runs = {"first": (U.run_whole(eng, toks[:1]), ref[:1]), "tail": (U.run_tail(eng, toks, 20), ref)}
    for piece in (2, 3):
        eng.prefill_chunk = piece
        runs[f"pieces of {piece}"] = (U.run_whole(eng, toks), ref)
    for what, (got, want) in runs.items():
        off = float((got.double() - want).abs().max())
        assert off < tol, what
