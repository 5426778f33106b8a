"""The Derosun decoder through the engine, against ``plain_derosun``: whole prompts, decoding token by token, prompts in
pieces down to two tokens, batches of unequal requests, slots and pages used again, long decoding across page and chunk
borders, a key made to stand out far back and at page borders, a state that keeps one token's write, the first tokens of a
sequence, faults planted in the plain implementation that must show, other sizes (also ones where the usual sizes coincide or
are 1), the residual after every layer, greedy generation through the engine's entry point, the command line and the trace
replay tool."""
import json
import os
import random
import subprocess
import sys

import numpy as np
import pytest
import torch

import engine_utils as U
import plain_derosun as P

pytestmark = pytest.mark.gpu

CONFIGS = {
    # every mixer, with and without a feed-forward, sizes that are no multiples of 16
    "mixed": lambda: P.config([
        P.attention_layer(6, 3, 16, 20, 8, base=900.0, factor=3.0, low=1.5, high=5.0, original=70, softcap=6.0, mlp=P.dense(24)),
        P.mlstm_layer(3, 12, 20, gate_cap=7.5, mlp=None),
        P.latent_layer(3, 12, 6, 20, 28, 40, base=500.0, factor=5.0, fast=20.0, slow=2.0, original=90, mlp=P.dense(56)),
        P.mlstm_layer(2, 16, 8, gate_cap=11.0, mlp=P.dense(40)),
        P.attention_layer(4, 1, 24, 16, 24, mlp=None)], vocab=131, width=40, eps=2e-6, alpha=1.75, embed_scale=0.8),
    # a width that is no multiple of 8 (no matrix-core packing), one head everywhere, state rows that are no steps of four,
    # latents of one element, one pair turned, a factor on the stream below one
    "odd": lambda: P.config([
        P.mlstm_layer(1, 10, 7, gate_cap=4.0, mlp=P.dense(30)),
        P.latent_layer(1, 5, 2, 3, 1, 1, base=30.0, factor=2.0, original=20, mlp=None),
        P.attention_layer(1, 1, 10, 7, 2, base=3.0, factor=2.5, original=40, softcap=3.0, mlp=P.dense(18)),
        P.mlstm_layer(5, 3, 1, gate_cap=20.0, mlp=None),
        P.latent_layer(5, 1, 4, 7, 3, 19, base=77.0, factor=1.0, mlp=P.dense(30))], vocab=97, width=60, eps=1e-3, alpha=0.6, embed_scale=7.0),
    # sizes the matrix cores take everywhere, the prompt form with every head's own keys
    "even": lambda: P.config([
        P.mlstm_layer(4, 32, 64, mlp=None),
        P.latent_layer(8, 16, 8, 32, 64, 48, mlp=P.dense(256)),
        P.attention_layer(8, 2, 32, 32, 16, original=128, mlp=P.dense(192)),
        P.latent_layer(20, 32, 16, 16, 32, 64, base=100.0, factor=8.0, original=100, mlp=P.dense(64)),
        P.mlstm_layer(2, 64, 32, mlp=P.dense(64))], vocab=256, width=128, alpha=3.0, embed_scale=2.0),
    # wide heads of state (two and four loads a lane, more columns than four waves hold), the widest latent rows
    "wide": lambda: P.config([
        P.mlstm_layer(1, 260, 530, mlp=P.dense(40)),
        P.latent_layer(3, 64, 64, 80, 40, 512, original=50, mlp=None),
        P.mlstm_layer(2, 128, 96, mlp=None)], vocab=61, width=72),
}


@pytest.fixture(scope="module")
def models(tmp_path_factory):
    made = {}

    def get(name):
        if name not in made:
            cfg = CONFIGS[name]()
            w = P.random_weights(cfg, seed=len(name))
            folder = U.write_model(str(tmp_path_factory.mktemp(name)), cfg, w)
            made[name] = (cfg, w, folder)
        return made[name]
    return get


def engine(folder, dtype, **kw):
    from agave_amd.engine import Engine
    kw.setdefault("max_slots", 4)
    kw.setdefault("max_context", 512)
    return Engine.from_folder(folder, dtype=dtype, **kw)


def plain(cfg, w, toks, dtype):
    """(logits, how much each position's may be off in bfloat16 beyond the usual: three times what shaking moves them)."""
    ref = P.forward(cfg, w, toks)
    return ref, (3.0 * P.sensitivity(cfg, w, toks, ref) if dtype == "bfloat16" else torch.zeros(len(toks), dtype=P.F))


def close(got, want, dtype, what):
    """32-bit: every row within 4e-5 of the largest logit (one in fifty, a read-out that almost cancels and is normed to
    one, within ten times that).  bfloat16: 4 % of the largest logit, or what the position is sensitive to, for all rows but
    one in twenty, twice that for those; most rows are not sensitive."""
    ref, slack = want
    scale = float(ref.abs().max())
    err = (got.double() - ref).abs().max(dim=-1).values
    where = f"{what}: error {float(err.max()):.3e} of {scale:.3e} at row {int(err.argmax())}"
    if dtype == "float32":
        assert float(err.max()) <= 4e-4 * scale, where
        assert int((err > 4e-5 * scale).sum()) <= len(err) // 50, where
    else:
        most = torch.clamp(slack, min=0.04 * scale)
        assert int((most > 0.08 * scale).sum()) <= max(1, len(err) // 3), f"{what}: the positions are too sensitive to tell"
        assert int((err > 2 * most).sum()) == 0, where
        assert int((err > most).sum()) <= max(1, len(err) // 20), where


def rows(want, n):
    return want[0][:n], want[1][:n]


@pytest.mark.parametrize("name", list(CONFIGS))
@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_whole_tail_and_pieces(models, name, dtype):
    cfg, w, folder = models(name)
    eng = engine(folder, dtype)
    toks = U.random_tokens(200, cfg["vocab"], 1)
    ref = plain(cfg, w, toks, dtype)
    close(U.run_whole(eng, toks), ref, dtype, "whole")
    close(U.run_tail(eng, toks, 150), ref, dtype, "the last 150 one by one, across page and chunk borders")
    close(U.run_tail(eng, toks, 199), ref, dtype, "token by token from the first")
    for piece in (2, 7, 64, 100):                 # the prompt enters in pieces of this many tokens
        eng.prefill_chunk = piece
        close(U.run_whole(eng, toks[:170]), rows(ref, 170), dtype, f"pieces of {piece}")
    eng.prefill_chunk = 0
    assert eng.cache.slots.n_free == eng.cache.max_slots
    assert all(g.pool.n_free == g.pool.n_pages for g in eng.cache.groups)


@pytest.mark.parametrize("name", ["mixed", "even"])
def test_residual_after_every_layer(models, name):
    """The residual stream after each layer, read off the engine between its blocks."""
    from agave_amd.parts.norm import add_branch
    cfg, w, folder = models(name)
    eng = engine(folder, "float32")
    eng.use_graphs = False
    toks = U.random_tokens(90, cfg["vocab"], 4)
    want, seen = [], []
    P.forward(cfg, w, toks, layers_out=want)
    for b in eng.model.blocks:
        def wrapped(h, pending, step, memory, writes, inner=b.forward):
            if pending is not None:
                stream = h.clone()
                add_branch(stream, pending)
                seen.append(stream.cpu())
            return inner(h, pending, step, memory, writes)
        b.forward = wrapped
    U.run_whole(eng, toks)
    assert len(seen) == len(want) - 1 == 4
    for i, (got, ref) in enumerate(zip(seen, want)):
        assert float((got.double() - ref).abs().max()) < 3e-5 * float(ref.abs().max()), f"after layer {i}"


@pytest.mark.parametrize("name, dtype", [("mixed", "float32"), ("mixed", "bfloat16"), ("even", "bfloat16")])
def test_batches_of_unequal_requests_and_slots_used_again(models, name, dtype):
    """Three batches one after another over the same three slots, through pools of pages that only hold them because
    pages come back."""
    cfg, w, folder = models(name)
    eng = engine(folder, dtype, max_slots=3, max_context=256, cache_tokens=448)
    for b, (lens, first) in enumerate([((50, 1, 150), (30, 1, 2)), ((70, 33), (69, 1)), ((90, 9, 140), (5, 9, 131))]):
        reqs = [U.random_tokens(n, cfg["vocab"], 10 * b + i) for i, n in enumerate(lens)]
        outs = U.run_batched(eng, reqs, first)
        for i, (r, o) in enumerate(zip(reqs, outs)):
            close(o, plain(cfg, w, r, dtype), dtype, f"batch {b} request {i}")
    assert eng.cache.slots.n_free == eng.cache.max_slots
    assert all(g.pool.n_free == g.pool.n_pages for g in eng.cache.groups)


def test_a_batch_of_more_than_sixteen(models):
    """Eighteen sequences decoded together."""
    cfg, w, folder = models("even")
    eng = engine(folder, "bfloat16", max_slots=18, max_context=192)
    reqs = [U.random_tokens(70 + 3 * i, cfg["vocab"], 300 + i) for i in range(18)]
    for r, o in zip(reqs, U.run_batched(eng, reqs, [len(r) - 12 for r in reqs])):
        close(o, plain(cfg, w, r, "bfloat16"), "bfloat16", f"{len(r)} tokens in a batch of eighteen")


def test_a_request_alone_and_in_a_batch_give_the_same(models):
    """What else is in the step does not show beyond rounding."""
    cfg, w, folder = models("mixed")
    for dtype, tol in (("float32", 2e-5), ("bfloat16", 0.03)):
        eng = engine(folder, dtype)
        reqs = [U.random_tokens(n, cfg["vocab"], 500 + n) for n in (140, 20, 67)]
        together = U.run_batched(eng, reqs, (120, 3, 66))
        for r, o, head in zip(reqs, together, (120, 3, 66)):
            alone = U.run_tail(eng, r, len(r) - head)
            assert float((alone - o).abs().max()) < tol * float(alone.abs().max())


def test_the_cache_as_the_mixers_asked(models):
    cfg, w, folder = models("mixed")
    eng = engine(folder, "bfloat16")
    keys = {m: eng.cache.group_keys[g] for m, g in eng.cache.group_of_memory.items()}
    assert set(keys) == {0, 2, 4} and set(eng.cache.state) == {1, 3}
    assert (keys[0].n_kv_heads, keys[0].head_dim, keys[0].v_head_dim) == (3, 16, 20) and (keys[2].n_kv_heads, keys[2].head_dim, keys[2].v_head_dim) == (1, 46, 40)
    state = eng.cache.state[1]
    assert {k: tuple(v.shape) for k, v in state.items()} == {"S": (4, 3, 20, 12), "n": (4, 3, 12), "m": (4, 3)}
    slot = eng.alloc_slot()
    eng.step([slot], [[1, 2]])
    assert all(float(t[slot].abs().max()) > 0 for t in (state["S"], state["n"]))
    eng.free_slot(slot)
    assert eng.alloc_slot() == slot and all(float(t[slot].abs().max()) == 0 for t in state.values())
    eng.free_slot(slot)
    from agave_amd.ops import library
    loaded = library.loaded_paths()
    for name in ("mlstm.so", "latent.so", "attention_biased.so", "elementwise.so", "gemm_mfma.so"):
        assert any(p.endswith(name) for p in loaded), name


def test_biases_ride_inside_other_kernels(models):
    """A layer's feed-forward biases cost no kernel of their own in bfloat16: gate's and up's inside the product's form, down's
    inside the norm of the sum."""
    cfg, w, folder = models("even")
    eng = engine(folder, "bfloat16")
    eng.enable_profiling(True)
    slot = eng.alloc_slot()
    eng.step([slot], [U.random_tokens(70, cfg["vocab"], 1)])
    eng.step([slot], [[3]])
    ops = {name.split(":")[0] for name, _, _ in eng.profile_table()}
    eng.enable_profiling(False)
    assert "norm_of_sum" in ops and "mlstm_chunks" in ops and "mlstm_step" in ops
    assert not ops & {"add_bias", "gated_act"}, ops


@pytest.mark.parametrize("name, dtype", [("even", "float32"), ("even", "bfloat16"), ("mixed", "float32")])
def test_long_decoding(models, name, dtype):
    cfg, w, folder = models(name)
    eng = engine(folder, dtype, max_slots=1, max_context=1024, cache_tokens=64 * 11)
    toks = U.random_tokens(700, cfg["vocab"], 9)
    close(U.run_tail(eng, toks, 500), plain(cfg, w, toks, dtype), dtype, "500 tokens decoded")


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
def test_the_first_tokens(models, dtype):
    """Sequences of one, two and three tokens, alone and together."""
    cfg, w, folder = models("even")
    eng = engine(folder, dtype, max_slots=3)
    reqs = [U.random_tokens(n, cfg["vocab"], 60 + n) for n in (1, 2, 3)]
    refs = [plain(cfg, w, r, dtype) for r in reqs]
    for r, ref in zip(reqs, refs):
        close(U.run_whole(eng, r), ref, dtype, f"{len(r)} tokens")
    for o, ref in zip(U.run_batched(eng, reqs, (1, 1, 1)), refs):
        close(o, ref, dtype, "together, one by one")


# ---------------------------------------------------------------- one token that stands out
VOCAB_NEEDLE = 40
A, Q = 0, 1


def needle_model(kind: str):
    """One layer that is made to look for one token: the key of token ``A`` is turned towards the query of token ``Q`` (in
    elements that are not rotated) and its value made large, so that the logits at a ``Q`` change much with whether ``A`` is
    seen.  A layer's input is a function of the token alone in a model of one layer, and there are fewer tokens than the rows
    are long: the matrices are changed along the part of ``A``'s row that is orthogonal to every other token's, so no other
    token's key or value moves."""
    if kind == "attention":
        # (k's whole row is normed: a boost in one head's key shrinks the row's other elements for A alone)
        cfg = P.config([P.attention_layer(2, 1, 16, 12, 8, scale=1.0, softcap=30.0)], vocab=VOCAB_NEEDLE, width=64, alpha=1.0, embed_scale=1.0)
    elif kind == "latent":
        cfg = P.config([P.latent_layer(2, 8, 8, 12, 32, 64)], vocab=VOCAB_NEEDLE, width=64, alpha=1.0, embed_scale=1.0)
    else:
        cfg = P.config([P.mlstm_layer(2, 16, 12, gate_cap=30.0)], vocab=VOCAB_NEEDLE, width=64, alpha=1.0, embed_scale=1.0)
    w = P.random_weights(cfg, 3)
    eps, m, p = cfg["norm"]["eps"], cfg["layers"][0]["mixer"], "l0.mix."
    h = w["embed"]                                                          # [vocab, width]: every token's input

    def only_for_a(rows):
        coef = torch.linalg.lstsq(rows[1:].T, rows[A][:, None]).solution[:, 0]
        d = rows[A] - rows[1:].T @ coef                                     # orthogonal to every other token's row
        return d / float(d @ rows[A])
    if kind == "attention":
        q0 = (P.rms(h[Q] @ w[p + "q"].T, eps) * w[p + "q.norm"]).view(2, 16)[0].clone()
        q0[:8] = 0.0
        d = only_for_a(h)
        w[p + "q"][8:16] *= 6.0
        w[p + "k"] = w[p + "k"] + 60.0 * torch.outer(q0 / q0.norm(), d)
        w[p + "v"] = w[p + "v"] + 25.0 * torch.outer(torch.ones(12, dtype=P.F), d)
        names = [p + "q", p + "k", p + "v"]
    elif kind == "latent":
        c = P.rms((h @ w[p + "dkv"].T)[:, :m["kv_rank"]], eps) * w[p + "dkv.norm"]
        cq = P.rms(h[Q] @ w[p + "dq"].T, eps) * w[p + "dq.norm"]
        q0 = (w[p + "uq"] @ cq).view(2, 16)[0, :8]
        d = only_for_a(c)
        w[p + "uk"][:8] += 30.0 * torch.outer(q0 / (q0.norm() ** 2), d) / m["scale"]
        w[p + "uv"][:12] += 25.0 * torch.outer(torch.ones(12, dtype=P.F), d)
        names = [p + "uk", p + "uv"]
    else:
        # A's input gate stands 12 above the others'; the forget gates keep (head 0) or drop (head 1)
        d = only_for_a(h)
        w[p + "i"] *= 0.2
        w[p + "f"] *= 0.2
        w[p + "i.b"][:], w[p + "f.b"][:] = 0.0, torch.tensor([12.0, -2.0], dtype=P.F)
        w[p + "i"] = w[p + "i"] + 12.0 * torch.outer(torch.ones(2, dtype=P.F), d)
        q0 = (h[Q] @ w[p + "q"].T).view(2, 16)[0]
        w[p + "k"][:16] += 8.0 * torch.outer(q0 / q0.norm(), d)
        w[p + "v"][:12] += 5.0 * torch.outer(torch.ones(12, dtype=P.F), d)
        names = [p + "i", p + "f", p + "k", p + "v"]
    for n in names:
        w[n] = w[n].to(torch.float32).to(P.F)
    return cfg, w


@pytest.mark.parametrize("dtype", ["float32", "bfloat16"])
@pytest.mark.parametrize("kind", ["attention", "latent", "mlstm"])
def test_a_token_that_stands_out_far_back(dtype, kind):
    """The token that the last query looks for stands at the sequence's first positions, on both sides of pages' and chunks'
    borders, and beside the query; the query comes in the prompt, in pieces of it, and decoded."""
    from agave_amd.engine import Engine
    cfg, w = needle_model(kind)
    # (the changed matrices are handed over in 32-bit, so that the orthogonal direction survives; a bfloat16 engine casts them)
    eng = Engine.from_tensors(cfg, {k: v.float() for k, v in w.items()}, dtype=dtype, max_slots=2, max_context=512,
                              keep_stored_precision=False)
    T = 420
    for at in (0, 1, 63, 64, 127, 128, 300, T - 2):
        toks = [2 + t % (VOCAB_NEEDLE - 2) for t in U.random_tokens(T, 1000, at + 5)]
        toks[-1] = Q
        toks[at] = A
        without = list(toks)
        without[at] = 7
        ref, ref_without = P.forward(cfg, w, toks), P.forward(cfg, w, without)
        scale = float(ref.abs().max())
        moved = float((ref[-1] - ref_without[-1]).abs().max())
        assert moved > 0.1 * scale, (at, moved, scale)
        eng.prefill_chunk = 0
        runs = {"whole": U.run_whole(eng, toks), "decoded": U.run_tail(eng, toks, 60 if at < 300 else T - at + 3)}
        eng.prefill_chunk = 50
        runs["pieces"] = U.run_whole(eng, toks)
        for what, got in runs.items():
            if dtype == "float32":
                close(got, (ref, None), dtype, f"token at {at}, {what}")
            assert float((got[-1].double() - ref[-1]).abs().max()) < (0.002 if dtype == "float32" else 0.25) * moved, (at, what)


# ---------------------------------------------------------------- faults planted in the plain implementation
def planted(monkeypatch, fault):
    """The plain implementation with one mistake."""
    def wrapped_memory(change):
        def memory(q, k, v, i, f, state=None, inner=P.matrix_memory):
            return inner(*change(q, k, v, i, f), state)
        monkeypatch.setattr(P, "matrix_memory", memory)
    if fault == "the norm in front of the sum":
        monkeypatch.setattr(P, "norm_of_sum", lambda x, b, g, alpha, eps: alpha * x + P.rms(b, eps) * g)
    elif fault == "no factor on the stream":
        inner = P.norm_of_sum
        monkeypatch.setattr(P, "norm_of_sum", lambda x, b, g, alpha, eps: inner(x, b, g, 1.0, eps))
    elif fault == "scores without their cap":
        monkeypatch.setattr(P, "capped", lambda z, cap: z if cap == 6.0 or cap == 15.0 else cap * torch.tanh(z / cap))
    elif fault == "gates without their cap":
        monkeypatch.setattr(P, "capped", lambda z, cap: z if cap == 7.5 or cap == 11.0 else cap * torch.tanh(z / cap))
    elif fault == "plain frequencies in attention":
        monkeypatch.setattr(P, "banded_frequencies", P.plain_frequencies)
    elif fault == "plain frequencies in latent attention":
        monkeypatch.setattr(P, "yarn_frequencies", P.plain_frequencies)
    elif fault == "no magnitude":
        monkeypatch.setattr(P, "yarn_magnitude", lambda rot: 1.0)
    elif fault == "the other pairs turned":
        monkeypatch.setattr(P, "turn_neighbours", lambda x, pos, f, mag: torch.cat(
            [mag * P.turn_halves(x, pos, f)[..., :2 * len(f)], x[..., 2 * len(f):]], -1))
    elif fault == "norms per head":
        def attention(h, w, p, m, eps, inner=P.rms):
            T, H, G, d, vd = h.shape[0], m["heads"], m["kv_heads"], m["dim"], m["vdim"]
            pos, freq = torch.arange(T), P.banded_frequencies(m["rot"])
            q = inner((h @ w[p + "q"].T).view(T, H, d), eps) * w[p + "q.norm"].view(H, d)
            k = inner((h @ w[p + "k"].T).view(T, G, d), eps) * w[p + "k.norm"].view(G, d)
            q, k, v = P.turn_halves(q, pos, freq), P.turn_halves(k, pos, freq), (h @ w[p + "v"].T).view(T, G, vd)
            out = torch.stack([P.softmax_seen(P.capped((q[:, n] @ k[:, n // (H // G)].T) * m["scale"], m["softcap"])) @ v[:, n // (H // G)]
                               for n in range(H)], 1)
            return out.reshape(T, H * vd) @ w[p + "o"].T
        monkeypatch.setattr(P, "attention", attention)
    elif fault == "queries of the memory without their scale":
        wrapped_memory(lambda q, k, v, i, f: (q * q.shape[1] ** 0.5, k, v, i, f))
    elif fault == "keys of the memory scaled too":
        wrapped_memory(lambda q, k, v, i, f: (q, k * k.shape[1] ** -0.5, v, i, f))
    elif fault == "no divisor":
        def memory(q, k, v, i, f, state=None, inner=P.matrix_memory):
            o, end = inner(q, k, v, i, f, state)
            return o * 0 + torch.stack([inner(q[:t + 1], k[:t + 1], v[:t + 1], i[:t + 1], f[:t + 1], state)[1][0].T @ q[t] for t in range(q.shape[0])]), end
        monkeypatch.setattr(P, "matrix_memory", memory)
    elif fault == "the divisor's floor at one":
        def memory(q, k, v, i, f, state=None):
            S, n, m = torch.zeros(q.shape[1], v.shape[1], dtype=P.F), torch.zeros(q.shape[1], dtype=P.F), 0.0
            out = []
            for t in range(q.shape[0]):
                now = max(float(f[t]) + m, float(i[t]))
                keep, write = np.exp(float(f[t]) + m - now), np.exp(float(i[t]) - now)
                S, n, m = keep * S + write * torch.outer(k[t], v[t]), keep * n + write * k[t], now
                out.append((S.T @ q[t]) / (max(abs(float(n @ q[t])), 1.0) + 1e-6))
            return torch.stack(out), (S, n, m)
        monkeypatch.setattr(P, "matrix_memory", memory)
    elif fault == "a state that forgets at a chunk's border":
        def memory(q, k, v, i, f, state=None, inner=P.matrix_memory):
            parts = [inner(q[t:t + 128], k[t:t + 128], v[t:t + 128], i[t:t + 128], f[t:t + 128]) for t in range(0, q.shape[0], 128)]
            return torch.cat([o for o, _ in parts]), parts[-1][1]
        monkeypatch.setattr(P, "matrix_memory", memory)
    elif fault == "gates exchanged":
        wrapped_memory(lambda q, k, v, i, f: (q, k, v, f, i))
    elif fault == "a feed-forward without down's bias":
        inner = P.dense_ff
        monkeypatch.setattr(P, "dense_ff", lambda h, w, p: inner(h, w, p) - w[p + "down.b"])
    elif fault == "a feed-forward without gate's bias":
        inner = P.dense_ff
        monkeypatch.setattr(P, "dense_ff", lambda h, w, p: inner(h, dict(w, **{p + "gate.b": w[p + "gate.b"] * 0}), p))
    else:
        raise AssertionError(fault)


FAULTS = ["the norm in front of the sum", "no factor on the stream", "scores without their cap", "gates without their cap",
          "plain frequencies in attention", "plain frequencies in latent attention", "no magnitude", "the other pairs turned",
          "norms per head", "queries of the memory without their scale", "keys of the memory scaled too", "no divisor",
          "the divisor's floor at one", "a state that forgets at a chunk's border", "gates exchanged",
          "a feed-forward without down's bias", "a feed-forward without gate's bias"]


def test_planted_faults_show(models, monkeypatch):
    """The engine's logits are far (several times the tolerance) from what each mistake would give, and near what the plain
    implementation gives without it: the comparisons of this file would show every one of these.  The read-out's norm hides
    most of a divisor's effect; with an eps that is not small beside the read-outs it shows."""
    cfg = CONFIGS["mixed"]()
    cfg["norm"]["eps"] = 1e-2
    w = P.random_weights(cfg, 77)
    from agave_amd.engine import Engine
    eng = Engine.from_tensors(cfg, {k: v.bfloat16() for k, v in w.items()}, dtype="float32", max_slots=1, max_context=256)
    toks = U.random_tokens(150, cfg["vocab"], 31)
    got = U.run_tail(eng, toks, 40)
    ref = P.forward(cfg, w, toks)
    close(got, (ref, None), "float32", "no fault")
    scale = float(ref.abs().max())
    for fault in FAULTS:
        with monkeypatch.context() as mp:
            planted(mp, fault)
            wrong = P.forward(cfg, w, toks)
        assert float((got.double() - wrong).abs().max()) > 3e-3 * scale, fault
    close(got, (P.forward(cfg, w, toks), None), "float32", "the mistakes are gone again")


# ---------------------------------------------------------------- other sizes
def random_config(seed: int) -> dict:
    """A configuration drawn from a seed: two to six layers of any kind in any order, head counts and sizes that the matrix
    cores take and ones they do not."""
    rng = random.Random(seed)
    layers = []
    for _ in range(rng.randint(2, 6)):
        mlp = None if rng.random() < 0.3 else P.dense(rng.choice([64, 96, 200, 50, 9]))
        base, kind = rng.choice([100.0, 1e4, 1e6]), rng.randrange(3)
        if kind == 0:
            kv = rng.choice([1, 1, 2, 3])
            dim = rng.choice([8, 16, 24, 48, 64, 80, 128, 20, 36])
            layers.append(P.attention_layer(kv * rng.choice([1, 2, 4, 8]), kv, dim, rng.choice([dim, dim, 16, 32, 128, 20]),
                                            rng.choice([dim, dim // 2 // 2 * 2, 2]), base=base, factor=rng.choice([1.0, 2.0, 8.0]),
                                            low=rng.choice([1.0, 2.0]), high=rng.choice([4.0, 6.0]), original=rng.choice([16, 64, 300, 4096]),
                                            scale=rng.choice([dim ** -0.5, 1.7 * dim ** -0.5]), softcap=rng.choice([2.0, 10.0, 50.0]), mlp=mlp))
        elif kind == 1:
            layers.append(P.latent_layer(rng.choice([1, 2, 3, 4, 8, 17]), rng.choice([8, 16, 24, 32, 64, 12, 128]),
                                         rng.choice([2, 8, 16, 32, 64, 6]), rng.choice([16, 32, 48, 128, 20]), rng.choice([8, 24, 64, 30]),
                                         rng.choice([16, 48, 64, 96, 160, 256, 20, 30]), base=base, factor=rng.choice([1.0, 2.0, 16.0]),
                                         fast=rng.choice([32.0, 8.0]), slow=rng.choice([1.0, 2.0]), original=rng.choice([16, 64, 300, 4096]), mlp=mlp))
        else:
            layers.append(P.mlstm_layer(rng.choice([1, 2, 3, 4, 8]), rng.choice([8, 16, 32, 48, 64, 20, 30, 5]), rng.choice([16, 32, 64, 128, 20, 7]),
                                        gate_cap=rng.choice([2.0, 8.0, 15.0]), mlp=mlp))
    return P.config(layers, vocab=rng.choice([97, 256, 1000]), width=rng.choice([64, 96, 128, 160, 320, 72, 100]),
                    eps=rng.choice([1e-6, 1e-5]), alpha=rng.choice([0.5, 1.0, 2.0, 3.7]), embed_scale=rng.choice([0.3, 1.0, 4.0, 11.0]))


@pytest.mark.parametrize("seed", list(range(41, 53)))
def test_configurations_drawn_at_random(seed):
    from agave_amd.engine import Engine
    cfg = random_config(seed)
    w = P.random_weights(cfg, seed)
    toks = U.random_tokens(330, cfg["vocab"], seed)
    others = [U.random_tokens(n, cfg["vocab"], seed + 100 + n) for n in (1, 150)]
    refs = [plain(cfg, w, t, "bfloat16") for t in [toks] + others]
    for dtype in ("float32", "bfloat16"):
        eng = Engine.from_tensors(cfg, {k: v.bfloat16() for k, v in w.items()}, dtype=dtype, max_slots=3, max_context=512)
        close(U.run_tail(eng, toks, 140), refs[0], dtype, f"{cfg}: tail")
        for o, r in zip(U.run_batched(eng, [toks] + others, (300, 1, 100)), refs):
            close(o, r, dtype, f"{cfg}: in a batch")


# ---------------------------------------------------------------- the ways in
@pytest.mark.parametrize("name, dtype", [("mixed", "float32"), ("wide", "float32")])
def test_greedy_generation_through_the_entry_point(models, name, dtype):
    from agave_amd.sampling import SamplingParams
    cfg, w, folder = models(name)
    eng = engine(folder, dtype, max_slots=2, max_context=128)
    prompts = [U.random_tokens(7, cfg["vocab"], 50), U.random_tokens(45, cfg["vocab"], 51), U.random_tokens(1, cfg["vocab"], 52)]
    res = eng.generate(prompts, SamplingParams(temperature=0.0, max_tokens=8))      # three requests, two slots: a slot is used again
    for p, r in zip(prompts, res):
        seq = list(p)
        for _ in range(8):
            seq.append(P.argmax_first(P.forward(cfg, w, seq)[-1]))
        assert list(r.tokens) == seq[len(p):]


def test_decode_steps_replayed_as_graphs_match_eager_ones(models):
    """The recorded decode step, replayed many times with other steps between, against the same steps run eagerly."""
    cfg, w, folder = models("even")
    toks = [U.random_tokens(n, cfg["vocab"], 400 + n) for n in (100, 66)]
    outs = []
    for graphs in (True, False):
        eng = engine(folder, "bfloat16", max_slots=3, max_context=256)
        eng.use_graphs = graphs
        a = U.run_batched(eng, toks, (40, 30))
        U.run_tail(eng, toks[0], 20)                     # a step of another kind between
        b = U.run_batched(eng, toks, (40, 30))
        for x, y in zip(a, b):
            assert torch.equal(x, y)
        outs.append(b)
    for x, y in zip(*outs):
        assert float((x - y).abs().max()) <= 0.02 * float(y.abs().max())


def test_command_line_and_trace_replay(models, tmp_path):
    cfg, w, folder = models("mixed")
    root = U.ROOT
    out = subprocess.run([sys.executable, os.path.join(root, "bin", "agave_amd"), folder, "3 17 5 80 2", "-n", "5", "--dtype", "float32",
                          "--json"], capture_output=True, text=True, timeout=600)
    assert out.returncode == 0, out.stderr[-2000:]
    seq = [3, 17, 5, 80, 2]
    for _ in range(5):
        seq.append(P.argmax_first(P.forward(cfg, w, seq)[-1]))
    got = json.loads(out.stdout.strip().splitlines()[-1])
    assert got["outputs"][0]["tokens"] == seq[5:] and got["outputs"][0]["prompt_tokens"] == 5
    batches = [[U.random_tokens(n, cfg["vocab"], 70 + n) for n in (40, 3, 150)], [U.random_tokens(n, cfg["vocab"], 90 + n) for n in (25, 60)]]
    firsts = [(8, 3, 118), (1, 59)]
    records, where = U.trace_steps_batched(batches, firsts)
    for dtype in ("float32", "bfloat16"):
        steps = U.run_trace_tool(folder, dtype, records, str(tmp_path / dtype), 193, cfg["vocab"])
        for bi, reqs in enumerate(batches):
            for i, r in enumerate(reqs):
                got = torch.from_numpy(np.stack([steps[s][row] for s, row in where[(bi, i)]]))
                close(got, plain(cfg, w, r, dtype), dtype, f"replay {dtype} batch {bi} request {i}")
