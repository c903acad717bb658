"""Dumazen through the serving engine against the plain whole-sequence implementation in
``tests/oracles/dumazen_plain.py``: every mechanism alone, whole prompts against token-by-token decoding,
portions down to two tokens, unequal batches, reused pages and state slots, far keys and the edges of pages, chunks
and windows, the first tokens of a sequence, long decoding, other sizes, and greedy generation through the scheduler.

Each test runs on the CPU path and, marked ``gpu``, on the HIP kernels: fp32 with a tight bound at every position; bf16
with loose bounds on the median and on nine positions in ten and a sanity bound on the rest."""

import math
import random

import pytest
import torch

from tests.models import dumazen_util as U
from tests.oracles import dumazen_plain as plain

DEVICES = [("cpu", torch.float32, 2e-4),
           pytest.param(("cuda", torch.float32, 2e-4), marks=pytest.mark.gpu),
           pytest.param(("cuda", torch.bfloat16, 0.1), marks=pytest.mark.gpu)]
EPS = 1e-6
F64 = torch.float64


@pytest.fixture(params=DEVICES, ids=lambda p: f"{p[0]}-{str(p[1]).split('.')[-1]}")
def dev(request):
    return request.param


def tokens(n, vocab, seed):
    r = random.Random(seed)
    return [r.randrange(vocab) for _ in range(n)]


def check(tmp_path, dev, cfg, requests, steps, seed=0, blocks=64, block_size=4, W=None, max_seqs=4, bf16_tol=None):
    device, dtype, tol = dev
    if bf16_tol is not None and dtype == torch.bfloat16:
        tol = bf16_tol
    W = {k: v.bfloat16().float() for k, v in (W if W is not None else U.random_weights(cfg, seed)).items()}
    eng = U.engine(U.write_checkpoint(tmp_path / "ck", cfg, W), device, dtype, blocks, block_size, max_seqs)
    free0 = eng.kv.num_free_blocks
    got = U.run_schedule(eng, requests, steps)
    assert eng.kv.num_free_blocks == free0 and (eng.kv_cache.slots is None or eng.kv_cache.slots.num_free == max_seqs)
    errs = {rid: U.rel_errs(got[rid], plain.forward(cfg, W, toks)[0].float()) for rid, toks in requests.items()}
    if dtype == torch.bfloat16:
        per = torch.cat(list(errs.values()))
        assert float(per.median()) < tol / 2 and float(per.quantile(0.9)) < 2 * tol and float(per.max()) < 1.0, per
    else:
        for rid, per in errs.items():
            assert float(per.max()) < tol, f"{rid}: {per.max()} at {int(per.argmax())}"
    eng.close()


def whole(requests):
    return [[(rid, len(t))] for rid, t in requests.items()]


FULL = [(U.par(), U.dense()), (U.ssm(), None), (U.ret(), U.dense(9)),
        (U.par(U.left(heads=3, kv_heads=1, dim=6, vdim=9, window=11, dims=4), U.right(heads=4, kv_heads=2, dim=5, vdim=7, conv=2)), None),
        (U.ssm(heads=2, vdim=9, state=4, groups=1, conv=4, norm_groups=1), U.dense(7)), (U.ret(heads=2, dim=5, vdim=8, dims=2), None)]


# ------------------------------------------------------------------ each mechanism alone
def test_attention_alone(tmp_path, dev):
    cfg = U.config([(U.par(right_scale=0.0), None)])
    r = {"a": tokens(29, 50, 1)}
    check(tmp_path, dev, cfg, r, whole(r))


@pytest.mark.parametrize("sizes", [dict(heads=3, kv_heads=3, dim=10, vdim=4, window=1), dict(heads=6, kv_heads=1, dim=4, vdim=8, window=3, dims=2),
                                   dict(heads=1, kv_heads=1, dim=2, vdim=3, window=200), dict(heads=4, kv_heads=2, dim=8, vdim=16, window=26, scaling=None),
                                   dict(heads=2, kv_heads=2, dim=7, vdim=33, window=16, dims=6), dict(heads=4, kv_heads=4, dim=12, vdim=12, window=5, dims=0),
                                   dict(heads=8, kv_heads=2, dim=16, vdim=8, window=9, dims=8, scale=1.0)])
def test_attention_sizes(tmp_path, dev, sizes):
    # as many kv heads as heads, one kv head, one head, a window of one key, one as long as and one longer than the
    # sequence, key and value sizes that differ, part of a head turned, none of it, no frequency scaling
    cfg = U.config([(U.par(U.left(**sizes), right_scale=0.0), None)])
    r = {"a": tokens(26, 50, 2)}
    check(tmp_path, dev, cfg, r, [[("a", 9)], [("a", 1)], [("a", 16)]])


def test_norms_run_over_all_heads_together(tmp_path, dev):
    # one query head and one key head are 30 times larger than the others: a norm head by head would level them
    cfg = U.config([(U.par(U.left(heads=4, kv_heads=2, dim=8), right_scale=0.0), None)])
    W = U.random_weights(cfg, 3)
    for n, d in (("q", 8), ("k", 8)):
        W[f"l0.mix.left.{n}"][:d] *= 30.0
        W[f"l0.mix.left.{n}.b"][:d] *= 30.0
    r = {"a": tokens(24, 50, 3)}
    check(tmp_path, dev, cfg, r, [[("a", 11)], [("a", 1)], [("a", 12)]], W=W)


def test_biases_are_in_the_projection(tmp_path, dev):
    # all embeddings zero: only the biases speak (before the norms, so their size does not matter but their direction does)
    cfg = U.config([(U.par(U.left(dims=0), right_scale=0.0), U.dense())])
    W = U.random_weights(cfg, 4)
    W["embed"] *= 0.01
    for n in ("q.b", "k.b", "v.b"):
        W["l0.mix.left." + n] *= 3.0
    r = {"a": tokens(12, 50, 4)}
    check(tmp_path, dev, cfg, r, whole(r), W=W)


@pytest.mark.parametrize("base,dims,scaling", [(250000.0, 56, {"factor": 16.0, "low": 1.5, "high": 5.0, "original": 2048}), (10000.0, 32, None),
                                               (300.0, 16, U.SCALING), (50.0, 10, {"factor": 2.0, "low": 0.7, "high": 8.0, "original": 100}),
                                               (1000.0, 24, {"factor": 3.0, "low": 2.0, "high": 2.5, "original": 700})])
def test_frequencies(base, dims, scaling):
    # wavelengths on both sides of both borders and between them
    from llmctl.models.mixers import rotary_frequencies

    want = plain.frequencies({"base": base, "dims": dims, "scaling": scaling})
    got, amp = rotary_frequencies(base, dims, scaling)
    assert amp == 1.0 and got.dtype == torch.float32
    assert torch.allclose(got.double(), torch.tensor(want, dtype=F64), rtol=1e-6, atol=0.0)
    if scaling:
        plain_f = plain.frequencies({"base": base, "dims": dims})
        ratio = [a / b for a, b in zip(want, plain_f)]
        assert max(ratio) == 1.0 and abs(min(ratio) - 1.0 / scaling["factor"]) < 1e-9


def test_delta_rule_alone(tmp_path, dev):
    cfg = U.config([(U.par(left_scale=0.0), None)])
    r = {"a": tokens(27, 50, 5)}
    check(tmp_path, dev, cfg, r, whole(r))


@pytest.mark.parametrize("sizes", [dict(heads=1, kv_heads=1, dim=1, vdim=1, conv=1), dict(heads=4, kv_heads=2, dim=16, vdim=8, conv=2),
                                   dict(heads=6, kv_heads=1, dim=20, vdim=33, conv=3), dict(heads=2, kv_heads=2, dim=40, vdim=16, conv=6),
                                   dict(heads=3, kv_heads=3, dim=7, vdim=70, conv=4)])
def test_delta_rule_sizes(tmp_path, dev, sizes):
    cfg = U.config([(U.par(U.left(), U.right(**sizes), left_scale=0.0), None)])
    r = {"a": tokens(90, 50, 6), "b": tokens(4, 50, 7)}
    check(tmp_path, dev, cfg, r, [[("a", 70), ("b", 2)], [("a", 1), ("b", 1)], [("a", 19), ("b", 1)]], bf16_tol=0.2 if sizes["dim"] == 1 else None)


@pytest.mark.parametrize("left_scale,right_scale", [(1.0, 1.0), (0.2, 0.9), (-0.5, 0.3)])
def test_both_sides_of_the_pair(tmp_path, dev, left_scale, right_scale):
    cfg = U.config([(U.par(left_scale=left_scale, right_scale=right_scale), U.dense())])
    r = {"a": tokens(31, 50, 8)}
    check(tmp_path, dev, cfg, r, [[("a", 13)], [("a", 1)], [("a", 17)]])


def test_mamba2_alone(tmp_path, dev):
    cfg = U.config([(U.ssm(), None)])
    r = {"a": tokens(27, 50, 9)}
    check(tmp_path, dev, cfg, r, whole(r))


@pytest.mark.parametrize("sizes", [dict(heads=1, vdim=1, state=1, groups=1, conv=1, norm_groups=1), dict(heads=6, vdim=4, state=16, groups=3, conv=2, norm_groups=6),
                                   dict(heads=4, vdim=8, state=12, groups=4, conv=4, norm_groups=2), dict(heads=2, vdim=35, state=40, groups=1, conv=7, norm_groups=1),
                                   dict(heads=3, vdim=10, state=5, groups=1, conv=3, norm_groups=5)])
def test_mamba2_sizes(tmp_path, dev, sizes):
    # one of everything, a group per head, norm groups that are single heads and that split heads, one tap (no carried inputs)
    # and seven
    one = sizes["heads"] * sizes["vdim"] == 1
    cfg = U.config([(U.ssm(**sizes), None)], eps=0.05 if one else EPS)  # (a norm over one number is a sign, were eps small)
    r = {"a": tokens(90, 50, 10), "b": tokens(4, 50, 11)}
    check(tmp_path, dev, cfg, r, [[("a", 70), ("b", 2)], [("a", 1), ("b", 1)], [("a", 19), ("b", 1)]])


def test_gate_ahead_of_the_grouped_norm(tmp_path, dev):
    # gates that differ by orders of magnitude between the norm's groups and inside them
    cfg = U.config([(U.ssm(norm_groups=2), None)])
    W = U.random_weights(cfg, 12)
    inner = 24
    W["l0.mix.in"][:inner // 2] *= 6.0
    W["l0.mix.in"][inner // 4:inner // 2] *= 0.1
    r = {"a": tokens(24, 50, 12)}
    check(tmp_path, dev, cfg, r, [[("a", 11)], [("a", 1)], [("a", 12)]], W=W)


def test_steps_without_a_clamp(tmp_path, dev):
    # step sizes from nearly nothing to far above one, decays from nearly one to nearly zero
    cfg = U.config([(U.ssm(heads=4), None), (U.par(left_scale=0.0), None)])
    W = U.random_weights(cfg, 13)
    W["l0.mix.dt_bias"] = torch.tensor([-9.0, 0.0, 6.0, 12.0])
    W["l0.mix.A_log"] = torch.tensor([2.0, -3.0, -4.0, 1.0])
    W["l1.mix.right.dt_bias"] = torch.tensor([-7.0, 3.0, 25.0])
    W["l1.mix.right.A_log"] = torch.tensor([1.0, -4.0, 0.0])
    r = {"a": tokens(100, 50, 13)}
    check(tmp_path, dev, cfg, r, [[("a", 80)], [("a", 1)], [("a", 19)]], W=W)


def test_retention_alone(tmp_path, dev):
    cfg = U.config([(U.ret(), None)])
    r = {"a": tokens(27, 50, 14)}
    check(tmp_path, dev, cfg, r, whole(r))


@pytest.mark.parametrize("sizes", [dict(heads=1, dim=2, vdim=1, decay=[0.7]), dict(heads=4, dim=16, vdim=8, dims=8, decay=[1.0, 0.999, 0.03, 0.5]),
                                   dict(heads=2, dim=21, vdim=40, dims=0, decay=[0.9, 0.99]), dict(heads=3, dim=36, vdim=20, decay=[0.96, 0.98, 0.99])])
def test_retention_sizes(tmp_path, dev, sizes):
    # part of a head turned, none of it, no decay at all, a memory of hardly one token
    cfg = U.config([(U.ret(**sizes), None)], eps=0.05 if sizes["vdim"] == 1 else EPS)
    r = {"a": tokens(90, 50, 15), "b": tokens(4, 50, 16)}
    check(tmp_path, dev, cfg, r, [[("a", 70), ("b", 2)], [("a", 1), ("b", 1)], [("a", 19), ("b", 1)]])


@pytest.mark.parametrize("ff,mult,eps", [(1, 1.0, 1e-6), (40, 0.3, 1e-3), (64, 2.0, 1e-5)])
def test_feed_forward_and_residual(tmp_path, dev, ff, mult, eps):
    cfg = U.config([(U.ret(), U.dense(ff)), (U.ssm(), U.dense(ff + 3))], mult=mult, eps=eps)
    r = {"a": tokens(30, 50, 17), "b": tokens(9, 50, 18)}
    check(tmp_path, dev, cfg, r, [[("a", 30), ("b", 2)], [("b", 1)], [("b", 6)]])


def test_norms_stored_around_zero(tmp_path, dev):
    # weights near -1 shut a coordinate's update off, large ones blow it up; the stream itself is not normed on the way in
    cfg = U.config([(U.ret(), U.dense()), (U.ssm(), None)])
    W = U.random_weights(cfg, 19)
    W["embed"] *= 4.0
    W["l0.norm1"][:8], W["l0.norm2"][4:12], W["final.norm"][:3] = -1.0, 3.0, -1.0
    r = {"a": tokens(20, 50, 19)}
    check(tmp_path, dev, cfg, r, [[("a", 9)], [("a", 1)], [("a", 10)]], W=W)


def test_stream_after_every_layer(tmp_path):
    from llmctl.serve.scheduler import PrefillChunk

    cfg = U.config(FULL)
    W = {k: v.bfloat16().float() for k, v in U.random_weights(cfg, 20).items()}
    eng = U.engine(U.write_checkpoint(tmp_path / "ck", cfg, W), "cpu")
    toks = tokens(15, 50, 20)
    seq = eng.open_sequence(toks)
    trail = []
    eng.forward_portions([PrefillChunk(seq, 0, len(toks))], [[0]], trail=trail)
    want = plain.forward(cfg, W, toks)[1]
    assert len(trail) == len(want) == len(FULL)
    for a, b in zip(trail, want):
        assert float((a.double() - b).abs().max()) < 1e-4 * float(b.abs().max())


def test_no_layers(tmp_path, dev):
    cfg = U.config([])
    r = {"a": tokens(5, 50, 21)}
    check(tmp_path, dev, cfg, r, whole(r))


# ------------------------------------------------------------------ schedules
def test_prefill_against_token_by_token(tmp_path, dev):
    cfg = U.config(FULL)
    r = {"a": tokens(26, 50, 22)}
    check(tmp_path, dev, cfg, r, [[("a", 1)]] * 26)


def test_portions_of_several_sizes(tmp_path, dev):
    cfg = U.config(FULL)
    r = {"a": tokens(61, 50, 23)}
    check(tmp_path, dev, cfg, r, [[("a", n)] for n in (2, 17, 3, 2, 30, 1, 1, 5)])


def test_portions_around_the_chunk(tmp_path, dev):
    # portions of one chunk of the scan less one, one chunk, one more, two of them and one more
    cfg = U.config([(U.par(U.left(), U.right(dim=16, vdim=20)), None), (U.ssm(state=16), None), (U.ret(dim=12), None)])
    r = {"a": tokens(63 + 64 + 65 + 128 + 129, 50, 24), "b": tokens(64, 50, 25)}
    check(tmp_path, dev, cfg, r, [[("a", 63)], [("a", 64), ("b", 63)], [("a", 65), ("b", 1)], [("a", 128)], [("a", 129)]], blocks=160)


def test_unequal_batches(tmp_path, dev):
    cfg = U.config(FULL)
    r = {"a": tokens(40, 50, 26), "b": tokens(7, 50, 27), "c": tokens(19, 50, 28), "d": tokens(2, 50, 29)}
    steps = [[("a", 11), ("b", 2)], [("a", 1), ("b", 4), ("c", 9)], [("c", 1), ("a", 20), ("b", 1), ("d", 2)], [("a", 8), ("c", 9)]]
    check(tmp_path, dev, cfg, r, steps)


def test_long_portion_beside_short_ones_and_decoded_rows(tmp_path, dev):
    # one step with a portion of several chunks, one of a few tokens, one of a single first token and two decoded rows
    cfg = U.config(FULL)
    r = {"a": tokens(210, 50, 30), "b": tokens(14, 50, 31), "c": tokens(9, 50, 32), "d": tokens(3, 50, 33)}
    steps = [[("b", 5), ("c", 7)], [("a", 200), ("b", 1), ("c", 1), ("d", 1)], [("d", 2), ("a", 10), ("b", 8), ("c", 1)]]
    check(tmp_path, dev, cfg, r, steps, blocks=80)


def test_pages_and_slots_used_again(tmp_path, dev):
    # 12 pages of 4 tokens and 2 state slots for five requests: every later request runs in pages and a slot that hold
    # an earlier one's rows, memories and carried inputs
    cfg = U.config(FULL)
    r = {k: tokens(n, 50, 34 + i) for i, (k, n) in enumerate([("a", 22), ("b", 18), ("c", 20), ("d", 9), ("e", 23)])}
    steps = [[("a", 10), ("b", 18)], [("a", 12), ("c", 3)], [("c", 17), ("d", 1)], [("d", 1)], [("d", 7), ("e", 2)], [("e", 21)]]
    check(tmp_path, dev, cfg, r, steps, blocks=12, max_seqs=2)


def test_token_by_token_start_in_a_used_slot(tmp_path, dev):
    # fewer tokens than taps lie behind the first decoded ones: what the slot held before must not enter
    cfg = U.config([(U.par(), None), (U.ssm(conv=5), U.dense())])
    r = {"a": tokens(30, 50, 40), "b": tokens(12, 50, 41)}
    check(tmp_path, dev, cfg, r, [[("a", 30)]] + [[("b", 1)]] * 12, blocks=10, max_seqs=1)


def test_two_token_portions_from_the_start(tmp_path, dev):
    cfg = U.config(FULL)
    r = {"a": tokens(30, 50, 42), "b": tokens(24, 50, 43)}
    check(tmp_path, dev, cfg, r, [[("a", 30)]] + [[("b", 2)]] * 12, blocks=10, max_seqs=1)


def test_long_decoding_over_window_and_tile_borders(tmp_path, dev):
    # 150 decoded tokens after a short prompt: the window (37) passes over decoded tokens, contexts cross 64-key tiles and
    # many pages, the memories carry on for long
    cfg = U.config([(U.par(U.left(window=37, heads=2, kv_heads=1, dim=8, vdim=16)), None), (U.ssm(), U.dense()), (U.ret(), None),
                    (U.par(U.left(window=66)), None)])
    r = {"a": tokens(156, 50, 44)}
    check(tmp_path, dev, cfg, r, [[("a", 6)]] + [[("a", 1)]] * 150, blocks=48)


def test_long_portions(tmp_path, dev):
    # 650-token portions (many chunks, several query blocks) continued in a second and a third step, beside others
    cfg = U.config([(U.par(U.left(window=70), U.right(dim=16, vdim=16)), None), (U.ssm(state=20), None), (U.ret(), U.dense(8))])
    r = {"a": tokens(700, 50, 45), "b": tokens(300, 50, 46)}
    check(tmp_path, dev, cfg, r, [[("a", 650), ("b", 10)], [("a", 49), ("b", 290)], [("a", 1)]], blocks=260)


def test_heads_that_fit_the_matrix_cores(tmp_path, dev):
    # head sizes in multiples of 8 (the bf16 runs take the matrix-core form of the attention), a prompt over several 64-key
    # tiles, windows of 70 and 130 keys, then decoding, beside a short request; values of more than four column tiles
    cfg = U.config([(U.par(U.left(heads=4, kv_heads=2, dim=32, vdim=48, window=70), U.right(heads=2, kv_heads=1, dim=32, vdim=96)), None),
                    (U.ssm(heads=3, vdim=80, state=32, groups=1, norm_groups=1), U.dense(32)),
                    (U.par(U.left(heads=4, kv_heads=1, dim=24, vdim=80, window=130), U.right(heads=2, kv_heads=2, dim=64, vdim=64)), None),
                    (U.ret(heads=2, dim=48, vdim=144), None)], width=64)
    r = {"a": tokens(230, 50, 47), "b": tokens(9, 50, 48)}
    check(tmp_path, dev, cfg, r, [[("a", 200), ("b", 4)]] + [[("a", 1), ("b", 1)]] * 5 + [[("a", 25)]], blocks=80)


@pytest.mark.parametrize("seed", range(10))
def test_random_configurations(tmp_path, dev, seed):
    # sizes, layer order, windows, constants and schedules drawn at random (some sizes fit the vector and matrix-core
    # forms, some do not)
    r = random.Random(700 + seed)
    step = r.choice([1, 4, 8])
    size = lambda lo, hi: max(1, r.randint(lo, hi) // step) * step
    layers = []
    for _ in range(r.randint(2, 5)):
        kind = r.choice(["par", "ssm", "ret"])
        if kind == "par":
            G, K, dim = r.choice([1, 2, 3]), r.choice([1, 2]), size(4, 40)
            m = U.par(U.left(heads=G * r.choice([1, 2, 3]), kv_heads=G, dim=dim, vdim=size(4, 72), window=r.randint(1, 90),
                             base=r.choice([100.0, 10000.0]), dims=r.choice([dim // 2 * 2, dim // 4 * 2]), scaling=r.choice([None, U.SCALING])),
                      U.right(heads=K * r.choice([1, 3]), kv_heads=K, dim=size(4, 70), vdim=size(4, 80), conv=r.choice([2, 3, 4, 5])),
                      r.choice([0.3, 1.0]), r.choice([0.5, 0.8]))
        elif kind == "ssm":
            G, K = r.choice([1, 2]), r.choice([1, 2, 3])
            H = G * K
            m = U.ssm(heads=H, vdim=size(4, 60), state=size(4, 70), groups=G, conv=r.choice([1, 2, 3, 4]), norm_groups=r.choice([1, H]))
        else:
            H, dim = r.choice([1, 2, 4]), size(4, 60)
            m = U.ret(heads=H, dim=dim, vdim=size(4, 90), dims=r.choice([dim // 2 * 2, dim // 4 * 2]),
                      decay=[r.choice([0.5, 0.95, 0.99, 0.999, 1.0]) for _ in range(H)])
        layers.append((m, r.choice([None, U.dense(size(4, 60))])))
    cfg = U.config(layers, width=r.choice([12, 16, 33, 40, 72]), vocab=r.choice([37, 64, 101]), eps=r.choice([1e-6, 1e-4]), mult=r.choice([0.2, 0.5, 1.0]))
    reqs = {k: tokens(r.randint(3, 200), cfg["vocab"], 701 + i) for i, k in enumerate("abc")}
    left, steps = {k: len(t) for k, t in reqs.items()}, []
    while any(left.values()):
        entries = []
        for k in list(left):
            if left[k] and r.random() < 0.7:
                n = min(left[k], r.choice([1, 1, 2, 3, 17, 64, 90, 150]))
                entries.append((k, n))
                left[k] -= n
        if entries:
            steps.append(entries)
    check(tmp_path, dev, cfg, reqs, steps, seed=seed, blocks=48, block_size=16, bf16_tol=0.2)


# ------------------------------------------------------------------ far keys and edges
def _standing_out(cfg, special, seed):
    """Weights with which token ``special`` draws every later query that sees it: its embedding alone has coordinate 0, its key
    and value come from there, all queries point along that key."""
    m = cfg["layers"][0]["mixer"]["left"]
    H, G, d, dv = m["heads"], m["kv_heads"], m["dim"], m["vdim"]
    W = U.random_weights(cfg, seed)
    g = torch.Generator().manual_seed(seed)
    u = torch.randn(d, generator=g)
    W["embed"][:, 0] = 0.0
    W["embed"][special, 0] = 8.0
    p = "l0.mix.left."
    W[p + "q"] *= 0.2
    W[p + "k"] *= 0.5
    W[p + "q.b"] = u.repeat(H) * 2.0
    W[p + "k.b"] *= 0.1
    W[p + "k"][:, 0] = u.repeat(G)
    W[p + "v"][:, 0] = torch.randn(G * dv, generator=g) * 2.0
    for n in ("q.norm", "k.norm"):
        W[p + n] = torch.ones_like(W[p + n])
    return {k: v.bfloat16().float() for k, v in W.items()}


EDGES = [(4, 60, 44, 9), (8, 200, 2, 300), (16, 200, 63, 100), (16, 200, 64, 100), (16, 330, 127, 140), (16, 330, 128, 140), (4, 90, 31, 33), (16, 70, 0, 64),
         (16, 70, 0, 5), (8, 140, 70, 1)]


@pytest.mark.parametrize("bs,L,j0,window", EDGES)
def test_far_keys_and_window_edges(tmp_path, dev, bs, L, j0, window):
    # the standing-out key lies far back, and the queries pass from just inside to just outside its window, in a prompt's
    # portion and in decoding; on either side of page and 64-key-tile borders
    device, dtype, tol = dev
    cfg = U.config([(U.par(U.left(heads=4, kv_heads=2, dim=16, vdim=8, window=window, dims=0, scale=1.5), right_scale=0.0), None)], width=24)
    special = 7
    W = _standing_out(cfg, special, 100 + j0)
    toks = [t if t != special else 8 for t in tokens(L, 50, 60)]
    toks[j0] = special
    want = plain.forward(cfg, W, toks)[0].float()
    edge = j0 + window  # the first query that no longer sees it
    if edge < L:  # the oracle with a window one token off must differ there, or the test would hide the fault
        for off in (-1, 1):
            other = dict(cfg, layers=[dict(cfg["layers"][0], mixer=dict(cfg["layers"][0]["mixer"], left=dict(cfg["layers"][0]["mixer"]["left"], mask={"size": window + off})))])
            if window + off >= 1:
                d = U.rel_errs(plain.forward(other, W, toks)[0].float(), want)
                assert float(d[edge - 1 if off < 0 else edge]) > 0.3
    path = U.write_checkpoint(tmp_path / "ck", cfg, W)
    dec = min(L - 2, max(12, L - edge + 6)) if edge < L else 12  # decode over the edge
    for steps in ([[("a", L)]], [[("a", L - min(dec, 80))]] + [[("a", 1)]] * min(dec, 80)):
        eng = U.engine(path, device, dtype, blocks=(L + bs - 1) // bs + 2, block_size=bs)
        err = U.rel_errs(U.run_schedule(eng, {"a": toks}, steps)["a"], want)
        assert float(err.max()) < tol, (len(steps), int(err.argmax()), float(err.max()))
        eng.close()


# ------------------------------------------------------------------ ops
def _batch(parts, device):
    """A StepBatch's sequence part for portions [(length, first position, slot)], prompt portions first."""
    from llmctl.models.mixers import StepBatch

    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=device)
    cu = [0]
    for n, _, _ in parts:
        cu.append(cu[-1] + n)
    pre = [c for c in parts if c[0] > 1 or c[1] == 0]
    Tp = sum(c[0] for c in pre)
    assert parts[:len(pre)] == pre
    seq_of = [i for i, (n, _, _) in enumerate(parts) for _ in range(n)]
    return StepBatch(ids=None, pos=None, slots=None, Tp=Tp, p_cu=None, p_ctx=i32([c[0] + c[1] for c in pre]) if pre else None, p_bt=None,
                     d_ctx=None, d_bt=None, cu=i32(cu), start=i32([c[1] for c in parts]), state=i32([c[2] for c in parts]),
                     max_q=max((c[0] for c in pre), default=0), cu_host=cu, seq_of=i32(seq_of))


def _memory_case(dev, kind, steps, H, KH, dk, dv, seed, edit=None, qk32=None):
    """Runs ``steps`` (lists of portions, every sequence from its slot) through the scan and through the oracle; returns the
    largest output and memory errors relative to the largest wanted entries."""
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(seed)
    nslots = 1 + max(s for st in steps for _, _, s in st)
    pool = torch.randn(nslots, H, dk, dv, generator=g)
    state = {s: pool[s].double() for s in range(nslots)}
    pool = pool.to(device)
    par = dict(a_log=torch.randn(H, generator=g) * 0.5 - 1.0, dt_bias=torch.randn(H, generator=g) - 2.0, log_decay=torch.log(torch.rand(H, generator=g) * 0.3 + 0.7),
               skip=torch.randn(H, generator=g))
    worst_o = worst_s = 0.0
    for st in steps:
        T = sum(n for n, _, _ in st)
        q, k = torch.randn(T, KH, dk, generator=g), torch.randn(T, KH, dk, generator=g)
        if kind == "delta":
            q, k = plain.unit(q), plain.unit(k)
        else:
            k = k * dk ** -0.5
        v, ga, gb = torch.randn(T, H, dv, generator=g), torch.randn(T, H + 3, generator=g), torch.randn(T, H, generator=g) * 2.0
        if edit is not None:
            edit(q, k, v, ga, gb, par)
        qd = dtype if (kind == "ssm" and not qk32) else torch.float32
        q, k, v, ga, gb = q.to(qd), k.to(qd), v.to(dtype), ga.to(dtype), gb.to(dtype)
        if kind == "fixed":
            la, beta = par["log_decay"].double()[None].expand(T, H), torch.ones(T, H, dtype=F64)
        else:
            dt = plain.softplus(ga[:, 1:H + 1].double() + par["dt_bias"].double())
            la = -torch.exp(par["a_log"].double()) * dt
            beta = dt if kind == "ssm" else plain.sigmoid(gb.double())
        want, at = torch.zeros(T, H, dv, dtype=F64), 0
        for n, p, s in st:
            if p == 0:
                state[s] = torch.zeros(H, dk, dv, dtype=F64)
            new = []
            for h in range(H):
                kh = h // (H // KH)
                fn = plain.delta_memory if kind == "delta" else plain.decayed_memory
                o, S = fn(q[at:at + n, kh].double(), k[at:at + n, kh].double(), v[at:at + n, h].double(), torch.exp(la[at:at + n, h]), beta[at:at + n, h], state[s][h])
                want[at:at + n, h] = o + (par["skip"][h].double() * v[at:at + n, h].double() if kind == "ssm" else 0.0)
                new.append(S)
            state[s], at = torch.stack(new), at + n
        # operands as columns of wider rows
        wide = lambda x: torch.cat([x, torch.full_like(x[:, :1], 9.0)], 1).to(device)[:, :x.shape[1]]
        kw = {n: par[n].to(device) for n in {"fixed": ["log_decay"], "ssm": ["a_log", "dt_bias", "skip"], "delta": ["a_log", "dt_bias"]}[kind]}
        if kind != "fixed":
            kw["ga"] = ga.to(device)[:, 1:H + 1]
        if kind == "delta":
            kw["gb"] = gb.to(device)
        gate, w = torch.randn(T, H * dv, generator=g).to(dtype), torch.randn(H * dv, generator=g)
        eps = float((0.01 * want.abs().max()) ** 2)  # (rows far below the largest ones would show the fp32 rounding of those)
        for weight in (None, w):  # the same with the head norm, on a copy of the memories
            y = hybrid.memory_scan(wide(q), wide(k), wide(v), kind, pool.clone(), _batch(st, device), **kw,
                                   norm=(weight.to(device) if weight is not None else None, wide(gate), eps))
            ref = plain.rms(want, eps).reshape(T, -1) * plain.silu(gate.double()) * (weight.double() if weight is not None else 1.0)
            assert y.dtype == dtype and float((y.double().cpu() - ref).abs().max() / ref.abs().max()) < (1e-3 if dtype == torch.float32 else 1e-2)
        got = hybrid.memory_scan(wide(q), wide(k), wide(v), kind, pool, _batch(st, device), **kw).double().cpu()
        assert bool(torch.isfinite(got).all()) and bool(torch.isfinite(pool.cpu()).all())
        worst_o = max(worst_o, float((got - want).abs().max() / want.abs().max()))
        for _, _, s in st:
            worst_s = max(worst_s, float((pool[s].double().cpu() - state[s]).abs().max() / state[s].abs().max().clamp(min=1e-3)))
    return worst_o, worst_s


@pytest.mark.parametrize("kind", ["fixed", "ssm", "delta"])
@pytest.mark.parametrize("H,KH,dk,dv", [(1, 1, 1, 1), (4, 2, 16, 16), (3, 1, 20, 36), (2, 2, 48, 64), (6, 3, 7, 9), (2, 1, 64, 128), (1, 1, 130, 20), (2, 1, 96, 150), (1, 1, 256, 40)])
def test_memory_scan_sizes(dev, kind, H, KH, dk, dv):
    # the scan over whole portions, portions of several chunks and decoded rows, in steps that begin, continue and mix
    # sequences; slots hold junk at first
    long = 150 if dk * dv < 6000 else 80
    steps = [[(long, 0, 2), (3, 0, 0)], [(30, 3, 0), (2, 0, 1), (1, long, 2)], [(1, 33, 0), (1, 2, 1), (1, long + 1, 2)], [(64, long + 2, 2), (17, 3, 1)],
             [(66, 0, 1), (1, long + 66, 2)]]
    o, s = _memory_case(dev, kind, steps, H, KH, dk, dv, 10 * dk + dv)
    assert o < 2e-5 and s < 2e-5, (o, s)


@pytest.mark.parametrize("kind", ["fixed", "ssm", "delta"])
@pytest.mark.parametrize("T,cuts,far", [(40, [40], 2), (64, [64], 0), (300, [7, 1, 1, 290, 1], 5), (700, [257, 443], 3), (130, [64, 64, 2], 63), (200, [129, 1, 70], 64)])
def test_memory_lasts_and_fades(dev, kind, T, cuts, far):
    # head 0 hardly decays and one token writes along a key that nothing else touches: the last token reads it back; head 1
    # forgets within a token or two.  A lost memory at any border of the schedule would show in full
    def edit(q, k, v, ga, gb, par):
        par["a_log"][:], par["dt_bias"][:], par["skip"][:] = torch.tensor([-14.0, 4.0]), torch.tensor([1.0, 2.0]), 0.0
        par["log_decay"][:] = torch.log(torch.tensor([1.0, 0.01]))
        ga.zero_(), gb.fill_(3.0)
        n = edit.at
        q[:, :, 0], k[:, :, 0] = 0.0, 0.0
        m = q.shape[0]
        if n <= far < n + m:
            k[far - n] = 0.0
            k[far - n, :, 0] = 1.0
            v[far - n] = 5.0
        if n + m == T:
            q[-1] = 0.0
            q[-1, :, 0] = 1.0
        edit.at += m

    edit.at = 0
    steps, at = [], 0
    for n in cuts:
        steps.append([(n, at, 1)])
        at += n
    o, s = _memory_case(dev, kind, steps, 2, 1, 12, 10, T + far, edit)
    assert o < 2e-5 and s < 2e-5, (o, s)


def test_delta_rule_with_keys_alike(dev):
    # nearly equal keys and full write strength: every token takes off what the one before it wrote, and the chunk's solve
    # has large entries below its diagonal
    def edit(q, k, v, ga, gb, par):
        base = torch.randn(k.shape[-1], generator=torch.Generator().manual_seed(3))
        k.copy_(plain.unit(base + 0.05 * k))
        gb.fill_(8.0)
        par["dt_bias"].fill_(-9.0)

    o, s = _memory_case(dev, "delta", [[(200, 0, 0)], [(40, 200, 0)], [(1, 240, 0)]], 2, 2, 32, 24, 77, edit)
    assert o < 1e-4 and s < 1e-4, (o, s)


@pytest.mark.parametrize("kind", ["ssm", "delta"])
def test_strong_and_weak_decay_in_one_chunk(dev, kind):
    # sums of logarithms of the decay in the thousands beside steps of almost no decay: differences of the sums stay exact
    def edit(q, k, v, ga, gb, par):
        par["a_log"].fill_(0.0), par["dt_bias"].fill_(0.0)
        ga.fill_(-7.0)
        ga[::9] = 160.0
        ga[1::9] = 0.5
        if kind == "ssm":
            v[::9] *= 0.01

    o, s = _memory_case(dev, kind, [[(200, 0, 0)], [(50, 200, 0)]], 2, 1, 16, 24, 5, edit)
    assert o < 2e-5 and s < 2e-5, (o, s)


@pytest.mark.parametrize("C,nq,nk,dk,taps,bias", [(24, 1, 1, 8, 4, False), (40, 0, 0, 0, 3, True), (30, 2, 1, 6, 2, False), (33, 1, 1, 5, 4, True), (700, 3, 3, 64, 4, False),
                                                  (600, 1, 1, 256, 3, True), (23, 2, 2, 5, 7, False), (520, 1, 1, 130, 2, False), (64, 1, 2, 12, 1, True), (1032, 0, 0, 0, 4, True)])
def test_convolution_with_unit_groups(dev, C, nq, nk, dk, taps, bias):
    # three steps that begin, continue and mix sequences (long portions, short ones, decoded rows), junk in the slots
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(C + taps)
    w, bs = torch.randn(C, taps, generator=g) * 0.6, torch.randn(C, generator=g) * 0.3 if bias else None
    state = torch.randn(5, taps - 1, C, generator=g).to(device)
    hist = {}
    n0 = (nq + nk) * dk
    for parts in ([(90, 0, 2), (3, 0, 0), (33, 0, 1)], [(2, 3, 0), (40, 0, 4), (1, 90, 2), (1, 33, 1)], [(1, 5, 0), (1, 40, 4), (1, 91, 2)], [(3, 41, 4), (2, 0, 3), (1, 6, 0)]):
        T = sum(p[0] for p in parts)
        wide = torch.randn(T, C + 8, generator=g).to(dtype)
        u = wide[:, :C]
        want, at = torch.zeros(T, C, dtype=F64), 0
        for n, p, s in parts:
            ext = u[at:at + n].double() if p == 0 else torch.cat([hist[s], u[at:at + n].double()])
            want[at:at + n] = plain.silu(plain.conv(ext, w.double(), bs.double() if bias else None))[-n:]
            hist[s], at = ext, at + n
        qk, y = hybrid.conv_silu_unit(wide.to(device)[:, :C], w.t().contiguous().to(device), bs.to(device) if bias else None, state, _batch(parts, device),
                                      nq, nk, dk, 0.37, 1e-6)
        tol = 1e-5 if dtype == torch.float32 else 1e-2
        assert y.dtype == dtype and float((y.double().cpu() - want[:, n0:]).abs().max()) < tol * float(want.abs().max())
        if n0:
            x = plain.unit(want[:, :n0].view(T, nq + nk, dk))
            x[:, :nq] *= 0.37
            assert qk.dtype == torch.float32 and float((qk.double().cpu() - x).abs().max()) < (1e-5 if dtype == torch.float32 or device == "cuda" else 1e-2)
        for n, p, s in parts:
            tail = hist[s][-(taps - 1):] if taps > 1 else hist[s][:0]
            m = tail.shape[0]
            assert m == 0 or float((state[s, taps - 1 - m:].double().cpu() - tail).abs().max()) < 1e-6


@pytest.mark.parametrize("nq,nk,dk,dims", [(2, 2, 8, 8), (3, 1, 10, 4), (1, 1, 7, 6), (4, 4, 64, 32), (2, 3, 12, 0), (1, 2, 6, 2)])
def test_rotary_for_the_recurrence(dev, nq, nk, dk, dims):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(dk)
    T, rot = 40, {"base": 77.0, "dims": dims}
    z = torch.randn(T, (nq + nk) * dk + 4, generator=g).to(dtype)
    freq = torch.tensor(plain.frequencies(rot), dtype=torch.float32)
    pos = torch.arange(T, dtype=torch.int32)
    for inter in (False, True):
        got = hybrid.rotary_f32(z.to(device), nq, nk, dk, pos.to(device), freq.to(device), dims, inter, 1.0, 0.3).double().cpu()
        for h in range(nq + nk):
            x = z[:, h * dk:(h + 1) * dk].double()
            if inter:  # neighbours: bring them to halves, turn, and bring them back
                order = [i for i in range(0, dims, 2)] + [i for i in range(1, dims, 2)] + list(range(dims, dk))
                want = torch.empty_like(x)
                want[:, order] = plain.rotate(x[:, order], rot)
            else:
                want = plain.rotate(x, rot)
            want = want * (0.3 if h >= nq else 1.0)
            assert float((got[:, h] - want).abs().max()) < 2e-5, (inter, h)


@pytest.mark.parametrize("H,G,dk,dv,dims", [(4, 2, 8, 8, 8), (3, 3, 10, 5, 4), (2, 1, 64, 48, 32), (6, 2, 7, 9, 6), (1, 1, 16, 4, 0)])
def test_query_and_key_rows(dev, H, G, dk, dv, dims):
    # norms over whole rows, rotation by position, cache rows at scattered slots (one row is not to be written)
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(dk + dv)
    T, bs, rot = 13, 4, {"base": 50.0, "dims": dims}
    z = (torch.randn(T, (H + G) * dk + G * dv + 4, generator=g) * 2.0).to(dtype)
    qn, kn = torch.randn(H * dk, generator=g), torch.randn(G * dk, generator=g)
    freq = torch.tensor(plain.frequencies(rot), dtype=torch.float32)
    pos = torch.arange(T)
    zd = z.double()
    q = plain.rms(zd[:, :H * dk], EPS) * qn.double()
    k = plain.rms(zd[:, H * dk:(H + G) * dk], EPS) * kn.double()
    v = zd[:, (H + G) * dk:(H + G) * dk + G * dv]
    slots = torch.randperm(6 * bs, generator=g)[:T]
    slots[3] = -1
    cache = torch.zeros(6, bs, G * (dk + dv), dtype=dtype, device=device)
    got = hybrid.qk_fullnorm_prep(z.to(device), H, G, dk, dv, qn.to(device), kn.to(device), EPS, pos.to(torch.int32).to(device), 0.0, 1, cache,
                                  slots.to(device), freq.to(device), dims, False, 1.0).double().cpu()
    rows = cache.view(-1, G, dv + dk).double().cpu()
    tol = 2e-5 if dtype == torch.float32 else 4e-2
    for h in range(H):
        assert float((got[:, h] - plain.rotate(q[:, h * dk:(h + 1) * dk], rot)).abs().max()) < tol
    for j in range(G):
        kr = plain.rotate(k[:, j * dk:(j + 1) * dk], rot)
        for t, s in enumerate(slots.tolist()):
            if s >= 0:
                assert float((rows[s, j, dv:] - kr[t]).abs().max()) < tol and float((rows[s, j, :dv] - v[t, j * dv:(j + 1) * dv]).abs().max()) < tol
    assert int((rows.flatten(1).abs().sum(1) > 0).sum()) == T - 1


@pytest.mark.parametrize("W", [1, 24, 30, 1000, 1026, 4096, 6144, 9000])
def test_out_norm_pass(dev, W):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(W)
    T = 7
    x, w = torch.randn(T, W, generator=g), torch.randn(W, generator=g) * 0.3
    wide = torch.randn(2, T, W + 4, generator=g).to(dtype)
    wide[0, 2] *= 1000.0
    for two in (False, True):
        y = wide[0, :, :W].double() * 0.6 + (wide[1, :, :W].double() * 1.7 if two else 0.0)
        want = x.double() + 0.4 * plain.norm_one_plus(y, w.double(), EPS)
        xd = x.to(device).clone()
        d = wide.to(device)
        h = hybrid.norm_add_f32_(xd, d[0, :, :W], 0.6, d[1, :, :W] if two else None, 1.7, w.to(device), 0.4, EPS, True, dtype)
        assert h.dtype == dtype and float((xd.double().cpu() - want).abs().max()) < 1e-4
        assert float((h.double().cpu() - want).abs().max()) < (1e-4 if dtype == torch.float32 else 3e-2)
    table = torch.randn(9, W, generator=g).to(dtype)
    ids = torch.tensor([3, 0, 8, 3])
    xe, he = hybrid.embed_f32(ids.to(device), table.to(device))
    assert xe.dtype == torch.float32 and torch.equal(xe.cpu(), table[ids].float()) and torch.equal(he.cpu(), table[ids])


@pytest.mark.parametrize("C,groups", [(12, 1), (24, 6), (30, 5), (2048, 1), (2048, 8), (5000, 1), (7, 7)])
def test_gated_group_norm(dev, C, groups):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(C)
    T, eps = 9, 1e-4
    o, w = torch.randn(T, C, generator=g), torch.randn(C, generator=g)
    o[:, :C // groups] *= 40.0
    wide = (torch.randn(T, C + 8, generator=g) * 2.0).to(dtype)
    y = o.double() * plain.silu(wide[:, :C].double())
    part = C // groups
    want = torch.cat([plain.rms(y[:, i:i + part], eps) for i in range(0, C, part)], -1) * w.double()
    got = hybrid.gate_groupnorm(o.to(device), wide.to(device)[:, :C], w.to(device), groups, eps, dtype).double().cpu()
    assert float((got - want).abs().max()) < (1e-5 if dtype == torch.float32 else 1e-2) * float(want.abs().max())


@pytest.mark.parametrize("H,dv", [(1, 1), (3, 10), (4, 64), (2, 130), (8, 128), (2, 300)])
def test_head_norm_with_and_without_weight(dev, H, dv):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(dv)
    T, eps = 11, 1e-4
    o, w = torch.randn(T, H, dv, generator=g) * 3.0, torch.randn(H * dv, generator=g)
    wide = torch.randn(T, H * dv + 8, generator=g).to(dtype)
    z = wide[:, :H * dv]
    for silu in (True, False):
        gate = plain.silu(z.double()) if silu else plain.sigmoid(z.double())
        want = plain.rms(o.double(), eps).reshape(T, -1) * gate
        for weight in (None, w):
            ref = want if weight is None else want * w.double()
            got = hybrid.headnorm_gate(o.to(device), weight.to(device) if weight is not None else None, wide.to(device)[:, :H * dv], eps, dtype, silu)
            assert float((got.double().cpu() - ref).abs().max()) < (1e-5 if dtype == torch.float32 else 1e-2) * float(ref.abs().max())


# ------------------------------------------------------------------ the framework's own entry points
def test_greedy_generation_through_the_scheduler(tmp_path, dev):
    from llmctl.serve.scheduler import SamplingParams

    device, dtype, _ = dev
    cfg = U.config(FULL)
    W = {k: v.bfloat16().float() for k, v in U.random_weights(cfg, 50).items()}
    path = U.write_checkpoint(tmp_path / "ck", cfg, W)
    eng = U.engine(path, device, dtype, blocks=40, block_size=4, max_seqs=3, scheduler="dynamic")
    prompts = [tokens(9, 50, 51), tokens(2, 50, 52), tokens(14, 50, 53), tokens(5, 50, 54), tokens(1, 50, 55)]
    seqs = eng.generate(prompts, SamplingParams(max_tokens=12, temperature=0.0, ignore_eos=True))
    slack = 1e-3 if dtype == torch.float32 else 0.2
    for s in seqs:
        assert len(s.output_ids) == 12
        logits = plain.forward(cfg, W, s.all_ids[:-1])[0]
        for k, tok in enumerate(s.output_ids):
            row = logits[len(s.prompt_ids) - 1 + k]
            assert row[tok] >= row.max() - slack * float(row.std()), (s.request_id, k)
    assert eng.kv.num_free_blocks == 40 and eng.kv_cache.slots.num_free == 3
    eng.close()


def test_generation_with_preemption(tmp_path):
    # too few pages for all requests: the newest is preempted, loses its pages and state slot, and is recomputed;
    # greedy outputs stay those of an engine with room for all
    from llmctl.serve.scheduler import SamplingParams

    cfg = U.config(FULL)
    path = U.write_checkpoint(tmp_path / "ck", cfg, U.random_weights(cfg, 60))
    prompts = [tokens(6, 50, 61 + i) for i in range(4)]
    p = SamplingParams(max_tokens=10, temperature=0.0, ignore_eos=True)
    tight = U.engine(path, "cpu", blocks=10, block_size=4, max_seqs=4).generate(prompts, p)
    roomy = U.engine(path, "cpu", blocks=64, block_size=4, max_seqs=1).generate(prompts, p)
    assert sum(s.preemptions for s in tight) > 0
    assert [s.output_ids for s in tight] == [s.output_ids for s in roomy]


def test_checkpoint_names_round_trip(tmp_path):
    from llmctl.models import get_model_config
    from llmctl.models.dumazen import DumazenConfig, DumazenLM, load_dumazen

    cfg = U.config(FULL)
    W = {k: v.bfloat16().float() for k, v in U.random_weights(cfg, 70).items()}
    U.write_checkpoint(tmp_path / "ck", cfg, W)
    m = load_dumazen(tmp_path / "ck", DumazenConfig.from_file(tmp_path / "ck" / "config.json"), dtype=torch.float32)
    assert [k for k, _ in m.cache_kinds()] == ["rows+state", "state", "state", "rows+state", "state", "state"]
    back = m.export_named()
    assert set(back) == set(W)
    for k in W:
        assert torch.equal(back[k].float(), W[k]), k
    c = DumazenConfig.from_dict(cfg)
    assert DumazenConfig.from_dict(c.to_dict()).to_dict() == c.to_dict()
    t = get_model_config("dumazen-w64-l6-h4-g2")
    assert t.architecture == "Dumazen" and t.layers == 6 and {s["type"] for s in t.layer_specs} == {"parallel", "mamba2", "retention"}
    assert sum(p.numel() for p in DumazenLM(t, dtype=torch.float32).parameters()) == t.num_parameters()
    bad = dict(W)
    bad["l0.mix.left.q"], bad["l0.mix.left.k"] = W["l0.mix.left.k"], W["l0.mix.left.q"]
    with pytest.raises(ValueError):
        m.load_named(bad)
    for spec in ({"type": "mlstm", "mixer": {}, "mlp": None}, dict(U.ret(), mlp={"kind": "moe"})):
        with pytest.raises(ValueError):
            DumazenConfig.from_dict(dict(cfg, layers=[spec]))
    for m_ in (U.par(U.left(heads=3, kv_heads=2)), U.par(r=U.right(heads=3, kv_heads=2)), U.ssm(heads=3, groups=2), U.ssm(heads=2, vdim=5, norm_groups=3),
               U.ret(heads=2, decay=[0.5]), U.ret(dim=4, dims=6)):
        with pytest.raises(ValueError):
            DumazenLM(DumazenConfig.from_dict(U.config([(m_, None)])), dtype=torch.float32)


def test_trace_replay_command(tmp_path):
    # the replay command end to end on a written checkpoint: two requests, a shared step, logits files
    import json
    import subprocess
    import sys

    import numpy as np

    cfg = U.config(FULL)
    W = {k: v.bfloat16().float() for k, v in U.random_weights(cfg, 80).items()}
    path = U.write_checkpoint(tmp_path / "ck", cfg, W)
    a, b = tokens(10, 50, 81), tokens(5, 50, 82)
    steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:6], "want": [0, 5]}], "end": []},
             {"step": 1, "entries": [{"id": "a", "tokens": a[6:7], "want": []}, {"id": "b", "tokens": b[:4], "want": [3]}], "end": []},
             {"step": 2, "entries": [{"id": "b", "tokens": b[4:], "want": [0]}, {"id": "a", "tokens": a[7:], "want": [2]}], "end": ["a", "b"]}]
    out = tmp_path / "out"
    r = subprocess.run([sys.executable, "-m", "llmctl.serve.trace_replay", "--model", path, "--dtype", "float32", "--out", str(out),
                        "--max-tokens", "64", "--device", "cpu", "--block-size", "4"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=300)
    assert r.returncode == 0, r.stderr
    assert [l for l in r.stdout.splitlines() if l.startswith("done")] == ["done 0", "done 1", "done 2"]
    la, lb = plain.forward(cfg, W, a)[0], plain.forward(cfg, W, b)[0]
    for step, want in ((0, torch.stack([la[0], la[5]])), (1, lb[3:4]), (2, torch.stack([lb[4], la[9]]))):
        got = torch.from_numpy(np.fromfile(out / f"{step}.f32", dtype="<f4").reshape(-1, cfg["vocab"]).copy())
        assert U.rel_err(got, want.float()) < 1e-3
