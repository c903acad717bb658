"""Dapipel through the serving engine against the plain whole-sequence implementation in
``tests/oracles/dapipel_plain.py``: every mechanism alone, whole prompts against token-by-token decoding,
portions down to two tokens, unequal batches, reused pages and state slots, far keys and the edges of pages, key
tiles and windows, the first tokens of a sequence, long decoding, other sizes, and greedy generation through the
scheduler.

Each test runs on the CPU path and, marked ``gpu``, on the HIP kernels: fp32 with a tight bound at every
position; bf16 with loose bounds on the median and on nine positions in ten and a sanity bound on the rest.  Multi-layer
schedules in bf16 use routers that choose every expert (an expert near-tie that flips under bf16 rounding changes all
later positions through the recurrence); routed choice in bf16 is covered by the one-layer tests."""

import random

import pytest
import torch

from tests.models import dapipel_util as U
from tests.oracles import dapipel_plain as plain

DEVICES = [("cpu", torch.float32, 2e-4),
           pytest.param(("cuda", torch.float32, 2e-4), marks=pytest.mark.gpu),
           pytest.param(("cuda", torch.bfloat16, 0.1), marks=pytest.mark.gpu)]
EPS = 1e-5


@pytest.fixture(params=DEVICES, ids=lambda p: f"{p[0]}-{str(p[1]).split('.')[-1]}")
def dev(request):
    return request.param


def tokens(n, vocab, seed):
    r = random.Random(seed)
    return [r.randrange(vocab) for _ in range(n)]


def check(tmp_path, dev, cfg, requests, steps, seed=0, blocks=64, block_size=4, W=None, max_seqs=4, bf16_tol=None,
          bf16_all=False):
    device, dtype, tol = dev
    if bf16_tol is not None and dtype == torch.bfloat16:
        tol = bf16_tol
    if bf16_all and dtype == torch.bfloat16:
        cfg = U.without_choice(cfg)
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


FULL = [(U.gru(), U.dense()), (U.att(), U.moe()), (U.gru(30), None), (U.att(heads=2, kv_heads=2, dim=5, vdim=10, window=11, diff=0.6), U.dense(9)),
        (U.att(heads=3, kv_heads=1, dim=4, vdim=4, window=3), None), (U.gru(9), U.moe(experts=4, top=1, ff=7))]


# ------------------------------------------------------------------ each mechanism alone
def test_differential_attention_alone(tmp_path, dev):
    cfg = U.config([(U.att(), None)])
    r = {"a": tokens(23, 50, 1)}
    check(tmp_path, dev, cfg, r, whole(r))


@pytest.mark.parametrize("sizes", [dict(heads=3, kv_heads=3, dim=10, vdim=4, window=1), dict(heads=6, kv_heads=1, dim=4, vdim=8, window=3, diff=0.8),
                                   dict(heads=1, kv_heads=1, dim=1, vdim=3, window=200), dict(heads=4, kv_heads=2, dim=8, vdim=16, scale=0.9, window=26),
                                   dict(heads=2, kv_heads=2, dim=7, vdim=33, window=16, diff=0.0)])
def test_differential_attention_sizes(tmp_path, dev, sizes):
    # as many kv heads as heads, one kv head, one head, a window of one key, one that is longer than the sequence or as
    # long, key and value sizes that differ, one key channel, no part of the factor that is fixed
    cfg = U.config([(U.att(**sizes), None)], groups=1)
    r = {"a": tokens(26, 50, 2)}
    check(tmp_path, dev, cfg, r, [[("a", 9)], [("a", 1)], [("a", 16)]])


@pytest.mark.parametrize("dot1,dot2", [(0.7, -1.5), (-2.0, 1.1), (-4.0, -4.0)])
def test_factor_of_the_second_map(tmp_path, dev, dot1, dot2):
    # the learned part of the factor: exp(dot1) - exp(dot2), from large to negative to nearly nothing
    cfg = U.config([(U.att(dim=4), None)])
    W = U.random_weights(cfg, 3)
    for a, b, t in (("lq1", "lk1", dot1), ("lq2", "lk2", dot2)):
        W[f"l0.mix.{a}"], W[f"l0.mix.{b}"] = torch.tensor([0.5, -1.0, 0.0, 2.0]), torch.tensor([t, t, 3.0, 0.75 * t])
    r = {"a": tokens(17, 50, 3)}
    check(tmp_path, dev, cfg, r, [[("a", 8)], [("a", 1)], [("a", 8)]], W=W)


def test_mingru_alone(tmp_path, dev):
    cfg = U.config([(U.gru(), None)])
    r = {"a": tokens(27, 50, 4)}
    check(tmp_path, dev, cfg, r, whole(r))


@pytest.mark.parametrize("width", [1, 7, 64, 130])
def test_mingru_sizes(tmp_path, dev, width):
    cfg = U.config([(U.gru(width), None)])
    r = {"a": tokens(90, 50, 5), "b": tokens(4, 50, 6)}
    check(tmp_path, dev, cfg, r, [[("a", 70), ("b", 2)], [("a", 1), ("b", 1)], [("a", 19), ("b", 1)]])


def test_gates_open_and_shut(tmp_path, dev):
    # half of the channels keep their state almost for good, the others take every token's candidate; candidates on
    # both sides of zero, far out and close by
    cfg = U.config([(U.gru(12), None)])
    W = U.random_weights(cfg, 7)
    b = torch.full((12,), 9.0)
    b[::2] = -7.0
    W["l0.mix.z.b"] = b
    W["l0.mix.x.b"] = torch.tensor([-6.0, -6.0, 5.0, 5.0, 0.0, 0.0] * 2)
    r = {"a": tokens(80, 50, 7)}
    check(tmp_path, dev, cfg, r, [[("a", 13)], [("a", 67)]], W=W)


@pytest.mark.parametrize("f", [U.dense(1), U.dense(40), U.moe(experts=5, top=1, ff=7), U.moe(experts=4, top=4, ff=6), U.moe(experts=9, top=3, ff=1),
                               U.moe(experts=1, top=1, ff=12), U.moe(experts=16, top=2, ff=8)])
def test_feed_forwards(tmp_path, dev, f):
    cfg = U.config([(U.gru(6), f)])
    r = {"a": tokens(40, 50, 8), "b": tokens(9, 50, 9)}
    check(tmp_path, dev, cfg, r, [[("a", 40), ("b", 2)], [("b", 1)], [("b", 6)]], bf16_tol=0.3)


def test_weights_are_a_softmax_over_the_chosen_logits(tmp_path, dev):
    # router logits far apart: one expert takes nearly all, and the rest of the mass must not be lost to the unchosen
    cfg = U.config([(U.gru(6), U.moe(experts=6, top=2))])
    W = U.random_weights(cfg, 10)
    W["l0.mlp.router"] = W["l0.mlp.router"] * 0.05  # nearly equal scores: a softmax over all would halve the output
    r = {"a": tokens(30, 50, 10)}
    check(tmp_path, dev, cfg, r, whole(r), W=W, bf16_tol=0.6)


@pytest.mark.parametrize("width,groups,taps", [(24, 1, 4), (24, 6, 2), (24, 24, 3), (20, 2, 1), (21, 3, 5), (30, 5, 4), (64, 4, 6)])
def test_norm_groups_and_taps(tmp_path, dev, width, groups, taps):
    # one group, groups of one channel (there a small eps would make a norm a sign: a larger one), groups that are no column quads, one tap (no state), more taps than the
    # one-pass form has
    cfg = U.config([(U.att(), U.dense()), (U.gru(), U.moe())], width=width, groups=groups, taps=taps, eps=0.05 if groups == width else EPS)
    r = {"a": tokens(25, 50, 11), "b": tokens(6, 50, 12)}
    check(tmp_path, dev, cfg, r, [[("a", 2), ("b", 1)], [("a", 1), ("b", 1)], [("a", 2), ("b", 4)], [("a", 20)]], bf16_all=True)


def test_groups_are_normed_each_by_itself(tmp_path, dev):
    # one part of the stream is 50 times larger than the others
    cfg = U.config([(U.gru(), None)], groups=4)
    W = U.random_weights(cfg, 13)
    for n in ("embed", "pos"):
        W[n][:, :6] *= 50.0
    r = {"a": tokens(19, 50, 13)}
    check(tmp_path, dev, cfg, r, [[("a", 9)], [("a", 1)], [("a", 9)]], W=W)


def test_embedding_scale_and_positions(tmp_path, dev):
    cfg = U.config([(U.att(), None)], scale=0.25)
    r = {"a": [7] * 20}  # one token over and over: only its position and the window tell the rows apart
    check(tmp_path, dev, cfg, r, [[("a", 6)], [("a", 1)], [("a", 13)]])


def test_stream_after_every_layer(tmp_path):
    from llmctl.serve.scheduler import PrefillChunk

    cfg = U.config(FULL)
    W = {k: v.bfloat16().float() for k, v in U.random_weights(cfg, 14).items()}
    eng = U.engine(U.write_checkpoint(tmp_path / "ck", cfg, W), "cpu")
    toks = tokens(15, 50, 14)
    seq = eng.open_sequence(toks)
    trail = []
    eng.forward_portions([PrefillChunk(seq, 0, len(toks))], [[0]], trail=trail)
    want = plain.forward(cfg, W, toks)[1]
    assert len(trail) == len(want) == len(FULL)
    for a, b in zip(trail, want):
        assert float((a.double() - b).abs().max()) < 1e-3 * float(b.abs().max())


def test_no_layers(tmp_path, dev):
    cfg = U.config([])
    r = {"a": tokens(5, 50, 15)}
    check(tmp_path, dev, cfg, r, whole(r))


# ------------------------------------------------------------------ schedules
def test_prefill_against_token_by_token(tmp_path, dev):
    cfg = U.config(FULL)
    r = {"a": tokens(26, 50, 20)}
    check(tmp_path, dev, cfg, r, [[("a", 1)]] * 26, bf16_all=True)


def test_portions_of_several_sizes(tmp_path, dev):
    cfg = U.config(FULL)
    r = {"a": tokens(61, 50, 21)}
    check(tmp_path, dev, cfg, r, [[("a", n)] for n in (2, 17, 3, 2, 30, 1, 1, 5)], bf16_all=True)


def test_unequal_batches(tmp_path, dev):
    cfg = U.config(FULL, taps=4)
    r = {"a": tokens(40, 50, 22), "b": tokens(7, 50, 23), "c": tokens(19, 50, 24), "d": tokens(2, 50, 25)}
    steps = [[("a", 11), ("b", 2)], [("a", 1), ("b", 4), ("c", 9)], [("c", 1), ("a", 20), ("b", 1), ("d", 2)], [("a", 8), ("c", 9)]]
    check(tmp_path, dev, cfg, r, steps, bf16_all=True)


def test_pages_and_slots_used_again(tmp_path, dev):
    # 12 pages of 4 tokens and 2 state slots for five requests: every later request runs in pages and a slot that hold
    # an earlier one's rows, states and carried inputs
    cfg = U.config(FULL, taps=4)
    r = {k: tokens(n, 50, 30 + i) for i, (k, n) in enumerate([("a", 22), ("b", 18), ("c", 20), ("d", 9), ("e", 23)])}
    steps = [[("a", 10), ("b", 18)], [("a", 12), ("c", 3)], [("c", 17), ("d", 1)], [("d", 1)], [("d", 7), ("e", 2)], [("e", 21)]]
    check(tmp_path, dev, cfg, r, steps, blocks=12, max_seqs=2, bf16_all=True)


def test_token_by_token_start_in_a_used_slot(tmp_path, dev):
    # fewer tokens than taps lie behind the first decoded ones: what the slot held before must not enter
    cfg = U.config([(U.gru(), None), (U.att(), U.dense())], taps=4)
    r = {"a": tokens(30, 50, 36), "b": tokens(12, 50, 37)}
    check(tmp_path, dev, cfg, r, [[("a", 30)]] + [[("b", 1)]] * 12, blocks=10, max_seqs=1)


def test_long_decoding_over_window_and_tile_borders(tmp_path, dev):
    # 150 decoded tokens after a short prompt: the window (37) passes over decoded tokens, contexts cross 64-key tiles and
    # many pages
    cfg = U.config([(U.att(window=37, heads=2, kv_heads=1, dim=8, vdim=16), None), (U.gru(), U.moe()), (U.att(window=66), None)], positions=160)
    r = {"a": tokens(156, 50, 38)}
    check(tmp_path, dev, cfg, r, [[("a", 6)]] + [[("a", 1)]] * 150, blocks=48, bf16_all=True)


def test_long_portions(tmp_path, dev):
    # 650-token portions (chunk-parallel scan, several query blocks, rows of a sequence over many workgroups) continued
    # in a second and a third step
    cfg = U.config([(U.gru(10), None), (U.att(window=70), None), (U.gru(12), U.dense(8))], taps=4, positions=720)
    r = {"a": tokens(700, 50, 39), "b": tokens(300, 50, 40)}
    check(tmp_path, dev, cfg, r, [[("a", 650), ("b", 10)], [("a", 49), ("b", 290)], [("a", 1)]], blocks=260)


def test_heads_that_fit_the_matrix_cores(tmp_path, dev):
    # head sizes in multiples of 8 (the bf16 runs take the matrix-core form), a prompt over several 64-key tiles, windows
    # of 70 and 130 keys, then decoding, beside a short request
    cfg = U.config([(U.att(heads=4, kv_heads=2, dim=32, vdim=48, window=70), None), (U.gru(40), U.dense(32)),
                    (U.att(heads=4, kv_heads=1, dim=24, vdim=80, window=130), None)], width=64, groups=2, taps=4, positions=256)
    r = {"a": tokens(230, 50, 41), "b": tokens(9, 50, 42)}
    check(tmp_path, dev, cfg, r, [[("a", 200), ("b", 4)]] + [[("a", 1), ("b", 1)]] * 5 + [[("a", 25)]], blocks=80)


@pytest.mark.parametrize("seed", range(8))
def test_random_configurations(tmp_path, dev, seed):
    # sizes, layer order, windows, constants and schedules drawn at random (some sizes fit the vector and matrix-core
    # forms, some do not)
    r = random.Random(900 + seed)
    step = r.choice([1, 4, 8])
    size = lambda lo, hi: max(1, r.randint(lo, hi) // step) * step
    layers = []
    for _ in range(r.randint(2, 4)):
        if r.random() < 0.5:
            m = U.gru(size(4, 70))
        else:
            G = r.choice([1, 2, 3])
            m = U.att(heads=G * r.choice([1, 2, 3]), kv_heads=G, dim=size(4, 40), vdim=size(4, 72), window=r.randint(1, 90),
                      diff=r.choice([0.2, 0.5, 0.8]))
        f = r.choice([None, U.dense(size(4, 60)), U.moe(experts=r.randint(1, 9), top=1, ff=size(4, 40))])
        if f is not None and f["kind"] == "moe":
            f["router"]["top"] = r.randint(1, f["router"]["experts"])
        layers.append((m, f))
    groups = r.choice([1, 2, 4])
    cfg = U.config(layers, width=groups * r.choice([12, 16, 20, 33]), vocab=r.choice([37, 64, 101]), eps=r.choice([1e-6, 1e-4]), groups=groups,
                   taps=r.choice([2, 3, 4, 5]), scale=r.choice([0.5, 2.0, 4.0]), positions=200)
    reqs = {k: tokens(r.randint(3, 150), cfg["vocab"], 901 + i) for i, k in enumerate("abc")}
    left, steps = {k: len(t) for k, t in reqs.items()}, []
    while any(left.values()):
        entries = []
        for k in list(left):
            if left[k] and r.random() < 0.7:
                n = min(left[k], r.choice([1, 1, 2, 3, 17, 64, 90]))
                entries.append((k, n))
                left[k] -= n
        if entries:
            steps.append(entries)
    check(tmp_path, dev, cfg, reqs, steps, seed=seed, blocks=40, block_size=16, bf16_all=True, bf16_tol=0.2)


# ------------------------------------------------------------------ far keys and edges, at op level
def _diff_case(device, dtype, bs, L, j0, form, mfma, window, H=4, G=2, dk=16, dv=24, which=0):
    """One key (position j0) stands out in map ``which`` for the last queries; they see it if it lies in their window.
    Returns (got, want) for the last ``n`` positions; pages lie anywhere in the pool."""
    from llmctl.ops import hybrid

    g = torch.Generator().manual_seed(1000 * L + j0)
    q = torch.randn(L, H, 2, dk, generator=g) * 0.3
    k = torch.randn(L, G, 2, dk, generator=g) * 0.3
    v = torch.randn(L, G, dv, generator=g)
    v[j0] += 9.0
    dirn = torch.randn(dk, generator=g)
    dirn /= dirn.norm()
    k[j0, :, which] = dirn * 4.0
    n = min(L, 70)
    q[L - n:, :, which] += dirn * 3.0
    q, k, v = q.to(dtype), k.to(dtype), v.to(dtype)
    scale, lam, post = 1.1, 0.45, 0.7
    vis = plain.window_mask(L, window)
    want = torch.zeros(L, H, dv, dtype=torch.float64)
    for h in range(H):
        a = [plain.attend(q[:, h, m].double(), k[:, h // (H // G), m].double(), v[:, h // (H // G)].double(), scale, vis) for m in (0, 1)]
        o = a[0] - lam * a[1]
        want[:, h] = o / torch.sqrt((o * o).mean(-1, keepdim=True) + EPS) * post
    dev_ = torch.device(device)
    nb = (L + bs - 1) // bs
    perm = torch.randperm(nb + 3, generator=g)[:nb]
    cache = torch.full((nb + 3, bs, G * (dv + 2 * dk)), 3.0, dtype=dtype)
    rows = torch.cat([v, k.reshape(L, G, 2 * dk)], -1).reshape(L, -1)
    for p in range(L):
        cache[perm[p // bs], p % bs] = rows[p]
    cache, bt = cache.to(dev_), perm.to(torch.int32).view(1, nb).to(dev_)
    i32 = lambda x: torch.tensor(x, dtype=torch.int32, device=dev_)
    pad = torch.zeros(L, 8, dtype=dtype)
    z = torch.cat([q.reshape(L, -1), pad], 1).to(dev_)  # queries as columns of a wider row
    args = (H, G, dk, dv, window, scale, torch.tensor([lam], device=dev_), post, EPS)
    if form == "prefill":
        out = torch.full((n, H * dv), 7.0, dtype=dtype, device=dev_)
        hybrid.diff_attention(z[L - n:], cache, bt, i32([0, n]), i32([L]), *args, out=out, max_q=n, mfma=mfma)
        got, want = out, want[L - n:]
    else:
        m = min(n, 8)
        outs = []
        for p in range(L - m, L):
            out = torch.full((1, H * dv), 7.0, dtype=dtype, device=dev_)
            outs.append(hybrid.diff_attention(z[p:p + 1], cache, bt, None, i32([p + 1]), *args, out=out, max_ctx=p + 1, mfma=mfma))
        got, want = torch.cat(outs), want[L - m:]
    return got.double().cpu().view(-1, H, dv), want


@pytest.mark.parametrize("form", ["prefill", "decode"])
@pytest.mark.parametrize("bs,L,j0,window", [(4, 60, 51, 9), (4, 60, 52, 9), (8, 200, 170, 30), (8, 200, 2, 300), (16, 200, 63, 137), (16, 200, 64, 137),
                                            (16, 420, 0, 420), (16, 420, 0, 419), (16, 700, 599, 100), (16, 700, 600, 100), (16, 700, 601, 100),
                                            (16, 700, 150, 1 << 30), (16, 330, 127, 203), (16, 330, 128, 203), (16, 5, 0, 4)])
def test_far_keys_and_window_edges(dev, form, bs, L, j0, window):
    # the standing-out key lies far back, just inside or just outside the last queries' windows, on either side of
    # page and 64-key-tile borders; it stands out in the first and in the second map
    device, dtype, _ = dev
    tol = 1e-4 if dtype == torch.float32 else 3e-2
    for mfma in ([True, False] if (device == "cuda" and dtype == torch.bfloat16) else [True]):
        for which in (0, 1):
            got, want = _diff_case(device, dtype, bs, L, j0, form, mfma, window, which=which)
            assert float((got - want).abs().max()) < tol, (mfma, which)


@pytest.mark.gpu
@pytest.mark.parametrize("H,G,dk,dv", [(8, 4, 56, 64), (4, 4, 64, 128), (6, 1, 128, 72), (3, 3, 24, 8), (12, 4, 64, 40), (2, 1, 72, 256), (5, 5, 20, 10),
                                       (2, 2, 160, 16), (4, 2, 8, 200), (3, 1, 9, 300), (40, 1, 16, 16)])
def test_differential_attention_kernels_gpu(H, G, dk, dv):
    # the matrix-core and the generic kernels on other head counts and sizes (values of one, two and several column tiles,
    # keys of one and two image blocks), prompt and decode forms
    for dtype, tol in ((torch.bfloat16, 5e-2), (torch.float32, 1e-4)):
        for form in ("prefill", "decode"):
            for mfma in (True, False):
                got, want = _diff_case("cuda", dtype, 16, 300, 215, form, mfma, 90, H=H, G=G, dk=dk, dv=dv, which=1)
                assert float((got - want).abs().max()) < tol, (dtype, form, mfma)


# ------------------------------------------------------------------ the recurrence and the stream pass at op level
def _batch(cuts_pos, device, W=1):
    """A StepBatch's sequence part for portions [(length, first position, slot)], prompt portions first."""
    from llmctl.models.mixers import StepBatch

    i32 = lambda a: torch.tensor(a, dtype=torch.int32, device=device)
    cu = [0]
    for n, _, _ in cuts_pos:
        cu.append(cu[-1] + n)
    pre = [c for c in cuts_pos if c[0] > 1 or c[1] == 0]
    Tp = sum(c[0] for c in pre)
    assert cuts_pos[:len(pre)] == pre
    seq_of = [i for i, (n, _, _) in enumerate(cuts_pos) for _ in range(n)]
    return StepBatch(ids=None, pos=None, slots=None, Tp=Tp, p_cu=None, p_ctx=i32([c[0] + c[1] for c in pre]) if pre else None, p_bt=None,
                     d_ctx=None, d_bt=None, cu=i32(cu), start=i32([c[1] for c in cuts_pos]), state=i32([c[2] for c in cuts_pos]),
                     max_q=max((c[0] for c in pre), default=0), cu_host=cu, seq_of=i32(seq_of),
                     carried=any(n > 1 and p > 0 for n, p, _ in cuts_pos))


@pytest.mark.parametrize("T,cuts,far,W", [(40, [40], 2, 6), (300, [300], 1, 10), (300, [7, 1, 1, 290, 1], 5, 7), (700, [257, 443], 3, 130), (130, [64, 64, 2], 63, 64)])
def test_state_survives_and_forgets(dev, T, cuts, far, W):
    # channel 0 takes token ``far``'s candidate and then keeps it to the end; channel 1 forgets at once; junk in the slot
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(T + W)
    z = torch.randn(T, 3 * W + 2, generator=g)
    z[:, 0] = -25.0
    z[far, 0], z[far, W] = 25.0, 30.0
    z[:, 1] = 25.0
    z = z.to(dtype)
    zb, xb = torch.randn(W, generator=g) * 0.3, torch.randn(W, generator=g) * 0.3
    zd = z.double()
    zeta = plain.sigmoid(zd[:, :W] + zb.double())
    u = zd[:, W:2 * W] + xb.double()
    cand = torch.where(u >= 0, u + 0.5, plain.sigmoid(u))
    S, want = torch.zeros(W, dtype=torch.float64), torch.zeros(T, W, dtype=torch.float64)
    for t in range(T):
        S = (1 - zeta[t]) * S + zeta[t] * cand[t]
        want[t] = S * plain.silu(zd[t, 2 * W:3 * W])
    assert float(S[0]) > 29.0
    tol = 1e-4 if dtype == torch.float32 else 2e-2
    for chunk in ([0, 16, 128, 1 << 20] if device == "cuda" else [0]):
        pool = torch.randn(3, W, generator=g).to(device)
        outs, at = [], 0
        for n in cuts:
            outs.append(hybrid.mingru_scan(z[at:at + n].to(device), zb.to(device), xb.to(device), pool, _batch([(n, at, 1)], device), chunk))
            at += n
        got = torch.cat(outs).double().cpu()
        assert float((got - want).abs().max()) / float(want.abs().max()) < tol, chunk
        assert float((pool[1].double().cpu() - S).abs().max()) < 1e-3, chunk


def test_scan_over_a_mixed_batch(dev):
    # two long portions (one that continues a sequence), a short one and two decoded rows in one step
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(9)
    W = 70
    cuts = [(200, 0, 3), (90, 5, 0), (2, 0, 4), (1, 8, 1), (1, 30, 2)]
    T = sum(c[0] for c in cuts)
    z = torch.randn(T, 3 * W, generator=g).to(dtype)
    zb, xb = torch.randn(W, generator=g), torch.randn(W, generator=g)
    pool = torch.randn(5, W, generator=g)
    zd, a = z.double(), 0
    want, end = torch.zeros(T, W, dtype=torch.float64), pool.double().clone()
    for n, p, slot in cuts:
        S = torch.zeros(W, dtype=torch.float64) if p == 0 else pool[slot].double()
        for t in range(a, a + n):
            zeta, u = plain.sigmoid(zd[t, :W] + zb.double()), zd[t, W:2 * W] + xb.double()
            S = (1 - zeta) * S + zeta * torch.where(u >= 0, u + 0.5, plain.sigmoid(u))
            want[t] = S * plain.silu(zd[t, 2 * W:])
        end[slot], a = S, a + n
    pool = pool.to(device)
    got = hybrid.mingru_scan(z.to(device), zb.to(device), xb.to(device), pool, _batch(cuts, device)).double().cpu()
    assert float((got - want).abs().max()) / float(want.abs().max()) < (1e-4 if dtype == torch.float32 else 2e-2)
    assert float((pool.double().cpu() - end).abs().max()) < 1e-4


@pytest.mark.parametrize("W,groups,taps", [(12, 3, 2), (64, 1, 4), (200, 2, 3), (1000, 5, 4), (1280, 2, 4), (2560, 4, 2), (4096, 1, 3), (6144, 3, 4), (30, 5, 4), (40, 2, 7),
                                           (16, 2, 1)])
def test_stream_pass(dev, W, groups, taps):
    # the update of the stream, the grouped norm and the convolution with its carried rows, over a batch whose sequences
    # span workgroups, then over a second step that continues them all, then one that also begins new ones in used slots;
    # every width tier and the unfused form
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(W + taps)
    lens = [(270, 0, 2), (3, 0, 0), (251, 0, 1), (2, 0, 4)] if W <= 1280 else [(40, 0, 2), (3, 0, 0), (30, 0, 1), (2, 0, 4)]
    then = [(n, p, s) for n, p, s in [(263, lens[0][0], 2), (2, 3, 0), (1, lens[2][0], 1), (1, 2, 4)]]
    if W > 1280:
        then[0] = (25, lens[0][0], 2)
    mixed = [(5, 0, 0), (7, then[0][0] + then[0][1], 2), (9, 0, 3), (1, 3, 4), (1, lens[2][0] + 1, 1)]
    w, cw = torch.randn(W, generator=g), torch.randn(W, taps, generator=g) * 0.5
    state = torch.randn(5, taps - 1, W, generator=g).to(device)
    hist = {}
    for step, cuts in enumerate((lens, then, mixed)):
        T = sum(c[0] for c in cuts)
        x, y = torch.randn(T, W, generator=g), torch.randn(T, W, generator=g).to(dtype)
        x[:, :W // groups] *= 30.0  # one group is much larger than the others
        xs = x.double() + y.double()
        h = plain.group_norm(xs, w.double(), groups, EPS)
        want, a = torch.zeros(T, W, dtype=torch.float64), 0
        for n, p, s in cuts:
            ext = h[a:a + n] if p == 0 else torch.cat([hist[s], h[a:a + n]])
            want[a:a + n] = plain.add_conv(ext, cw.double())[-n:]
            hist[s], a = ext, a + n
        xo, got = hybrid.add_norm_conv(x.to(device), y.to(device), w.to(device), groups, EPS, cw.t().contiguous().to(device), state,
                                       _batch(cuts, device), dtype)
        assert got.dtype == dtype
        assert float((xo.double().cpu() - xs).abs().max()) < 1e-4
        err = (got.double().cpu() - want).abs().max() / want.abs().max()
        assert float(err) < (2e-5 if dtype == torch.float32 else 5e-3), step
        for n, p, s in cuts:
            tail = hist[s][-(taps - 1):] if taps > 1 else hist[s][:0]
            k = tail.shape[0]
            assert k == 0 or float((state[s, taps - 1 - k:].double().cpu() - tail).abs().max()) < 2e-4, (step, s)


@pytest.mark.parametrize("W,groups,taps", [(24, 2, 4), (1536, 3, 4), (30, 3, 5)])
def test_stream_start(dev, W, groups, taps):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(W)
    table, ptab = torch.randn(11, W, generator=g).to(dtype), torch.randn(40, W, generator=g).to(dtype)
    w, cw = torch.randn(W, generator=g), torch.randn(W, taps, generator=g) * 0.5
    cuts = [(30, 0, 1), (4, 0, 0)]
    b = _batch(cuts, device)
    ids = torch.randint(0, 11, (34,), generator=g)
    pos = torch.cat([torch.arange(30), torch.arange(4)])
    b.ids, b.pos = ids.to(device), pos.to(torch.int32).to(device)
    xs = table.double()[ids] * 2.5 + ptab.double()[pos]
    h = plain.group_norm(xs, w.double(), groups, EPS)
    want = torch.cat([plain.add_conv(h[:30], cw.double()), plain.add_conv(h[30:], cw.double())])
    state = torch.randn(2, taps - 1, W, generator=g).to(device)
    x, got = hybrid.embed_norm_conv(table.to(device), ptab.to(device), 2.5, w.to(device), groups, EPS, cw.t().contiguous().to(device), state, b)
    assert float((x.double().cpu() - xs).abs().max()) < 1e-4
    assert float((got.double().cpu() - want).abs().max()) < (2e-4 if dtype == torch.float32 else 8e-2)
    _, hn = hybrid.group_norm_f32(x, None, w.to(device), groups, EPS, dtype)
    assert float((hn.double().cpu() - h).abs().max()) < (2e-4 if dtype == torch.float32 else 5e-2)


@pytest.mark.parametrize("F", [1, 24, 100])
def test_gated_activations(dev, F):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(F)
    wide = (torch.randn(9, 2 * F + 8, generator=g) * 3.0).to(dtype)
    wide[0, 8:8 + F] = -40.0
    gu = wide[:, 8:]
    s = torch.randn(9, generator=g)
    for kind, fn in (("silu", plain.silu), ("gelu_tanh", plain.gelu_tanh)):
        want = fn(gu[:, :F].double()) * gu[:, F:].double()
        for scale in (None, s):
            got = hybrid.glu_act(wide.to(device)[:, 8:], kind, scale.to(device) if scale is not None else None).double().cpu()
            ref = want if scale is None else want * s.double()[:, None]
            assert float((got - ref).abs().max()) < (1e-5 if dtype == torch.float32 else 1e-2) * float(ref.abs().max()), kind


@pytest.mark.parametrize("G,kw,dv", [(2, 16, 8), (3, 10, 5), (1, 128, 64)])
def test_cache_rows(dev, G, kw, dv):
    from llmctl.ops import hybrid

    device, dtype, _ = dev
    g = torch.Generator().manual_seed(kw)
    T, bs = 13, 4
    z = torch.randn(T, 8 + G * (kw + dv), generator=g).to(dtype).to(device)
    cache = torch.zeros(6, bs, G * (kw + dv), dtype=dtype, device=device)
    slots = torch.randperm(6 * bs, generator=g)[:T]
    slots[3] = -1  # a row that is not to be written
    hybrid.kv_rows_write(z[:, 8:8 + G * kw], z[:, 8 + G * kw:], cache, slots.to(device), G)
    rows = cache.view(-1, G, kw + dv).cpu()
    for t, s in enumerate(slots.tolist()):
        if s >= 0:
            assert torch.equal(rows[s, :, :dv].reshape(-1), z[t, 8 + G * kw:].cpu()) and torch.equal(rows[s, :, dv:].reshape(-1), z[t, 8:8 + G * kw].cpu())
    assert int((rows.flatten(1).abs().sum(1) > 0).sum()) == T - 1


# ------------------------------------------------------------------ the framework's own entry points
def test_greedy_generation_through_the_scheduler(tmp_path, dev):
    from llmctl.serve.scheduler import SamplingParams

    device, dtype, _ = dev
    cfg = U.config(FULL)
    if dtype == torch.bfloat16:
        cfg = U.without_choice(cfg)
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


def test_positions_beyond_the_table_are_refused(tmp_path):
    cfg = U.config([(U.gru(), None)], positions=12)
    eng = U.engine(U.write_checkpoint(tmp_path / "ck", cfg, U.random_weights(cfg, 65)), "cpu")
    with pytest.raises(ValueError):
        U.run_schedule(eng, {"a": tokens(13, 50, 65)}, [[("a", 13)]])


def test_checkpoint_names_round_trip(tmp_path):
    from llmctl.models import get_model_config
    from llmctl.models.dapipel import DapipelConfig, DapipelLM, load_dapipel

    cfg = U.config(FULL)
    W = {k: v.bfloat16().float() for k, v in U.random_weights(cfg, 70).items()}
    U.write_checkpoint(tmp_path / "ck", cfg, W)
    m = load_dapipel(tmp_path / "ck", DapipelConfig.from_file(tmp_path / "ck" / "config.json"), dtype=torch.float32)
    kinds = [k for k, _ in m.cache_kinds()]
    assert kinds == ["state", "rows+state", "state", "rows+state", "rows+state", "state"]
    back = m.export_named()
    assert set(back) == set(W)
    for k in W:
        assert torch.equal(back[k].float(), W[k]), k
    c = DapipelConfig.from_dict(cfg)
    assert DapipelConfig.from_dict(c.to_dict()).to_dict() == c.to_dict()
    t = get_model_config("dapipel-w64-l6-h4-g2-e4")
    assert t.architecture == "Dapipel" and t.layers == 6 and t.is_moe
    assert not get_model_config("dapipel-w64-l3-h4-g2").is_moe
    assert sum(p.numel() for p in DapipelLM(t, dtype=torch.float32).parameters()) == t.num_parameters()
    for bad in (dict(cfg, norm={"eps": 1e-5, "groups": 7}), dict(cfg, canon={"taps": 0}),
                dict(cfg, layers=[{"type": "mlstm", "mixer": {}, "mlp": None}])):
        with pytest.raises(ValueError):
            DapipelConfig.from_dict(bad)


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
    want = {0: la[[0, 5]], 1: lb[[3]], 2: torch.stack([lb[4], la[9]])}
    for n, w in want.items():
        got = torch.from_numpy(np.fromfile(out / f"{n}.f32", dtype="<f4").reshape(-1, 50))
        assert U.rel_err(got, w.float()) < 2e-4
