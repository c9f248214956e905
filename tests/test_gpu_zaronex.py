"""The Zaronex design (pre-norm layers with a learned average over the depth; biased rotary attention over a window and the
pooled blocks before it beside a gated linear attention; jointly normed windowed attention with rotated values beside a
Mamba scan; windowed latent attention with a query latent) on the GPU against the plain CPU implementation in
oracle/zaronex.py.

Every test makes its own small configuration and random weights. fp32 weights are compared tightly (the kernels then
run plain fp32); bf16 weights within the noise of bf16 operands. Schedules (whole prompt, token by token, portions,
batches, reused slots) must not change a position's logits beyond rounding. Where random weights would hide a fault
(a key at a window's or block's edge, the sink, a rotation, a token the state must keep) the operation is called on
crafted inputs.
"""

import json
import math
from pathlib import Path

import pytest
import torch
from torch.overrides import TorchFunctionMode

pytestmark = pytest.mark.gpu

from oracle import zaronex as orc  # noqa: E402

D = torch.float64


# ------------------------------------------------------------------------------------------------ configurations
def pooled(heads=4, kv_heads=2, dim=8, vdim=12, rot=6, base=50.0, size=9, pool=4, scale=None, factor=None, rheads=3, rdim=12,
           rvdim=8, tau=7.0):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
            "mask": {"size": size}}
    if pool:
        left["mask"]["pool"] = pool
    if rot:
        left["rot"] = {"dims": rot, "base": base}
        if factor:
            left["rot"]["scaling"] = {"factor": factor}
    return {"type": "parallel", "mixer": {"left": left, "right": {"heads": rheads, "dim": rdim, "vdim": rvdim, "tau": tau}}}


def rotval(heads=4, kv_heads=2, dim=12, vdim=6, rot=8, base=30.0, factor=3.0, size=7, scale=None, inner=20, state=5, rank=3,
           conv=4):
    left = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": vdim, "scale": dim ** -0.5 if scale is None else scale,
            "mask": {"size": size}, "rot": {"dims": rot, "base": base}}
    if factor:
        left["rot"]["scaling"] = {"factor": factor}
    return {"type": "parallel_2", "mixer": {"left": left, "right": {"inner": inner, "state": state, "dt_rank": rank,
                                                                   "conv": conv}}}


def latent(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=24, q_rank=18, base=40.0, size=11, scale=0.3):
    return {"type": "latent_attention",
            "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim, "kv_rank": kv_rank, "q_rank": q_rank,
                      "rot": {"dims": rot_dim, "base": base}, "scale": scale, "mask": {"size": size}}}


def dense(ff=28):
    return {"kind": "dense", "ff": ff}


def make_cfg(layers, width=40, vocab=53, eps=1e-5):
    return {"architecture": "Zaronex", "vocab": vocab, "width": width, "norm": {"eps": eps},
            "layers": [dict(l[0], mlp=l[1]) for l in layers]}


MIXED = [(latent(), dense()), (pooled(), dense(ff=20)), (rotval(), None),
         (pooled(heads=6, kv_heads=1, dim=10, vdim=4, rot=10, size=17, pool=5, rheads=2, rdim=6, rvdim=20), dense()),
         (rotval(heads=3, kv_heads=3, dim=6, vdim=8, rot=6, factor=None, size=33, inner=33, state=18, rank=8, conv=2), dense(ff=12))]


def build(cfg, dtype=torch.float32, seed=0, edit=None):
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT

    config = LayeredConfig.from_dict(cfg)
    weights = LayeredGPT.random_weights(config, seed=seed)
    if edit:
        edit(weights)
    model = LayeredGPT(config, weights, device=torch.device("cuda", 0), dtype=dtype)
    return model, weights


def tokens_of(n, vocab, seed=0):
    g = torch.Generator().manual_seed(3000 + seed)
    return torch.randint(0, vocab, (n,), generator=g).tolist()


def rel_err(got, want):
    """Per row: rms of the mean-free difference over the rms of the mean-free reference."""
    got, want = got.double().cpu(), want.double().cpu()
    d = got - want
    d = d - d.mean(-1, keepdim=True)
    w = want - want.mean(-1, keepdim=True)
    return d.pow(2).mean(-1).sqrt() / w.pow(2).mean(-1).sqrt().clamp_min(1e-9)


def engine_logits(model, seqs, cuts, max_seq=None, engine=None):
    """Run sequences together through the BatchEngine: ``cuts[i]`` lists how many tokens request i brings per step
    (0: it sits the step out). Returns the logits of every position per request."""
    from generate.batch import BatchEngine

    eng = engine or BatchEngine(model, max_seq_length=max_seq or max(len(s) for s in seqs), slots=1)
    out = [[] for _ in seqs]
    at = [0] * len(seqs)
    ids = [object() for _ in seqs]
    for step in range(max(len(c) for c in cuts)):
        entries, who, end = [], [], []
        for i, s in enumerate(seqs):
            n = cuts[i][step] if step < len(cuts[i]) else 0
            if n:
                entries.append((ids[i], s[at[i]:at[i] + n], list(range(n))))
                who.append((i, n))
                at[i] += n
                if at[i] == len(s):
                    end.append(ids[i])
        lg = eng.step(entries, end)
        row = 0
        for i, n in who:
            out[i].append(lg[row:row + n].cpu())
            row += n
    assert all(a == len(s) for a, s in zip(at, seqs))
    return [torch.cat(o) for o in out]


class RoundedOperands(TorchFunctionMode):
    """Rounds both operands of every matrix product to bf16: what rounding alone does to the plain implementation."""

    def __torch_function__(self, func, types, args=(), kwargs=None):
        if getattr(func, "__name__", "") in ("matmul", "__matmul__") and args[0].dim() == 2 and args[1].dim() == 2:
            args = tuple(a.to(torch.bfloat16).to(a.dtype) for a in args)
        return func(*args, **(kwargs or {}))


def bf16_tolerance(cfg, w, toks, want):
    """Three times the worst row error that bf16 operands alone cause (a random model's norms of small branch outputs
    amplify rounding by their own measure), at least TOL16 / 2."""
    with RoundedOperands():
        got = orc.forward(cfg, w, toks)
    return max(TOL16 / 2, 3.0 * float(rel_err(got, want).max()))


def portions(n, size):
    return [size] * (n // size) + ([n % size] if n % size else [])


TOL32, TOL16, SAME = 2e-4, 6e-2, 6e-5


def only(side):
    """An edit of the weights that silences one branch of every pair (its output norm's weight becomes zero)."""
    def edit(w):
        for k in w:
            if k.endswith(f"{side}.out"):
                w[k] = torch.zeros_like(w[k])
    return edit


# ------------------------------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("layers,edit", [
    ([(pooled(), None)], None),
    ([(pooled(), None)], only("right")),
    ([(pooled(), None)], only("left")),
    ([(pooled(heads=3, kv_heads=3, dim=16, vdim=136, rot=16, size=1, pool=1), None)], only("right")),  # own token + every one
    ([(pooled(heads=6, kv_heads=2, dim=6, vdim=3, rot=0, size=5, pool=7), None)], only("right")),  # no rotation, blocks > window
    ([(pooled(heads=2, kv_heads=1, dim=132, vdim=20, rot=64, size=16, pool=16), None)], only("right")),
    ([(pooled(size=6, pool=0, factor=2.5), None)], only("right")),  # a plain window
    ([(pooled(size=200, pool=8), None)], only("right")),  # a window longer than the sequence
    ([(pooled(rheads=1, rdim=5, rvdim=3, tau=1.0), None)], only("left")),
    ([(pooled(rheads=2, rdim=132, rvdim=70, tau=30.0), None)], only("left")),
    ([(rotval(), None)], None),
    ([(rotval(), None)], only("right")),
    ([(rotval(), None)], only("left")),
    ([(rotval(heads=6, kv_heads=1, dim=6, vdim=130, rot=2, factor=None, size=1), None)], only("right")),
    ([(rotval(heads=2, kv_heads=2, dim=64, vdim=2, rot=64, factor=8.0, size=300), None)], only("right")),
    ([(rotval(inner=1, state=1, rank=1, conv=1), None)], only("left")),
    ([(rotval(inner=70, state=16, rank=8, conv=3), None)], only("left")),
    ([(rotval(inner=136, state=40, rank=24, conv=7), None)], only("left")),
    ([(rotval(inner=12, state=200, rank=5, conv=16), None)], only("left")),
    ([(latent(), None)], None),
    ([(latent(heads=1, dim=5, rot_dim=2, vdim=1, kv_rank=7, q_rank=3, size=1), None)], None),
    ([(latent(heads=2, dim=16, rot_dim=8, vdim=24, kv_rank=64, q_rank=40, size=20), None)], None),  # 16-token tiles
    ([(latent(heads=4, dim=8, rot_dim=4, vdim=8, kv_rank=128, q_rank=8, size=300), None)], None),
    ([(latent(heads=2, dim=4, rot_dim=10, vdim=6, kv_rank=1000, q_rank=130, size=3), None)], None),
    ([(latent(), dense(ff=1))], None),
    ([(pooled(), dense(ff=50))], None),
])
def test_mechanism_against_plain(layers, edit):
    cfg = make_cfg(layers)
    model, w = build(cfg, seed=len(str(layers)), edit=edit)
    toks = tokens_of(70, cfg["vocab"], seed=3)
    want = orc.forward(cfg, w, toks)
    whole = engine_logits(model, [toks], [[len(toks)]])[0]
    assert rel_err(whole, want).max() < TOL32
    single = engine_logits(model, [toks], [[1] * len(toks)])[0]
    assert rel_err(single, want).max() < TOL32


def test_residual_after_every_layer():
    from lit_gpt.mixers import StepBatch

    cfg = make_cfg(MIXED)
    model, w = build(cfg, seed=1)
    toks = tokens_of(33, cfg["vocab"], seed=5)
    want, got = [], []
    orc.forward(cfg, w, toks, layers_out=want)
    model.set_kv_cache(1, 64)
    with torch.inference_mode():
        model._forward_sandwich(StepBatch.build([(0, 0, toks)], model.device), after_layer=lambda r, x: got.append(x.clone()))
    assert len(got) == len(want) == len(MIXED)
    for a, b in zip(got, want):
        assert (a.double().cpu() - b).abs().max() < 5e-5 * b.abs().max()


def test_depth_average_matters_and_reads_the_right_layers():
    """Weights that skip layers outright: the last layer hands on the embedding plus the first layer's result only."""
    def edit(w):
        n = max(int(k.split(".")[0][1:]) for k in w if k.endswith(".dwa"))
        w[f"l{n}.dwa"] = torch.zeros_like(w[f"l{n}.dwa"])
        w[f"l{n}.dwa"][0], w[f"l{n}.dwa"][1] = 1.0, -2.0

    cfg = make_cfg(MIXED)
    model, w = build(cfg, seed=8, edit=edit)
    toks = tokens_of(20, cfg["vocab"], seed=2)
    want = orc.forward(cfg, w, toks)
    assert rel_err(engine_logits(model, [toks], [[20]])[0], want).max() < TOL32
    assert rel_err(engine_logits(model, [toks], [[1] * 20])[0], want).max() < TOL32


@pytest.mark.parametrize("width,vocab", [(8, 11), (50, 33), (136, 260), (1100, 64)])
def test_other_widths(width, vocab):
    cfg = make_cfg(MIXED, width=width, vocab=vocab, eps=1e-6)
    model, w = build(cfg, seed=width)
    toks = tokens_of(31, vocab, seed=width)
    want = orc.forward(cfg, w, toks)
    assert rel_err(engine_logits(model, [toks], [[len(toks)]])[0], want).max() < TOL32
    assert rel_err(engine_logits(model, [toks], [[12] + [1] * 19])[0], want).max() < TOL32


@pytest.mark.parametrize("width,vocab", [(40, 53), (50, 300), (136, 70), (200, 97)])
def test_bf16_is_within_operand_noise_everywhere(width, vocab):
    """Every row within bf16 operand noise, also at widths and head sizes that are no multiples of the vector widths, as a
    whole prompt (MFMA tiles), in portions and token by token."""
    cfg = make_cfg(MIXED, width=width, vocab=vocab)
    model, w = build(cfg, dtype=torch.bfloat16, seed=5)
    toks = tokens_of(61, vocab, seed=3)
    want = orc.forward(cfg, w, toks)
    tol = bf16_tolerance(cfg, w, toks, want)
    for cuts in ([61], [40] + [1] * 21, [13, 9, 20, 19]):
        err = rel_err(engine_logits(model, [toks], [cuts])[0], want)
        assert err.max() < tol and err.median() < TOL16, cuts


# ------------------------------------------------------------------------------------------------ schedules
@pytest.fixture(scope="module")
def mixed():
    cfg = make_cfg(MIXED)
    model, w = build(cfg, seed=4)
    return cfg, model, w


@pytest.mark.parametrize("size", [2, 3, 4, 5, 7, 9, 16, 17, 64, 65])
def test_portions_of_a_prompt(mixed, size):
    cfg, model, _ = mixed
    toks = tokens_of(150, cfg["vocab"], seed=size)
    whole = engine_logits(model, [toks], [[len(toks)]])[0]
    cut = engine_logits(model, [toks], [portions(len(toks), size)])[0]
    assert rel_err(cut, whole).max() < SAME


def test_mixed_portions_then_decoding(mixed):
    cfg, model, w = mixed
    toks = tokens_of(90, cfg["vocab"], seed=77)
    whole = engine_logits(model, [toks], [[len(toks)]])[0]
    cut = engine_logits(model, [toks], [[1, 2, 30, 1, 1, 17, 9] + [1] * 29])[0]
    assert rel_err(cut, whole).max() < SAME
    assert rel_err(whole, orc.forward(cfg, w, toks)).max() < TOL32


def test_first_token_alone_and_single_token_request(mixed):
    cfg, model, w = mixed
    toks = tokens_of(6, cfg["vocab"], seed=31)
    want = orc.forward(cfg, w, toks)
    assert rel_err(engine_logits(model, [toks], [[1, 5]])[0], want).max() < TOL32
    one = toks[:1]
    assert rel_err(engine_logits(model, [one], [[1]])[0], orc.forward(cfg, w, one)).max() < TOL32


def test_batch_of_unequal_requests_against_each_alone(mixed):
    cfg, model, _ = mixed
    seqs = [tokens_of(n, cfg["vocab"], seed=n) for n in (70, 1, 33, 130, 8)]
    alone = [engine_logits(model, [s], [[len(s)]])[0] for s in seqs]
    # one prompt step for all (every request keeps its last tokens back), then decoded together; shorter ones end earlier
    keep = [5, 0, 9, 12, 2]
    cuts = [[len(s) - k] + [1] * k for s, k in zip(seqs, keep)]
    from generate.batch import BatchEngine

    eng = BatchEngine(model, max_seq_length=140, slots=2)  # grows in flight
    together = engine_logits(model, seqs, cuts, engine=eng)
    for a, b in zip(together, alone):
        assert rel_err(a, b).max() < SAME
    assert not eng.live


def test_prompts_beside_decoding_requests(mixed):
    """Steps that hold portions of one request and single tokens of others (the blocks that single tokens complete are
    then pooled by the prompt's launch)."""
    cfg, model, _ = mixed
    seqs = [tokens_of(n, cfg["vocab"], seed=300 + n) for n in (60, 41, 55)]
    alone = [engine_logits(model, [s], [[len(s)]])[0] for s in seqs]
    cuts = [[20] + [1] * 40, [0, 2, 0, 7, 1, 1] + [1] * 30, [0] * 10 + [16, 1, 16] + [1] * 22]
    together = engine_logits(model, seqs, cuts, max_seq=64)
    for a, b in zip(together, alone):
        assert rel_err(a, b).max() < SAME


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_many_sequences_decoded_together(dtype):
    """More than eight one-token rows in a step (the matrix-core products' row count, step sizes outside the scan's launch,
    the second stream) against each request alone."""
    cfg = make_cfg(MIXED, width=72)
    model, _ = build(cfg, dtype=dtype, seed=13)
    seqs = [tokens_of(5 + 3 * i, cfg["vocab"], seed=200 + i) for i in range(12)]
    alone = [engine_logits(model, [s], [[len(s) - 4] + [1] * 4])[0] for s in seqs]
    from generate.batch import BatchEngine

    eng = BatchEngine(model, max_seq_length=48, slots=3)
    together = engine_logits(model, seqs, [[len(s) - 4] + [1] * 4 for s in seqs], engine=eng)
    tol = SAME if dtype == torch.float32 else TOL16
    for a, b in zip(together, alone):
        assert rel_err(a, b).max() < tol


def test_slots_freed_and_used_again(mixed):
    cfg, model, _ = mixed
    from generate.batch import BatchEngine

    a, b, c = (tokens_of(n, cfg["vocab"], seed=50 + n) for n in (40, 25, 33))
    fresh = [engine_logits(model, [s], [[len(s)]])[0] for s in (a, b, c)]
    eng = BatchEngine(model, max_seq_length=64, slots=2)
    got_a, got_b = engine_logits(model, [a, b], [[30] + [1] * 10, [25]], engine=eng)
    got_c = engine_logits(model, [c], [[20, 13]], engine=eng)[0]  # lands in a slot that held another sequence
    got_b2 = engine_logits(model, [b], [[1] * 25], engine=eng)[0]
    for got, want in ((got_a, fresh[0]), (got_b, fresh[1]), (got_c, fresh[2]), (got_b2, fresh[1])):
        assert rel_err(got, want).max() < SAME


def test_long_decoding(mixed):
    cfg, model, w = mixed
    toks = tokens_of(330, cfg["vocab"], seed=8)
    want = orc.forward(cfg, w, toks)
    got = engine_logits(model, [toks], [[30] + [1] * 300])[0]
    assert rel_err(got, want).max() < 5e-4


# ------------------------------------------------------------------------------------------------ crafted: attention
def _tables(rows, slot, pos0, dev):
    from lit_gpt.mixers import StepBatch

    return StepBatch.build([(slot, pos0, [0] * rows)], dev)


def _cached(k, v, slot, cache_dtype, dev, slots=2, extra=3):
    """Caches (slots, T + extra, G, .) whose slot holds k, v and whose other rows are stale."""
    T = k.shape[0]
    ck = torch.full((slots, T + extra, *k.shape[1:]), 7.0, device=dev, dtype=cache_dtype)
    cv = torch.full((slots, T + extra, *v.shape[1:]), -9.0, device=dev, dtype=cache_dtype)
    ck[slot, :T], cv[slot, :T] = k.to(dev), v.to(dev)
    return ck, cv


@pytest.mark.parametrize("cache_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("size,pool", [(1, 0), (1, 1), (2, 3), (16, 16), (17, 5), (40, 8), (100, 64), (255, 16), (256, 2), (257, 0),
                                       (300, 16), (1000, 4)])
def test_keys_at_the_edges_of_windows_and_blocks(size, pool, cache_dtype):
    """Every key of head 0 is aligned with every query; one key (or whole block) at a time stands out: the last one in the
    window, the first one outside, the last block seen, the first not seen, the sequence's first token, the query's own.
    Values are near-one-hot by position, so a weight on a wrong key shows. As 16-query tiles and as one-token steps."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, H, G, d, dv = 330, 2, 1, 8, 6
    g = torch.Generator().manual_seed(size + pool)
    q = torch.zeros(T, H, d)
    q[..., 0] = 1.0
    q[:, 1] = torch.randn(T, d, generator=g)
    v = torch.randn(T, G, dv, generator=g).to(cache_dtype).float()
    sink = torch.tensor([-3.0, 1.0])
    i = T - 1
    nb = max(0, (i - size + 1)) // pool if pool else 0
    spots = {max(0, i - size + 1): 1, max(0, i - size): 1, 0: 1, i: 1}
    if pool and nb:
        spots[(nb - 1) * pool] = pool
        if (nb + 1) * pool <= T:
            spots[nb * pool] = pool
        spots[0] = pool
    for at, n in spots.items():
        k = 0.1 * torch.randn(T, G, d, generator=g)
        k[at:at + n, 0, 0] = 12.0
        k = k.to(cache_dtype).float()
        want = orc.window_attention(q.to(D), k.to(D), v.to(D), 1.0, size, pool, sink.to(D))
        ck, cv = _cached(k, v, 1, cache_dtype, dev)
        step = _tables(T, 1, 0, dev)
        pk = None
        if pool:
            pk = (torch.full((2, T // pool, G, d), 5.0, device=dev), torch.full((2, T // pool, G, dv), 5.0, device=dev))
            seq_ops.pool_blocks(ck, cv, pk, pool, step.seq_start, step.seq_slot, step.seq_pos0, T)
        kw = dict(H=H, G=G, d=d, dv=dv, scale=1.0, window=size, pooled=pk, pool=pool)
        qd = q.reshape(T, H * d).contiguous().to(dev)
        got = seq_ops.sinkattn(qd, 0, ck, cv, sink.to(dev), step.seq_start, step.seq_slot, step.seq_pos0, T, **kw)
        assert (got.cpu().to(D).view(T, H, dv) - want).abs().max() < 2e-5
        for p in (i, i - 1, min(size - 1, i), min(size, i), 0):
            one = _tables(1, 1, p, dev)
            for splits in (None, 1, 7):
                got = seq_ops.sinkattn(qd[p:p + 1].contiguous(), 0, ck, cv, sink.to(dev), one.seq_start, one.seq_slot,
                                       one.seq_pos0, 1, splits=splits, **kw)
                assert (got.cpu().to(D).view(H, dv) - want[p]).abs().max() < 2e-5, (at, p, splits)


def test_a_sink_takes_the_weight():
    """All scores at -40: with a sink of 0 the output vanishes; left out, it would be the mean of the values."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, d, dv = 40, 4, 4
    q, k, v = torch.zeros(T, d), torch.zeros(T, 1, d), torch.ones(T, 1, dv)
    q[:, 0], k[:, 0, 0] = 1.0, -40.0
    ck, cv = _cached(k, v, 0, torch.float32, dev, slots=1)
    step = _tables(T, 0, 0, dev)
    for sink, want in ((torch.zeros(1, device=dev), 0.0), (None, 1.0)):
        got = seq_ops.sinkattn(q.to(dev), 0, ck, cv, sink, step.seq_start, step.seq_slot, step.seq_pos0, T, H=1, G=1, d=d, dv=dv,
                               scale=1.0, window=8)
        assert (got - want).abs().max() < 1e-5


@pytest.mark.parametrize("cache_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("pool", [1, 3, 16, 50])
def test_pooled_blocks_are_means_of_the_cached_rows(pool, cache_dtype):
    """However the tokens arrive (one step, portions, one by one), complete blocks hold the mean of the rows as cached;
    incomplete ones and other slots are left alone."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, H, G, d, dv = 103, 2, 2, 6, 5
    g = torch.Generator().manual_seed(pool)
    proj = torch.randn(T, H * d + G * (d + dv), generator=g).to(dev)
    results = []
    for cuts in ([T], portions(T, 7), [50] + [1] * 53, [1] * T):
        ck = torch.zeros(2, T, G, d, device=dev, dtype=cache_dtype)
        cv = torch.zeros(2, T, G, dv, device=dev, dtype=cache_dtype)
        pk = (torch.full((2, max(1, T // pool), G, d), 5.0, device=dev), torch.full((2, max(1, T // pool), G, dv), 5.0, device=dev))
        at = 0
        for n in cuts:
            step = _tables(n, 1, at, dev)
            rows = proj[at:at + n].contiguous()
            seq_ops.normattn_prepare(rows, 0, H * d, H * d + G * d, ck, cv, step.slot, step.pos, H=H, G=G, d=d, dv=dv, eps=1e-5,
                                     norm=0, pooled=pk if n == 1 else None, pool=pool)
            if n > 1:
                seq_ops.pool_blocks(ck, cv, pk, pool, step.seq_start, step.seq_slot, step.seq_pos0, n)
            at += n
        assert (pk[0][0] == 5.0).all() and (pk[1][0] == 5.0).all()
        want_k = orc.pooled_blocks(ck[1].cpu().to(D), pool)
        want_v = orc.pooled_blocks(cv[1].cpu().to(D), pool)
        nb = want_k.shape[0]
        if nb:
            assert (pk[0][1, :nb].cpu().to(D) - want_k).abs().max() < 1e-6
            assert (pk[1][1, :nb].cpu().to(D) - want_v).abs().max() < 1e-6
        results.append(torch.cat([pk[0].flatten(), pk[1].flatten()]))
    assert all(torch.equal(r, results[0]) for r in results)


@pytest.mark.parametrize("layout", ["half", "interleaved"])
def test_joint_norm_rotation_layouts_and_rotated_values(layout):
    from lit_gpt import seq_ops
    from lit_gpt.config import RotarySpec

    dev = torch.device("cuda", 0)
    T, H, G, d, dv, rot, pos0, eps = 19, 6, 3, 10, 8, 6, 41, 1e-5
    g = torch.Generator().manual_seed(9)
    q, k, v = (torch.randn(T, n, generator=g) for n in (H * d, G * d, G * dv))
    qw, kw = 1.0 + 0.3 * torch.randn(H * d, generator=g), 1.0 + 0.3 * torch.randn(G * d, generator=g)
    rs = {"dims": rot, "base": 20.0, "scaling": {"factor": 2.5}}
    f, fv = orc.rot_frequencies(rs), orc.frequencies(dv, 20.0)
    spec = RotarySpec(rot, 20.0, {"factor": 2.5})
    assert f == pytest.approx(spec.inv_freq(), rel=1e-12)
    pos = [pos0 + t for t in range(T)]
    wq = orc.rotate(orc.rms_norm(q.to(D), qw.to(D), eps).view(T, H, d), pos, f, layout)
    wk = orc.rotate(orc.rms_norm(k.to(D), kw.to(D), eps).view(T, G, d), pos, f, layout)
    wv = orc.rotate(v.to(D).view(T, G, dv), pos, fv, layout)
    ck, cv = torch.zeros(1, 80, G, d, device=dev), torch.zeros(1, 80, G, dv, device=dev)
    proj = torch.cat([q, k, v], 1).to(dev)
    step = _tables(T, 0, pos0, dev)
    vf = torch.tensor(fv, device=dev, dtype=torch.float32)
    seq_ops.normattn_prepare(proj, 0, H * d, (H + G) * d, ck, cv, step.slot, step.pos, H=H, G=G, d=d, dv=dv, eps=eps, norm=2,
                             q_weight=qw.to(dev), k_weight=kw.to(dev),
                             inv_freq=torch.tensor(spec.inv_freq(), device=dev, dtype=torch.float32), rot_dims=rot,
                             interleaved=layout == "interleaved", v_freq=vf)
    assert (proj[:, :H * d].cpu().to(D).view(T, H, d) - wq).abs().max() < 2e-5
    assert (ck[0, pos0:pos0 + T].cpu().to(D) - wk).abs().max() < 2e-5
    assert (cv[0, pos0:pos0 + T].cpu().to(D) - wv).abs().max() < 2e-5
    # outputs are turned back by the query's position, whatever form and whatever gate follows
    gate = torch.randn(T, H * dv, generator=g)
    want = orc.rotate(orc.window_attention(wq, wk, wv, 0.3, 6), pos, fv, layout, -1.0) * torch.sigmoid(gate.to(D)).view(T, H, dv)
    rows = torch.cat([proj[:, :H * d], gate.to(dev)], 1).contiguous()
    kw2 = dict(H=H, G=G, d=d, dv=dv, scale=0.3, window=6, v_freq=vf, interleaved=layout == "interleaved", gate_off=H * d,
               gate_cols=dv)
    # (keys before pos0 are zeros of the cache: only rows whose window starts at pos0 or later are compared)
    got = seq_ops.sinkattn(rows, 0, ck, cv, None, step.seq_start, step.seq_slot, step.seq_pos0, T, **kw2)
    assert (got.cpu().to(D).view(T, H, dv) - want)[5:].abs().max() < 2e-5
    for t in (5, T - 1):
        one = _tables(1, 0, pos0 + t, dev)
        for splits in (1, 3):
            got = seq_ops.sinkattn(rows[t:t + 1].contiguous(), 0, ck, cv, None, one.seq_start, one.seq_slot, one.seq_pos0, 1,
                                   splits=splits, **kw2)
            assert (got.cpu().to(D).view(H, dv) - want[t]).abs().max() < 2e-5


@pytest.mark.parametrize("cache_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("r", [24, 64, 100, 192])
@pytest.mark.parametrize("size", [1, 3, 15, 16, 17, 31, 64, 500])
def test_latent_attention_window_edges(r, size, cache_dtype):
    """One cached row stands out: just inside and just outside the last query's window, the first row, its own."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, H, d, dr = 150, 2, 4, 6
    g = torch.Generator().manual_seed(r + size)
    qc = torch.zeros(T, H, r)
    qc[:, 0, 0] = 1.0
    qc[:, 1] = 0.2 * torch.randn(T, r, generator=g)
    q = torch.randn(T, H * (d + dr), generator=g)
    kr = torch.randn(T, dr, generator=g)
    i = T - 1
    for at in {max(0, i - size + 1), max(0, i - size), 0, i}:
        c = 0.1 * torch.randn(T, r, generator=g)
        c[at, 0] = 40.0
        c = c.to(cache_dtype).float()
        keys = torch.cat([c, kr], 1).to(D).unsqueeze(1)
        qf = torch.cat([qc, q.view(T, H, d + dr)[..., d:]], -1).to(D)
        want = orc.window_attention(qf, keys, c.to(D).unsqueeze(1), 0.5, size)
        cc = torch.full((2, T + 5, r), 3.0, device=dev, dtype=cache_dtype)
        ckr = torch.full((2, T + 5, dr), 3.0, device=dev)
        cc[1, :T], ckr[1, :T] = c.to(dev), kr.to(dev)
        step = _tables(T, 1, 0, dev)
        args = (qc.reshape(T, -1).contiguous().to(dev), q.to(dev), 0, cc, ckr, None)
        kw = dict(H=H, d=d, dr=dr, r=r, scale=0.5, window=size)
        for splits in (1, 3):
            got = seq_ops.latent_attention(*args, step.slot, step.pos, splits=splits, **kw)
            assert (got.cpu().to(D).view(T, H, r) - want).abs().max() < 5e-5 * 40
        if r % 64 == 0:
            got = seq_ops.latent_attention_tiles(*args, step.seq_start, step.seq_slot, step.seq_pos0, T, **kw)
            assert (got.cpu().to(D).view(T, H, r) - want).abs().max() < 5e-5 * 40


# ------------------------------------------------------------------------------------------------ crafted: the scan
@pytest.mark.parametrize("inner,N,rank", [(1, 1, 1), (7, 4, 3), (64, 8, 8), (130, 5, 16), (70, 16, 24), (96, 20, 5), (40, 33, 8),
                                          (33, 64, 70), (20, 100, 8), (12, 256, 6)])
@pytest.mark.parametrize("n,pos0,form", [(1, 0, "map"), (1, 9, "map"), (5, 3, "map"), (1, 4, "walk"), (37, 0, "walk"), (90, 2, "walk"),
                                         (1, 4, "chunks"), (64, 0, "chunks"), (65, 5, "chunks"), (200, 0, "chunks")])
def test_channel_scan_against_float64(inner, N, rank, n, pos0, form):
    """Two sequences (the second one token shorter, if it can be), one slot stale, from a stored state or a fresh start."""
    from lit_gpt import seq_ops
    from lit_gpt.mixers import StepBatch

    dev = torch.device("cuda", 0)
    g = torch.Generator().manual_seed(inner + N + n)
    ns = [n, max(1, n - 1)]
    T = sum(ns)
    x, z, bias = torch.randn(T, inner, generator=g), torch.randn(T, inner, generator=g), torch.randn(inner, generator=g) - 1.0
    bc = torch.randn(T, rank + 2 * N, generator=g)
    w_dt = torch.randn(inner, rank, generator=g) * rank ** -0.5
    A = -torch.exp(torch.randn(inner, N, generator=g))
    Dv = torch.randn(inner, generator=g)
    state = torch.randn(3, 1, N, inner, generator=g)
    raw = bc[:, :rank].to(D) @ w_dt.to(D).T + bias.to(D)
    want, finals, at = [], [], 0
    for b, m in enumerate(ns):
        s0 = state[2 - b, 0].T.to(D) if pos0 else None
        sl = slice(at, at + m)
        y, S = orc.channel_scan(x[sl].to(D), orc.softplus(raw[sl]), A.to(D), bc[sl, rank:rank + N].to(D), bc[sl, rank + N:].to(D),
                                Dv.to(D), s0)
        want.append(y * orc.silu(z[sl].to(D)))
        finals.append(S.T)
        at += m
    want = torch.cat(want)
    step = StepBatch.build([(2, pos0, [0] * ns[0]), (1, pos0, [0] * ns[1])], dev)
    st = state.clone().to(dev)
    a2 = (A.double() * math.log2(math.e)).t().float().contiguous().to(dev)
    proj = torch.cat([torch.zeros(T, 3), z], 1).to(dev)
    kw = dict(w_dt=w_dt.to(dev), dt_bias=bias.to(dev)) if form == "map" else dict(dt=raw.float().to(dev))
    got = seq_ops.channel_scan(x.to(dev), proj, 3, bc.to(dev), rank, a2, Dv.to(dev), st, step.seq_start, step.seq_slot,
                               step.seq_pos0, max_len=n, chunked=form == "chunks", **kw)
    scale = want.abs().max().clamp_min(1.0)
    assert (got.cpu().to(D) - want).abs().max() < 3e-5 * scale
    for b in range(2):
        assert (st[2 - b, 0].cpu().to(D) - finals[b]).abs().max() < 3e-5 * finals[b].abs().max().clamp_min(1.0)
    assert torch.equal(st[0].cpu(), state[0])  # the third slot is left alone
    half = seq_ops.channel_scan(x.to(dev), proj, 3, bc.to(dev), rank, a2, Dv.to(dev), state.clone().to(dev), step.seq_start,
                                step.seq_slot, step.seq_pos0, max_len=n, chunked=form == "chunks", bf16=True, **kw)
    assert torch.equal(half, got.to(torch.bfloat16))


def test_states_keep_the_first_tokens():
    """Decays of nearly one in both recurrences: what the first tokens wrote must still be read 150 positions later, in
    every schedule and over a slot with stale contents. The attention branches are silent."""
    def edit(w):
        for k in w:
            if k.endswith("right.a2.b"):
                w[k] = torch.full_like(w[k], 30.0)  # sigmoid(30)^(1/tau) = 1
            if k.endswith("right.A_log"):
                w[k] = torch.full_like(w[k], -9.0)
            if k.endswith("left.out"):
                w[k] = torch.zeros_like(w[k])

    cfg = make_cfg([(pooled(), None), (rotval(inner=24, state=6), None)])
    model, w = build(cfg, seed=6, edit=edit)
    toks = tokens_of(150, cfg["vocab"], seed=1)
    other = [(toks[0] + 1) % cfg["vocab"]] + toks[1:]
    want, want_other = orc.forward(cfg, w, toks), orc.forward(cfg, w, other)
    assert rel_err(want[-1:], want_other[-1:]).max() > 1e-3  # the first token matters at the end
    from generate.batch import BatchEngine

    eng = BatchEngine(model, max_seq_length=150, slots=1)
    engine_logits(model, [other], [[150]], engine=eng)  # leaves the slot with another sequence's state
    for cuts in ([150], portions(150, 64), portions(150, 7), [100] + [1] * 50, [1] * 150):
        got = engine_logits(model, [toks], [cuts], engine=eng)[0]
        assert rel_err(got, want).max() < TOL32


# ------------------------------------------------------------------------------------------------ crafted: rows
@pytest.mark.parametrize("n", [8, 40, 320, 1100, 2500, 4100, 5000])
@pytest.mark.parametrize("prev", [1, 2, 5])
def test_boundary_launch_with_the_average_over_the_depth(n, prev):
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, eps = 5, 1e-5
    g = torch.Generator().manual_seed(n + prev)
    hist = torch.randn(prev + 1, T, n, generator=g)
    x0, y0, y1 = (torch.randn(T, n, generator=g) for _ in range(3))
    w0, w1, wn = (1.0 + 0.2 * torch.randn(n, generator=g) for _ in range(3))
    dwa = torch.randn(prev + 1, generator=g)
    for branches, coef in (([(y0, w0), (y1, w1)], 0.5), ([(y0, None)], 1.0)):
        s = sum(y.to(D) if w is None else orc.rms_norm(y.to(D), w.to(D), eps) for y, w in branches) * coef
        xn = x0.to(D) + s
        want = orc.depth_average([h.to(D) for h in hist[:prev]] + [xn], dwa.to(D))
        want_h = orc.rms_norm(want, wn.to(D), eps)
        for room in (prev + 1, prev):  # with and without a place for this layer's result
            hd = hist[:room].contiguous().to(dev)
            x = torch.full((T, n), 3.0, device=dev)
            h, h16 = seq_ops.sandwich_step(x, branches=[(y.to(dev), None if w is None else w.to(dev)) for y, w in branches],
                                           coef=coef, next_w=wn.to(dev), eps=eps, bf16_copy=True, x_in=x0.to(dev), hist=hd,
                                           depth_w=dwa.to(dev))
            assert (x.cpu().to(D) - want).abs().max() < 3e-5
            assert (h.cpu().to(D) - want_h).abs().max() < 3e-5
            assert torch.equal(h16.cpu(), h.cpu().to(torch.bfloat16))
            assert torch.equal(hd[:prev].cpu(), hist[:prev])
            if room > prev:
                assert (hd[prev].cpu().to(D) - xn).abs().max() < 2e-5
        # a boundary inside a layer: no average, no output norm
        x = x0.clone().to(dev)
        h, _ = seq_ops.sandwich_step(x, branches=[(y.to(dev), None if w is None else w.to(dev)) for y, w in branches], coef=coef,
                                     next_w=wn.to(dev), eps=eps)
        assert (x.cpu().to(D) - xn).abs().max() < 2e-5
        assert (h.cpu().to(D) - orc.rms_norm(xn, wn.to(D), eps)).abs().max() < 2e-5


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("M,N,K", [(1, 5, 8), (3, 4100, 16), (8, 40, 33), (9, 40, 33), (70, 130, 64), (200, 17, 40)])
def test_projection_with_a_bias(M, N, K, dtype):
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    g = torch.Generator().manual_seed(M + N)
    a = torch.randn(M, K, generator=g).to(dtype).float()
    w = (torch.randn(N, K, generator=g) * K ** -0.5).to(dtype)
    b = torch.randn(N, generator=g)
    want = a.to(D) @ w.to(D).T + b.to(D)
    y = torch.empty(M, N, device=dev)
    seq_ops.linear(a.to(dev), w.to(dev), M=M, N=N, K=K, y=y, lda=K, ldy=N, bias=b.to(dev))
    assert (y.cpu().to(D) - want).abs().max() < 1e-5 * K
    seq_ops.linear(a.to(dev), w.to(dev), M=M, N=N, K=K, y=y, lda=K, ldy=N, bias=b.to(dev), act=seq_ops.ACT_SILU)
    assert (y.cpu().to(D) - orc.silu(want)).abs().max() < 1e-5 * K


@pytest.mark.parametrize("M,N,K", [(9, 33, 1000), (130, 20, 520), (70, 260, 64), (300, 5, 2048)])
@pytest.mark.parametrize("ksplit", [2, 3, 16])
def test_thin_product_over_ranges_of_k(M, N, K, ksplit):
    """Ranges of K side by side: the plain product with bias, activation, accumulation and bf16 operands and results."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    g = torch.Generator().manual_seed(M + N + ksplit)
    a = torch.randn(M, K, generator=g).to(torch.bfloat16)
    w = (torch.randn(N, K, generator=g) * K ** -0.5).to(torch.bfloat16)
    b = torch.randn(N, generator=g)
    want = a.to(D) @ w.to(D).T + b.to(D)
    kw = dict(M=M, N=N, K=K, lda=K, ldy=N, bias=b.to(dev), ksplit=ksplit)
    y = torch.full((M, N), 2.0, device=dev)
    seq_ops.linear(a.float().to(dev), w.to(dev), y=y, accumulate=True, **kw)
    assert (y.cpu().to(D) - 2.0 - want).abs().max() < 2e-5
    y16 = torch.empty(M, N, device=dev, dtype=torch.bfloat16)
    seq_ops.linear(a.to(dev), w.to(dev), y=y16, act=seq_ops.ACT_SILU, **kw)
    assert (y16.cpu().to(D) - orc.silu(want)).abs().max() < 4e-2


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("M", [1, 2, 3, 8])
@pytest.mark.parametrize("N,K", [(1, 1024), (160, 4096), (512, 1032), (77, 2051)])
def test_short_deep_products_of_few_rows(M, N, K, dtype):
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    g = torch.Generator().manual_seed(M + N)
    a = torch.randn(M, K, generator=g).to(dtype).float()
    w = (torch.randn(N, K, generator=g) * K ** -0.5).to(dtype)
    b = torch.randn(N, generator=g)
    y = torch.full((M, N), 1.0, device=dev)
    seq_ops.linear(a.to(dev), w.to(dev), M=M, N=N, K=K, y=y, lda=K, ldy=N, bias=b.to(dev), accumulate=True)
    assert (y.cpu().to(D) - 1.0 - a.to(D) @ w.to(D).T - b.to(D)).abs().max() < 3e-5


# ------------------------------------------------------------------------------------------------ entry points
def follows_plain_greedy(cfg, w, prompt, out, margin=1e-3):
    """Every generated token is the plain implementation's argmax given the tokens before it (or within a rounding
    margin of it)."""
    lg = orc.forward(cfg, w, out[:-1])
    for i in range(len(prompt), len(out)):
        row = lg[i - 1]
        if row[out[i]] < row.max() - margin * row.abs().max():
            return False
    return True


def test_greedy_generation_through_the_entry_points():
    from generate.base import generate
    from generate.batch import BatchEngine

    cfg = make_cfg(MIXED)
    model, w = build(cfg, seed=7)
    prompts = [tokens_of(9, cfg["vocab"], seed=1), tokens_of(4, cfg["vocab"], seed=2), tokens_of(15, cfg["vocab"], seed=3)]
    new = 20
    eng = BatchEngine(model, max_seq_length=40)
    batched = eng.generate(prompts, new)
    assert not eng.live
    for p, out in zip(prompts, batched):
        assert out[:len(p)] == p and len(out) == len(p) + new
        assert follows_plain_greedy(cfg, w, p, out)
    assert BatchEngine(model, max_seq_length=40).generate(prompts, new, use_graph=True) == batched
    model.set_kv_cache(1, 40)
    single = generate(model, torch.tensor(prompts[0], dtype=torch.int32, device="cuda"), len(prompts[0]) + new,
                      temperature=0.0).cpu().tolist()
    assert single == batched[0]
    sampled = BatchEngine(model, max_seq_length=40).generate(prompts, 3, temperature=0.8, top_k=5)
    assert [len(o) for o in sampled] == [len(p) + 3 for p in prompts]


def test_captured_decode_step_replays():
    """One-token steps as replays of one HIP graph (blocks completed and windows passed on the way), every replay against
    the eager step, with eager work between."""
    from generate.batch import BatchEngine

    cfg = make_cfg(MIXED)
    model, _ = build(cfg, seed=21)
    prompts = [tokens_of(11, cfg["vocab"], seed=4), tokens_of(3, cfg["vocab"], seed=5)]
    eager = BatchEngine(model, max_seq_length=60).generate(prompts, 32)
    eng = BatchEngine(model, max_seq_length=60)
    ids = ["a", "b"]
    lg = eng.step([(ids[i], p, [len(p) - 1]) for i, p in enumerate(prompts)])
    first = [int(lg[i].argmax()) for i in range(2)]
    graph = eng.decode_graph(ids, first)
    outs = [list(p) + [first[i]] for i, p in enumerate(prompts)]
    for n in range(31):
        drawn = graph.step().cpu().tolist()
        torch.cuda.synchronize()
        (torch.randn(64, 64, device="cuda") @ torch.randn(64, 64, device="cuda")).sum().item()  # other eager work
        for i in range(2):
            outs[i].append(drawn[i])
    assert outs == eager


def test_command_line_serves_a_checkpoint_folder(tmp_path, capsys):
    from safetensors.torch import save_file

    from generate.base import main
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT

    cfg = make_cfg(MIXED, vocab=70)
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=15)
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    main(checkpoint_dir=tmp_path, max_new_tokens=5, temperature=0.0, top_k=None, prompt_len=7, precision="32-true")
    ids = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert len(ids) == 12
    assert follows_plain_greedy(cfg, w, ids[:7], ids)


def test_two_streams_against_one():
    from lit_gpt.mixers import ParallelMixer

    cfg = make_cfg(MIXED)
    model, _ = build(cfg, seed=2)
    toks = tokens_of(80, cfg["vocab"], seed=6)
    both = engine_logits(model, [toks], [[len(toks)]])[0]
    ParallelMixer.overlap = False
    try:
        one = engine_logits(model, [toks], [[len(toks)]])[0]
    finally:
        ParallelMixer.overlap = True
    assert torch.equal(both, one)


def test_checkpoint_folder_through_registry_and_runner(tmp_path):
    import subprocess
    import sys

    import numpy as np
    from safetensors.torch import save_file

    from lit_gpt.config import LayeredConfig, load_config, model_class
    from lit_gpt.layered import LayeredGPT

    REPO = Path(__file__).resolve().parent.parent
    for dtype, width in (("float32", 40), ("bfloat16", 136)):
        cfg = make_cfg(MIXED, width=width)
        weights = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=11)
        folder = tmp_path / dtype
        folder.mkdir()
        (folder / "config.json").write_text(json.dumps(cfg))
        save_file({k: v.contiguous() for k, v in weights.items()}, str(folder / "model.safetensors"))
        config = load_config(folder)
        assert model_class(config) is LayeredGPT
        a, b = tokens_of(14, cfg["vocab"], seed=1), tokens_of(6, cfg["vocab"], seed=2)
        steps = [{"step": 0, "entries": [{"id": "a", "tokens": a[:10], "want": [3, 9]}, {"id": "b", "tokens": b[:5], "want": []}], "end": []},
                 {"step": 1, "entries": [{"id": "a", "tokens": a[10:11], "want": [0]}, {"id": "b", "tokens": b[5:], "want": [0]}], "end": ["b"]},
                 {"step": 2, "entries": [{"id": "a", "tokens": a[11:12], "want": []}], "end": []},
                 {"step": 3, "entries": [{"id": "a", "tokens": a[12:], "want": [1]}], "end": ["a"]}]
        out = folder / "out"
        r = subprocess.run([sys.executable, str(REPO / "bin" / "trace_run"), "--model", str(folder), "--dtype", dtype,
                            "--out", str(out), "--max-tokens", "32"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                           capture_output=True, text=True, timeout=300)
        assert r.returncode == 0, r.stderr[-2000:]
        assert [l for l in r.stdout.split("\n") if l.startswith("done")] == [f"done {i}" for i in range(4)]
        la, lb = orc.forward(cfg, weights, a), orc.forward(cfg, weights, b)
        got0 = torch.from_numpy(np.fromfile(out / "0.f32", dtype="<f4").reshape(2, -1))
        got1 = torch.from_numpy(np.fromfile(out / "1.f32", dtype="<f4").reshape(2, -1))
        got3 = torch.from_numpy(np.fromfile(out / "3.f32", dtype="<f4").reshape(1, -1))
        assert not (out / "2.f32").exists()
        tol = TOL32 if dtype == "float32" else max(bf16_tolerance(cfg, weights, t, lt) for t, lt in ((a, la), (b, lb)))
        assert rel_err(got0, la[[3, 9]]).max() < tol
        assert rel_err(got1, torch.stack([la[10], lb[5]])).max() < tol
        assert rel_err(got3, la[13:14]).max() < tol
