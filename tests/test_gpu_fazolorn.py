"""The Fazolorn design (pre-norm layers that run several passes over a looped range; minGRU, sigmoid-weighted attention in
aligned chunks whose values are its keys, latent attention with a query latent and YaRN positions; clamped dense and
group-routed expert feed-forwards) on the GPU against the plain CPU implementation in oracle/fazolorn.py.

Every test makes its own small configuration and random weights. fp32 weights are compared tightly (the kernels then
run plain fp32); bf16 weights within the noise of bf16 operands. Schedules (whole prompt, token by token, portions,
batches, reused slots) must not change a position's logits beyond rounding. Where random weights would hide a fault
(a key at a chunk's edge, a far key, a group left out, a token the state must keep) the operation is called on crafted
inputs.
"""

import json
from pathlib import Path

import pytest
import torch
from torch.overrides import TorchFunctionMode

pytestmark = pytest.mark.gpu

from oracle import fazolorn as orc  # noqa: E402

D = torch.float64


# ------------------------------------------------------------------------------------------------ configurations
def gru(width=36):
    return {"type": "mingru", "mixer": {"width": width}}


def sig(heads=4, kv_heads=2, dim=12, rot=8, base=50.0, size=9, scale=None):
    m = {"heads": heads, "kv_heads": kv_heads, "dim": dim, "vdim": dim, "scale": dim ** -0.5 if scale is None else scale}
    if size:
        m["mask"] = {"size": size}
    if rot:
        m["rot"] = {"dims": rot, "base": base}
    return {"type": "attention", "mixer": m}


YARN = {"factor": 4.0, "original": 64, "fast": 8.0, "slow": 1.0}


def latent(heads=3, dim=10, rot_dim=6, vdim=7, kv_rank=24, q_rank=18, base=40.0, scale=0.3, scaling=YARN):
    rot = {"dims": rot_dim, "base": base}
    if scaling:
        rot["scaling"] = scaling
    return {"type": "latent_attention", "mixer": {"heads": heads, "dim": dim, "rot_dim": rot_dim, "vdim": vdim,
                                                  "kv_rank": kv_rank, "q_rank": q_rank, "rot": rot, "scale": scale}}


def dense(ff=28, limit=1.5):
    return {"kind": "dense", "ff": ff, "limit": limit}


def moe(ff=12, experts=12, top=3, count=4, keep=2, scale=1.7):
    return {"kind": "moe", "expert": {"ff": ff}, "router": {"experts": experts, "top": top, "scale": scale,
                                                           "groups": {"count": count, "keep": keep}}}


def make_cfg(layers, width=40, vocab=53, eps=1e-5, loop=None, logit_scale=0.7):
    cfg = {"architecture": "Fazolorn", "vocab": vocab, "width": width, "norm": {"eps": eps}, "logit_scale": logit_scale,
           "layers": [dict(l[0], mlp=l[1]) for l in layers]}
    if loop:
        cfg["loop"] = dict(zip(("start", "stop", "times"), loop))
    return cfg


MIXED = [(sig(), moe()), (gru(), dense()), (latent(), None), (gru(width=21), moe(ff=5, experts=9, top=4, count=3, keep=2)),
         (sig(heads=3, kv_heads=3, dim=10, rot=10, size=32), dense(ff=20, limit=0.6))]
LOOP = (1, 4, 2)


def build(cfg, dtype=torch.float32, seed=0, edit=None):
    from lit_gpt.config import LayeredConfig
    from lit_gpt.layered import LayeredGPT

    config = LayeredConfig.from_dict(cfg)
    weights = LayeredGPT.random_weights(config, seed=seed)
    if edit:
        edit(weights)
    model = LayeredGPT(config, weights, device=torch.device("cuda", 0), dtype=dtype)
    return model, weights


def plain_choices(weights):
    """Corrections so far apart that they alone decide which experts are chosen (rounding then flips no choice)."""
    for k in weights:
        if k.endswith("correction"):
            n = weights[k].numel()
            g = torch.Generator().manual_seed(n)
            weights[k] = (2.0 * torch.randperm(n, generator=g) - n).to(torch.bfloat16)


def tokens_of(n, vocab, seed=0):
    g = torch.Generator().manual_seed(4000 + seed)
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
        if getattr(func, "__name__", "") in ("matmul", "__matmul__") and min(args[0].dim(), args[1].dim()) >= 1:
            args = tuple(a.to(torch.bfloat16).to(a.dtype) for a in args)
        return func(*args, **(kwargs or {}))


def bf16_tolerance(cfg, w, toks, want):
    """Three times the worst row error that bf16 operands alone cause, at least TOL16 / 2."""
    with RoundedOperands():
        got = orc.forward(cfg, w, toks)
    return max(TOL16 / 2, 3.0 * float(rel_err(got, want).max()))


def portions(n, size):
    return [size] * (n // size) + ([n % size] if n % size else [])


TOL32, TOL16, SAME = 2e-4, 6e-2, 6e-5


# ------------------------------------------------------------------------------------------------ mechanisms alone
@pytest.mark.parametrize("layers", [
    [(gru(), None)],
    [(gru(width=1), None)],
    [(gru(width=300), None)],
    [(sig(), None)],
    [(sig(heads=1, kv_heads=1, dim=2, rot=2, size=1), None)],  # every position sees itself only
    [(sig(heads=6, kv_heads=2, dim=5, rot=0, size=2), None)],
    [(sig(heads=6, kv_heads=1, dim=20, rot=4, size=64), None)],
    [(sig(heads=2, kv_heads=2, dim=132, rot=132, size=33), None)],
    [(sig(size=0), None)],  # no chunks
    [(sig(size=500, scale=1.1), None)],  # a chunk longer than the sequence
    [(latent(), None)],
    [(latent(scaling=None), None)],
    [(latent(heads=1, dim=5, rot_dim=2, vdim=1, kv_rank=7, q_rank=3), None)],
    [(latent(heads=2, dim=16, rot_dim=8, vdim=24, kv_rank=64, q_rank=40), None)],  # 16-token tiles
    [(latent(heads=4, dim=8, rot_dim=32, vdim=8, kv_rank=128, q_rank=8, base=1e4,
             scaling={"factor": 30.0, "original": 40, "fast": 3.0, "slow": 0.2}), None)],
    [(latent(heads=2, dim=4, rot_dim=10, vdim=6, kv_rank=1000, q_rank=130,
             scaling={"factor": 0.5, "original": 4096, "fast": 32.0, "slow": 1.0}), None)],
    [(gru(width=8), dense())],
    [(gru(width=8), dense(ff=1, limit=0.2))],
    [(gru(width=8), moe())],
    [(gru(width=8), moe(ff=3, experts=4, top=4, count=1, keep=1))],  # one group, every expert
    [(gru(width=8), moe(ff=7, experts=6, top=2, count=6, keep=2, scale=1.0))],  # groups of one expert
    [(gru(width=8), moe(ff=16, experts=40, top=5, count=5, keep=1))],  # one group kept
    [(gru(width=8), moe(ff=8, experts=8, top=1, count=4, keep=3, scale=0.25))],
])
def test_mechanism_against_plain(layers):
    cfg = make_cfg(layers)
    model, w = build(cfg, seed=len(str(layers)))
    toks = tokens_of(70, cfg["vocab"], seed=3)
    want = orc.forward(cfg, w, toks)
    whole = engine_logits(model, [toks], [[len(toks)]])[0]
    assert rel_err(whole, want).max() < TOL32
    single = engine_logits(model, [toks], [[1] * len(toks)])[0]
    assert rel_err(single, want).max() < TOL32


@pytest.mark.parametrize("loop", [None, (0, 5, 1), (0, 5, 2), (0, 1, 3), (2, 5, 2), (4, 5, 4), (1, 4, 3)])
def test_looped_layers_and_the_residual_after_every_run(loop):
    from lit_gpt.mixers import StepBatch

    cfg = make_cfg(MIXED, loop=loop)
    model, w = build(cfg, seed=1)
    toks = tokens_of(33, cfg["vocab"], seed=5)
    want, got = [], []
    lg = orc.forward(cfg, w, toks, layers_out=want)
    model.set_kv_cache(1, 64)
    with torch.inference_mode():
        model._forward_sandwich(StepBatch.build([(0, 0, toks)], model.device), after_layer=lambda r, x: got.append(x.clone()))
    assert len(got) == len(want) == 5 + (0 if loop is None else (loop[1] - loop[0]) * (loop[2] - 1))
    for a, b in zip(got, want):
        assert (a.double().cpu() - b).abs().max() < 1e-4 * b.abs().max()
    assert rel_err(engine_logits(model, [toks], [[33]])[0], lg).max() < TOL32
    assert rel_err(engine_logits(model, [toks], [[20] + [1] * 13])[0], lg).max() < TOL32


@pytest.mark.parametrize("loop", [(0, 2, 3), (1, 2, 3)])
def test_what_joins_ahead_of_a_pass(loop):
    """Large vectors of the passes and a large embedding: a pass that misses either, or gets one twice, is far off."""
    def edit(w):
        w["loop.step"] = (10.0 * torch.randn(w["loop.step"].shape, generator=torch.Generator().manual_seed(3))).to(torch.bfloat16)
        w["embed"] = 30.0 * w["embed"]

    cfg = make_cfg([(gru(), None), (gru(width=9), dense())], loop=loop)
    model, w = build(cfg, seed=8, edit=edit)
    toks = tokens_of(20, cfg["vocab"], seed=2)
    want = orc.forward(cfg, w, toks)
    for t in range(3):
        without = dict(w)
        without["loop.step"] = w["loop.step"].clone()
        without["loop.step"][t] = 0.0
        assert rel_err(orc.forward(cfg, without, toks), want).max() > 1e-2
    assert rel_err(engine_logits(model, [toks], [[20]])[0], want).max() < TOL32
    assert rel_err(engine_logits(model, [toks], [[1] * 20])[0], want).max() < TOL32


def test_clamps_and_logit_scale():
    """Gate and up values far beyond the limit on either side."""
    def edit(w):
        for k in w:
            if k.endswith(("mlp.gate", "mlp.up")):
                w[k] = 6.0 * w[k]

    for scale in (1.0, -0.31, 20.0):
        cfg = make_cfg([(gru(), dense(limit=0.8)), (gru(width=50), dense(ff=70, limit=3.0))], logit_scale=scale)
        model, w = build(cfg, seed=5, edit=edit)
        toks = tokens_of(30, cfg["vocab"], seed=9)
        want = orc.forward(cfg, w, toks)
        got = engine_logits(model, [toks], [[30]])[0]
        assert rel_err(got, want).max() < TOL32
        assert (got.double() - want).abs().max() < 1e-3 * want.abs().max()


@pytest.mark.parametrize("width,vocab", [(8, 11), (50, 33), (136, 260), (1100, 64)])
def test_other_widths(width, vocab):
    cfg = make_cfg(MIXED, width=width, vocab=vocab, eps=1e-6, loop=LOOP)
    model, w = build(cfg, seed=width)
    toks = tokens_of(31, vocab, seed=width)
    want = orc.forward(cfg, w, toks)
    assert rel_err(engine_logits(model, [toks], [[len(toks)]])[0], want).max() < TOL32
    assert rel_err(engine_logits(model, [toks], [[12] + [1] * 19])[0], want).max() < TOL32


@pytest.mark.parametrize("width,vocab", [(40, 53), (50, 300), (136, 70), (200, 97)])
def test_bf16_is_within_operand_noise_everywhere(width, vocab):
    """Every row within bf16 operand noise, also at widths and head sizes that are no multiples of the vector widths, as a
    whole prompt (MFMA tiles), in portions and token by token."""
    cfg = make_cfg(MIXED, width=width, vocab=vocab, loop=LOOP)
    model, w = build(cfg, dtype=torch.bfloat16, seed=5, edit=plain_choices)
    toks = tokens_of(61, vocab, seed=3)
    want = orc.forward(cfg, w, toks)
    tol = bf16_tolerance(cfg, w, toks, want)
    for cuts in ([61], [40] + [1] * 21, [13, 9, 20, 19]):
        err = rel_err(engine_logits(model, [toks], [cuts])[0], want)
        assert err.max() < tol and err.median() < TOL16, cuts


# ------------------------------------------------------------------------------------------------ schedules
@pytest.fixture(scope="module")
def mixed():
    cfg = make_cfg(MIXED, loop=LOOP)
    model, w = build(cfg, seed=4)
    return cfg, model, w


@pytest.mark.parametrize("size", [2, 3, 4, 5, 7, 9, 16, 17, 32, 64, 65])
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
    """Steps that hold portions of one request and single tokens of others."""
    cfg, model, _ = mixed
    seqs = [tokens_of(n, cfg["vocab"], seed=300 + n) for n in (60, 41, 55)]
    alone = [engine_logits(model, [s], [[len(s)]])[0] for s in seqs]
    cuts = [[20] + [1] * 40, [0, 2, 0, 7, 1, 1] + [1] * 30, [0] * 10 + [16, 1, 16] + [1] * 22]
    together = engine_logits(model, seqs, cuts, max_seq=64)
    for a, b in zip(together, alone):
        assert rel_err(a, b).max() < SAME


@pytest.mark.parametrize("count", [8, 12, 20])
@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
def test_many_sequences_decoded_together(dtype, count):
    """Steps of 8 one-token rows (the last with the few-row kernels) and of more (matrix-core products, the recurrence from
    projected rows, sorted experts) against each request alone."""
    cfg = make_cfg(MIXED, width=72, loop=LOOP)
    model, _ = build(cfg, dtype=dtype, seed=13, edit=plain_choices)
    seqs = [tokens_of(5 + 3 * i, cfg["vocab"], seed=200 + i) for i in range(count)]
    alone = [engine_logits(model, [s], [[len(s) - 4] + [1] * 4])[0] for s in seqs]
    from generate.batch import BatchEngine

    eng = BatchEngine(model, max_seq_length=80, slots=3)
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
@pytest.mark.parametrize("size", [0, 1, 2, 15, 16, 17, 40, 64, 100, 255, 256, 257, 300, 1000])
def test_keys_at_the_edges_of_chunks(size, cache_dtype):
    """Nearly every key's weight vanishes; the weight of one at a time is nearly 1: the first of the last query's chunk, the
    last of the chunk before, the sequence's first, the query's own, the one before it. As tiles and as one-token steps."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, H, G, d, dv = 330, 4, 2, 8, 6
    g = torch.Generator().manual_seed(size)
    q = torch.zeros(T, H, d)
    q[..., 0] = 1.0
    q[:, 1::2] = torch.randn(T, H // 2, d, generator=g)
    v = torch.randn(T, G, dv, generator=g).to(cache_dtype).float()
    pb = torch.tensor([-14.0, 0.3, -14.0, -2.0])
    i = T - 1
    start = i - i % size if size else 0
    for at in {start, max(0, start - 1), 0, i, i - 1}:
        k = 0.1 * torch.randn(T, G, d, generator=g)
        k[at, :, 0] = 28.0
        k = k.to(cache_dtype).float()
        want = orc.sigmoid_attention(q.to(D), k.to(D), v.to(D), 1.0, size, pb.to(D))
        ck, cv = _cached(k, v, 1, cache_dtype, dev)
        step = _tables(T, 1, 0, dev)
        kw = dict(H=H, G=G, d=d, dv=dv, scale=1.0, chunk=size, score_bias=pb.to(dev))
        qd = q.reshape(T, H * d).contiguous().to(dev)
        tol = 2e-6 * float(want.abs().max()) + 1e-5
        got = seq_ops.sinkattn(qd, 0, ck, cv, None, step.seq_start, step.seq_slot, step.seq_pos0, T, **kw)
        assert (got.cpu().to(D).view(T, H, dv) - want).abs().max() < tol
        for p in {i, i - 1, min(max(size - 1, 0), i), min(size, i), 0}:
            one = _tables(1, 1, p, dev)
            for splits in (None, 1, 7, 64):
                got = seq_ops.sinkattn(qd[p:p + 1].contiguous(), 0, ck, cv, None, one.seq_start, one.seq_slot,
                                       one.seq_pos0, 1, splits=splits, **kw)
                assert (got.cpu().to(D).view(H, dv) - want[p]).abs().max() < tol, (at, p, splits)
        half = seq_ops.sinkattn(qd, 0, ck, cv, None, step.seq_start, step.seq_slot, step.seq_pos0, T, bf16_copy=True, **kw)
        full = seq_ops.sinkattn(qd, 0, ck, cv, None, step.seq_start, step.seq_slot, step.seq_pos0, T, **kw)
        assert torch.equal(half, full.to(torch.bfloat16))


def test_weights_are_not_normalised_and_saturate():
    """Scores and biases at either extreme: weights 0 and 1 each on its own, sums that grow with the keys."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, d = 300, 4
    q, k, v = torch.zeros(T, d), torch.zeros(T, 1, d), torch.ones(T, 1, d)
    q[:, 0], k[:, 0, 0] = 1.0, 200.0
    ck, cv = _cached(k, v, 0, torch.float32, dev, slots=1)
    step = _tables(T, 0, 0, dev)
    for bias, each in ((0.0, 1.0), (-200.0, 0.5), (-400.0, 0.0), (400.0, 1.0)):
        got = seq_ops.sinkattn(q.to(dev), 0, ck, cv, None, step.seq_start, step.seq_slot, step.seq_pos0, T, H=1, G=1, d=d, dv=d,
                               scale=1.0, score_bias=torch.tensor([bias], device=dev))
        want = each * torch.arange(1.0, T + 1)
        assert (got.cpu() - want.unsqueeze(1)).abs().max() < 1e-3
        one = _tables(1, 0, T - 1, dev)
        got = seq_ops.sinkattn(q[:1].to(dev), 0, ck, cv, None, one.seq_start, one.seq_slot, one.seq_pos0, 1, H=1, G=1, d=d,
                               dv=d, scale=1.0, score_bias=torch.tensor([bias], device=dev))
        assert (got.cpu() - each * T).abs().max() < 1e-3


def test_values_are_the_keys_before_rotation():
    from lit_gpt import seq_ops
    from lit_gpt.config import RotarySpec

    dev = torch.device("cuda", 0)
    T, H, G, d, rot, pos0 = 19, 6, 3, 10, 6, 41
    g = torch.Generator().manual_seed(9)
    q, k = torch.randn(T, H * d, generator=g), torch.randn(T, G * d, generator=g)
    rs = {"dims": rot, "base": 20.0, "scaling": YARN}
    f, mult = orc.rot_frequencies(rs)
    spec = RotarySpec(rot, 20.0, YARN)
    pos = [pos0 + t for t in range(T)]
    for m in (1.0, mult):
        wq = orc.rotate(q.to(D).view(T, H, d), pos, f, "half", m)
        wk = orc.rotate(k.to(D).view(T, G, d), pos, f, "half", m)
        ck, cv = torch.zeros(1, 80, G, d, device=dev), torch.zeros(1, 80, G, d, device=dev)
        proj = torch.cat([q, k], 1).to(dev)
        step = _tables(T, 0, pos0, dev)
        seq_ops.normattn_prepare(proj, 0, H * d, H * d, ck, cv, step.slot, step.pos, H=H, G=G, d=d, dv=d, eps=1e-5, norm=0,
                                 inv_freq=torch.tensor(spec.inv_freq(), device=dev, dtype=torch.float32), rot_dims=rot,
                                 rot_mult=m)
        assert (proj[:, :H * d].cpu().to(D).view(T, H, d) - wq).abs().max() < 2e-5
        assert (ck[0, pos0:pos0 + T].cpu().to(D) - wk).abs().max() < 2e-5
        assert torch.equal(cv[0, pos0:pos0 + T].cpu().reshape(T, -1), k)


@pytest.mark.parametrize("cache_dtype", [torch.float32, torch.bfloat16])
def test_latent_preparation_with_scaled_rotation(cache_dtype):
    from lit_gpt import seq_ops
    from lit_gpt.config import RotarySpec

    dev = torch.device("cuda", 0)
    T, H, d, dr, r, pos0, eps = 13, 3, 5, 8, 20, 700, 1e-5
    g = torch.Generator().manual_seed(4)
    q, kv = torch.randn(T, H * (d + dr), generator=g), torch.randn(T, r + dr, generator=g)
    nw = 1.0 + 0.3 * torch.randn(r, generator=g)
    sc = {"factor": 16.0, "original": 256, "fast": 16.0, "slow": 1.0}
    f, mult = orc.rot_frequencies({"dims": dr, "base": 500.0, "scaling": sc})
    spec = RotarySpec(dr, 500.0, sc)
    assert spec.inv_freq() == pytest.approx(f, rel=1e-12) and spec.mult == pytest.approx(mult, rel=1e-12) and mult > 1.2
    pos = [pos0 + t for t in range(T)]
    qh = q.to(D).view(T, H, d + dr)
    want_q = torch.cat([qh[..., :d], orc.rotate(qh[..., d:], pos, f, "interleaved", mult)], -1)
    want_c = orc.rms_norm(kv[:, :r].to(D), nw.to(D), eps)
    want_k = orc.rotate(kv[:, r:].to(D).view(T, 1, dr), pos, f, "interleaved", mult)[:, 0]
    cc, ckr = torch.zeros(2, 720, r, device=dev, dtype=cache_dtype), torch.zeros(2, 720, dr, device=dev)
    step = _tables(T, 1, pos0, dev)
    qd = q.to(dev)
    seq_ops.latent_prepare(qd, 0, kv.to(dev), 0, cc, ckr, nw.to(dev), torch.tensor(f, device=dev, dtype=torch.float32),
                           step.slot, step.pos, H=H, d=d, dr=dr, r=r, rot_dims=dr, eps=eps, rot_mult=spec.mult)
    assert (qd.cpu().to(D).view(T, H, d + dr) - want_q).abs().max() < 3e-4  # (angles of hundreds of radians in fp32)
    assert (ckr[1, pos0:pos0 + T].cpu().to(D) - want_k).abs().max() < 3e-4
    assert (cc[1, pos0:pos0 + T].cpu().to(D) - want_c).abs().max() < (1e-5 if cache_dtype == torch.float32 else 2e-2)


@pytest.mark.parametrize("cache_dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("r", [24, 64, 100, 192])
def test_latent_attention_far_and_near_keys(r, cache_dtype):
    """One cached row stands out: the sequence's first, rows at the borders of the 16-row tiles, the query's own. Every
    later query must see it, every earlier one must not."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, H, d, dr = 150, 2, 4, 6
    g = torch.Generator().manual_seed(r)
    qc = torch.zeros(T, H, r)
    qc[:, 0, 0] = 1.0
    qc[:, 1] = 0.2 * torch.randn(T, r, generator=g)
    q = torch.randn(T, H * (d + dr), generator=g)
    kr = torch.randn(T, dr, generator=g)
    for at in (0, 15, 16, 17, 63, 64, 128, T - 1):
        c = 0.1 * torch.randn(T, r, generator=g)
        c[at, 0] = 40.0
        c = c.to(cache_dtype).float()
        keys = torch.cat([c, kr], 1).to(D).unsqueeze(1).expand(T, H, r + dr)
        qf = torch.cat([qc, q.view(T, H, d + dr)[..., d:]], -1).to(D)
        want = orc.softmax_attention(qf, keys, c.to(D).unsqueeze(1).expand(T, H, r), 0.5)
        cc = torch.full((2, T + 5, r), 3.0, device=dev, dtype=cache_dtype)
        ckr = torch.full((2, T + 5, dr), 3.0, device=dev)
        cc[1, :T], ckr[1, :T] = c.to(dev), kr.to(dev)
        step = _tables(T, 1, 0, dev)
        args = (qc.reshape(T, -1).contiguous().to(dev), q.to(dev), 0, cc, ckr, None)
        kw = dict(H=H, d=d, dr=dr, r=r, scale=0.5)
        for splits in (1, 3):
            got = seq_ops.latent_attention(*args, step.slot, step.pos, splits=splits, **kw)
            assert (got.cpu().to(D).view(T, H, r) - want).abs().max() < 5e-5 * 40
        if r % 64 == 0:
            got = seq_ops.latent_attention_tiles(*args, step.seq_start, step.seq_slot, step.seq_pos0, T, **kw)
            assert (got.cpu().to(D).view(T, H, r) - want).abs().max() < 5e-5 * 40


# ------------------------------------------------------------------------------------------------ crafted: the recurrence
@pytest.mark.parametrize("n", [1, 7, 64, 255, 257, 600])
@pytest.mark.parametrize("rows,pos0,chunked", [(1, 0, False), (1, 9, False), (5, 3, False), (37, 0, False), (90, 2, False),
                                               (1, 4, True), (31, 0, True), (32, 5, True), (33, 5, True), (64, 0, True),
                                               (700, 1, True)])
def test_mingru_against_float64(n, rows, pos0, chunked):
    """Two sequences (the second one token shorter, if it can be), one slot stale, from a stored state or a fresh start;
    gates and candidates from saturated to small."""
    from lit_gpt import seq_ops
    from lit_gpt.mixers import StepBatch

    dev = torch.device("cuda", 0)
    g = torch.Generator().manual_seed(n + rows)
    ns = [rows, max(1, rows - 1)]
    T = sum(ns)
    z, u, gate = 3.0 * torch.randn(T, n, generator=g), 2.0 * torch.randn(T, n, generator=g), torch.randn(T, n, generator=g)
    z[::5], u[::7], u[::11] = -120.0, -90.0, 0.0
    z[3::17] = 120.0
    state = torch.randn(3, n, generator=g)
    want, finals, at = [], [], 0
    for b, m in enumerate(ns):
        sl = slice(at, at + m)
        S, last = orc.mingru_scan(z[sl].to(D), u[sl].to(D), state[2 - b].to(D) if pos0 else None)
        want.append(S * orc.silu(gate[sl].to(D)))
        finals.append(last)
        at += m
    want = torch.cat(want)
    step = StepBatch.build([(2, pos0, [0] * ns[0]), (1, pos0, [0] * ns[1])], dev)
    proj = torch.cat([u, torch.zeros(T, 5), z, gate], 1).to(dev)
    args = (proj, n + 5, 0, 2 * n + 5)
    kw = dict(max_len=rows, chunked=chunked)
    st = state.clone().to(dev)
    got = seq_ops.mingru(*args, st, step.seq_start, step.seq_slot, step.seq_pos0, **kw)
    assert (got.cpu().to(D) - want).abs().max() < 1e-5 * want.abs().max().clamp_min(1.0)
    for b in range(2):
        assert (st[2 - b].cpu().to(D) - finals[b]).abs().max() < 1e-5 * finals[b].abs().max().clamp_min(1.0)
    assert torch.equal(st[0].cpu(), state[0])  # the third slot is left alone
    half = seq_ops.mingru(*args, state.clone().to(dev), step.seq_start, step.seq_slot, step.seq_pos0, bf16=True, **kw)
    assert torch.equal(half, got.to(torch.bfloat16))


@pytest.mark.parametrize("dtype", [torch.float32, torch.bfloat16])
@pytest.mark.parametrize("M", [1, 2, 3, 5, 8])
@pytest.mark.parametrize("n,K", [(1, 8), (30, 40), (33, 33), (130, 1032)])
def test_mingru_step_with_its_projections(M, n, K, dtype):
    from lit_gpt import seq_ops
    from lit_gpt.mixers import StepBatch

    dev = torch.device("cuda", 0)
    g = torch.Generator().manual_seed(n + K + M)
    h = torch.randn(M, K, generator=g).to(dtype).float()
    rows = 3 * n + 10
    w = (torch.randn(rows, K, generator=g) * K ** -0.5).to(dtype)
    bias = torch.randn(rows, generator=g)
    state = torch.randn(M + 2, n, generator=g)
    z0, u0, g0 = 2 * n + 7, 3, n + 5
    y = h.to(D) @ w.to(D).T + bias.to(D)
    pos0 = [0 if m == 1 else 4 + m for m in range(M)]
    slots = [M + 1 - m for m in range(M)]
    step = StepBatch.build([(slots[m], pos0[m], [0]) for m in range(M)], dev)
    st = state.clone().to(dev)
    got = seq_ops.mingru_step(h.to(dev), w.to(dev), bias.to(dev), z0, u0, g0, st, step.seq_slot, step.seq_pos0)
    left = state.to(D).clone()
    for m in range(M):
        S, last = orc.mingru_scan(y[m:m + 1, z0:z0 + n], y[m:m + 1, u0:u0 + n], state[slots[m]].to(D) if pos0[m] else None)
        assert (got[m].cpu().to(D) - last * orc.silu(y[m, g0:g0 + n])).abs().max() < 2e-5
        left[slots[m]] = last
    assert (st.cpu().to(D) - left).abs().max() < 2e-5


def test_the_state_keeps_the_first_tokens():
    """Gates that are nearly shut: what the first tokens wrote must still be read 150 positions later, in every schedule and
    over a slot with stale contents."""
    def edit(w):
        for k in w:
            if k.endswith("mix.z.b"):
                w[k] = torch.full_like(w[k], -7.0)

    cfg = make_cfg([(gru(width=24), None), (gru(), dense())], loop=(0, 2, 2))
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


# ------------------------------------------------------------------------------------------------ crafted: routing
def _routed(z, corr, top, count, keep, scale):
    """(ids, weights) of both launches: from logits, and from a product with the identity."""
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, E = z.shape
    kw = dict(sigmoid=True, groups=count, keep=keep, scale=scale)
    proj = torch.cat([torch.full((T, 3), 99.0), z], 1).to(dev)
    a = seq_ops.moe_route_scores(proj, 3, E, top, corr.to(dev), **kw)
    b = seq_ops.moe_router(z.to(dev), torch.eye(E, device=dev), top, corr.to(dev), **kw)
    assert torch.equal(a[0], b[0]) and torch.equal(a[1], b[1])
    return a[0].cpu(), a[1].cpu()


@pytest.mark.parametrize("E,top,count,keep", [(4, 2, 2, 1), (12, 5, 4, 3), (16, 8, 8, 4), (9, 3, 3, 1), (6, 3, 6, 3), (64, 8, 8, 2),
                                              (100, 6, 20, 5), (130, 4, 65, 10), (256, 16, 32, 8), (256, 2, 256, 3),
                                              (250, 7, 1, 1), (20, 20, 4, 4)])
def test_group_routing_against_plain(E, top, count, keep):
    g = torch.Generator().manual_seed(E + top)
    z = 1.5 * torch.randn(50, E, generator=g)
    corr = torch.randn(E, generator=g) - 1.0  # (choice scores mostly negative)
    ids, wts = _routed(z, corr, top, count, keep, 1.3)
    for t in range(z.shape[0]):
        want = orc.route(z[t].to(D), corr.to(D), top, count, keep, 1.3)
        assert set(ids[t].tolist()) == set(want) and len(set(ids[t].tolist())) == top
        for e, wt in zip(ids[t].tolist(), wts[t].tolist()):
            assert wt == pytest.approx(want[e], rel=2e-5)


def test_groups_by_hand():
    """Three groups of three. Group 0 has the single best expert, group 1 the best pair, group 2 the best sum of three."""
    s = torch.tensor([[0.9, 0.05, 0.05, 0.6, 0.55, 0.01, 0.5, 0.5, 0.5]])
    z = torch.log(s / (1 - s))
    ids, wts = _routed(z, torch.zeros(9), 2, 3, 1, 2.0)
    assert ids.tolist() == [[3, 4]] and wts[0].tolist() == pytest.approx([1.2, 1.1], rel=1e-5)
    ids, _ = _routed(z, torch.zeros(9), 3, 3, 2, 2.0)  # the pairs 1.15, 1.0 stay, 0.95 goes
    assert ids.tolist() == [[3, 4, 6]]
    # a correction moves the choice, never the weight; choice scores below zero still win over experts of other groups
    corr = torch.full((9,), -3.0)
    corr[6:] = -2.0
    ids, wts = _routed(z, corr, 3, 3, 1, 1.0)
    assert sorted(ids[0].tolist()) == [6, 7, 8] and wts[0].tolist() == pytest.approx([0.5] * 3, rel=1e-5)


# ------------------------------------------------------------------------------------------------ crafted: rows
@pytest.mark.parametrize("n", [8, 40, 320, 1100, 2500, 4100, 5000])
def test_boundary_launch_ahead_of_a_pass(n):
    from lit_gpt import seq_ops

    dev = torch.device("cuda", 0)
    T, eps = 5, 1e-5
    g = torch.Generator().manual_seed(n)
    x0, y0, row = (torch.randn(T, n, generator=g) for _ in range(3))
    vec, wn = torch.randn(n, generator=g), 1.0 + 0.2 * torch.randn(n, generator=g)
    for branches in ([(y0, None)], []):
        for add in (None, row):
            for separate in (False, True):
                want = x0.to(D) + vec.to(D) + (y0.to(D) if branches else 0.0) + (add.to(D) if add is not None else 0.0)
                x = torch.full((T, n), 3.0, device=dev) if separate else x0.clone().to(dev)
                h, h16 = seq_ops.sandwich_step(x, branches=[(y.to(dev), None) for y, _ in branches], next_w=wn.to(dev), eps=eps,
                                               bf16_copy=True, x_in=x0.to(dev) if separate else None,
                                               add=None if add is None else add.to(dev), add_vec=vec.to(dev))
                assert (x.cpu().to(D) - want).abs().max() < 2e-5
                assert (h.cpu().to(D) - orc.rms_norm(want, wn.to(D), eps)).abs().max() < 3e-5
                assert torch.equal(h16.cpu(), h.cpu().to(torch.bfloat16))


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

    cfg = make_cfg(MIXED, loop=LOOP)
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
    """One-token steps as replays of one HIP graph (chunks passed on the way), every replay against the eager step, with
    eager work between."""
    from generate.batch import BatchEngine

    cfg = make_cfg(MIXED, loop=LOOP)
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

    cfg = make_cfg(MIXED, vocab=70, loop=LOOP)
    w = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=15)
    save_file({k: v.contiguous() for k, v in w.items()}, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    main(checkpoint_dir=tmp_path, max_new_tokens=5, temperature=0.0, top_k=None, prompt_len=7, precision="32-true")
    ids = json.loads(capsys.readouterr().out.strip().splitlines()[-1])
    assert len(ids) == 12
    assert follows_plain_greedy(cfg, w, ids[:7], ids)


def test_checkpoint_folder_through_registry_and_runner(tmp_path):
    import subprocess
    import sys

    import numpy as np
    from safetensors.torch import save_file

    from lit_gpt.config import LayeredConfig, load_config, model_class
    from lit_gpt.layered import LayeredGPT

    REPO = Path(__file__).resolve().parent.parent
    for dtype, width in (("float32", 40), ("bfloat16", 136)):
        cfg = make_cfg(MIXED, width=width, loop=LOOP)
        weights = LayeredGPT.random_weights(LayeredConfig.from_dict(cfg), seed=11)
        plain_choices(weights)
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
