"""Sandwich layers of the token language models on the GPU against the plain oracle (float64), fp32 and bf16."""
import json
import math

import pytest
import torch

from oracle import lm_oracle as O
from tests import lm_util as U

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
BOTH = pytest.mark.parametrize("dt", [F32, BF16])
TOL = {F32: 4e-5, BF16: 0.06}  # eight layer runs, every sublayer's output scaled up to unit size by its norm


def oracle(cfg, sd, toks):
    margins = []
    return O.forward(cfg, sd, toks, margins=margins), margins


def run_all(row, toks):
    return row.extend(toks, range(len(toks))).clone()


def attn_only(*a, **kw):
    return U.sandwich([(U.sig(*a, **kw), None)])


SINGLE = {
    "attention_grouped": lambda: attn_only(),
    "attention_one_group": lambda: attn_only(heads=5, kv_heads=1, dim=18, vdim=6),
    "attention_own_keys": lambda: attn_only(heads=3, kv_heads=3, dim=33, vdim=70),
    "attention_many_heads": lambda: attn_only(heads=40, kv_heads=2, dim=9, vdim=5),
    "attention_no_temperature": lambda: attn_only(q_temp=None),
    "attention_few_buckets": lambda: attn_only(buckets=2, bias_max=3),
    "attention_buckets_beyond_the_range": lambda: attn_only(buckets=40, bias_max=11),
    "attention_long_table": lambda: attn_only(buckets=30, bias_max=5000),
    "attention_wide": lambda: U.sandwich([(U.sig(heads=2, kv_heads=1, dim=130, vdim=200), None)], width=96),
    "attention_wider_than_the_matrix_form": lambda: U.sandwich([(U.sig(heads=2, kv_heads=1, dim=270, vdim=300), None)], width=96),
    "gla": lambda: U.sandwich([(U.gla(), None)]),
    "gla_strong_decay": lambda: U.sandwich([(U.gla(tau=0.2), None)]),
    "gla_one_head": lambda: U.sandwich([(U.gla(heads=1, dim=100, vdim=130, rank=1), None)]),
    "gla_wider_than_the_chunked_form": lambda: U.sandwich([(U.gla(heads=1, dim=270, vdim=300, rank=20), None)], width=96),
    "gla_small": lambda: U.sandwich([(U.gla(heads=7, dim=5, vdim=11, tau=30.0), None)]),
    "dense": lambda: U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.dense(150))]),
    "experts": lambda: U.sandwich([(U.sig(heads=1, kv_heads=1, dim=4, vdim=4), U.moe())]),
    "experts_one_choice": lambda: U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.moe(experts=5, top=1))]),
    "experts_all": lambda: U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.moe(ff=7, experts=4, top=4))]),
    "experts_many": lambda: U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.moe(ff=20, experts=75, top=6))]),
    "one_group_norm": lambda: U.sandwich([(U.sig(), U.dense()), (U.gla(), U.dense(30))], groups=1),
    "many_group_norm": lambda: U.sandwich([(U.sig(), U.dense()), (U.gla(), U.dense(30))], groups=10, scale=1.0),
    "loop_whole": lambda: U.sandwich([(U.sig(), U.dense()), (U.gla(), None)], loop=(0, 2, 3)),
    "loop_inside": lambda: U.sandwich([(U.gla(), None), (U.sig(), U.dense()), (U.sig(heads=2), U.dense(30))], loop=(1, 2, 2)),
    "loop_once_at_the_end": lambda: U.sandwich([(U.gla(), U.dense()), (U.sig(), None)], loop=(1, 2, 1)),
    "equal_sizes": lambda: U.sandwich([(U.sig(heads=2, kv_heads=2, dim=32, vdim=32, bias_max=32, buckets=32), U.dense(64)), (U.gla(heads=2, dim=32, vdim=32, rank=32), U.moe(ff=64, experts=2, top=1))],
                                      width=64, vocab=64, groups=2),
    "mixed": U.sandwich_mixed,
}


@BOTH
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_prompts_of_many_lengths(name, dt):
    """Each mechanism alone and together; lengths on both sides of every tile and chunk and of the switch to blocks."""
    cfg = SINGLE[name]()
    sd = U.sandwich_weights(cfg, 11)
    eng = U.engine(cfg, sd, dt, max_seq=160)
    for T in (1, 2, 5, 16, 17, 33, 64, 150):
        toks = U.tokens(T, cfg["vocab"], T)
        ref, margins = oracle(cfg, sd, toks)
        with eng.new_row() as row:
            got = run_all(row, toks)
        e = U.err_clear(got, ref, margins) if dt == BF16 and T > 16 else U.err(got, ref) if dt == F32 or not margins else 0.0
        assert e < TOL[dt], (name, T, e)


@BOTH
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_decoding_of_every_mechanism(name, dt):
    """Prompts of unequal lengths, then single tokens of all rows together: over tile, block and chunk borders."""
    cfg = SINGLE[name]()
    sd = U.sandwich_weights(cfg, 35)
    eng = U.engine(cfg, sd, dt, max_rows=4, max_seq=160)
    starts, n = (1, 13, 30, 125), 9
    seqs = [U.tokens(s + n, cfg["vocab"], s) for s in starts]
    rows = []
    for s, toks in zip(starts, seqs):
        rows.append(eng.new_row())
        rows[-1].extend(toks[:s])
    got = []
    for t in range(n):
        got.append(eng.decode_step(rows, torch.tensor([toks[s + t] for s, toks in zip(starts, seqs)], device="cuda")).clone())
    alone = [rows[1].extend([7 % cfg["vocab"]], [0]).clone()]  # and a row by itself
    for k, (s, toks) in enumerate(zip(starts, seqs)):
        ref, margins = oracle(cfg, sd, toks + [7 % cfg["vocab"]])
        mine = torch.stack([g[k] for g in got] + ([alone[0][0]] if k == 1 else []))
        for j in range(len(mine)):
            if dt == BF16 and any(m[s + j] < 0.05 for m in margins):
                continue  # a close call between experts
            e = U.err(mine[j:j + 1], ref[s + j:s + j + 1])
            assert e < TOL[dt], (name, s, j, e)


@BOTH
@pytest.mark.parametrize("width,groups", [(80, 16), (84, 4), (30, 3), (66, 1), (1100, 1), (1100, 4), (96, 24), (520, 2), (6, 2)])
def test_norms_of_many_shapes(width, groups, dt):
    """Parts that are no whole quads, that several waves share, and more parts than waves, with experts behind them: the
    router of one row, of few rows and of a prompt."""
    if dt == BF16 and width < 16:
        pytest.skip("norms over three numbers: rounding the weights alone to 8 bits moves the oracle's logits by more than their size")
    cfg = U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.moe(ff=24, experts=7, top=3)), (U.sig(), U.dense(24))], width=width, groups=groups, loop=(1, 2, 2))
    sd = U.sandwich_weights(cfg, 36)
    eng = U.engine(cfg, sd, dt, max_seq=120)
    toks = U.tokens(101, cfg["vocab"], 5)
    ref, margins = oracle(cfg, sd, toks)
    with eng.new_row() as row:
        got = torch.cat([row.extend(toks[:70], range(70)).clone(), row.extend(toks[70:83], range(13)).clone()]
                        + [row.extend([t], [0]).clone() for t in toks[83:]])
    e = U.err_clear(got, ref, margins) if dt == BF16 else U.err(got, ref)
    assert e < TOL[dt], e


def test_more_experts_than_the_row_kernel_routes():
    cfg = U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.moe(ff=8, experts=200, top=5))])
    sd = U.sandwich_weights(cfg, 37)
    eng = U.engine(cfg, sd, F32, max_seq=120)
    toks = U.tokens(60, cfg["vocab"], 6)
    ref = O.forward(cfg, sd, toks)
    with eng.new_row() as row:
        got = torch.cat([row.extend(toks[:50], range(50)).clone()] + [row.extend([t], [0]).clone() for t in toks[50:]])
    assert U.err(got, ref) < TOL[F32]


@pytest.mark.parametrize("T", [256, 300])
def test_prompts_on_the_large_tiles(T):
    """Wide layers and enough positions for tiles of 64 x 64 and 64 x 32, dense and of experts whose rows are put in order."""
    cfg = U.sandwich([(U.sig(heads=6, kv_heads=3, dim=50, vdim=70), U.dense(2200)), (U.gla(heads=2, dim=90, vdim=150), U.moe(ff=300, experts=5, top=2))],
                     width=1056, loop=(0, 1, 1))
    sd = U.sandwich_weights(cfg, 38)
    eng = U.engine(cfg, sd, BF16, max_seq=320)
    toks = U.tokens(T, cfg["vocab"], T)
    ref, margins = oracle(cfg, sd, toks)
    with eng.new_row() as row:
        got = run_all(row, toks)
    assert U.err_clear(got, ref, margins) < TOL[BF16]


def test_sizes_of_one():
    cfg = U.sandwich([(U.sig(heads=1, kv_heads=1, dim=1, vdim=1, bias_max=1, buckets=1, q_temp=(0.5, 1)), U.dense(1)),
                      (U.gla(heads=1, dim=1, vdim=1, rank=1), U.moe(ff=1, experts=1, top=1))], width=3, vocab=5, groups=1, eps=1e-2, loop=(0, 1, 1))
    sd = U.sandwich_weights(cfg, 12)
    eng = U.engine(cfg, sd, max_seq=50)
    toks = U.tokens(40, 5, 1)
    with eng.new_row() as row:
        assert U.err(run_all(row, toks), O.forward(cfg, sd, toks)) < 1e-4
    with eng.new_row() as row:
        got = torch.cat([row.extend([t], [0]).clone() for t in toks])
        assert U.err(got, O.forward(cfg, sd, toks)) < 1e-4


def test_residual_stream_of_every_layer_run():
    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 13)
    eng = U.engine(cfg, sd)
    toks = U.tokens(41, cfg["vocab"], 3)
    ref = []
    O.forward(cfg, sd, toks, layers_out=ref)
    assert len(ref) == 8
    buf = torch.zeros(len(ref), 41, cfg["width"], device="cuda")
    nat = eng.model._native
    nat.lib.vui_lm_debug_layers(nat.handle, buf.data_ptr())
    eng.new_row().extend(toks)
    torch.cuda.synchronize()
    nat.lib.vui_lm_debug_layers(nat.handle, None)
    for i, r in enumerate(ref):
        assert U.err(buf[i], r) < 2e-5, i


@BOTH
def test_prompt_against_token_by_token_and_portions(dt):
    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 14)
    toks = U.tokens(139, cfg["vocab"], 4)
    ref, margins = oracle(cfg, sd, toks)
    eng = U.engine(cfg, sd, dt)
    for cuts in ([1] * 139, [2] * 69 + [1], [3, 2, 5, 129], [64, 75], [70, 2, 67], [31, 1, 32, 1, 15, 16, 17, 26], [4, 135], [137, 2]):
        assert sum(cuts) == 139
        with eng.new_row() as row:
            at, outs = 0, []
            for n in cuts:
                outs.append(row.extend(toks[at:at + n], range(n)).clone())
                at += n
            e = U.err_clear(torch.cat(outs), ref, margins if dt == BF16 else [])
            assert e < TOL[dt], (cuts[:4], e)


@BOTH
def test_prompts_longer_than_one_native_call(dt, monkeypatch):
    from vui_amd.lm import TokenLM

    monkeypatch.setattr(TokenLM, "PREFILL_CHUNK", 40)
    cfg = U.sandwich_mixed(loop=(0, 5, 2)) if dt == F32 else U.sandwich([(U.sig(), U.dense()), (U.gla(), U.dense())], loop=(0, 2, 2))
    sd = U.sandwich_weights(cfg, 15)
    toks = U.tokens(131, cfg["vocab"], 15)
    want = [130, 0, 79, 80, 39, 3]
    eng = U.engine(cfg, sd, dt)
    with eng.new_row() as row:
        assert U.err(row.extend(toks, want), O.forward(cfg, sd, toks)[want]) < TOL[dt]


@BOTH
def test_both_forms_of_either_mixer_agree(dt):
    """Blocks and pieces of attention, chunks and single steps of the recurrence, behind prefixes of several lengths."""
    cfg = U.sandwich([(U.sig(dim=40, vdim=24), U.dense(64)), (U.gla(dim=36, vdim=50), None)])
    sd = U.sandwich_weights(cfg, 16)
    toks = U.tokens(230, cfg["vocab"], 5)
    ref = O.forward(cfg, sd, toks)
    eng = U.engine(cfg, sd, dt)
    nat = eng.model._native
    for first in (1, 130, 199):
        for attn, rec in ((2, 2), (1000, 1000), (2, 1000), (1000, 2)):
            nat.lib.vui_lm_block_from(nat.handle, attn, rec)
            with eng.new_row() as row:
                a = row.extend(toks[:first], range(first)).clone()
                b = row.extend(toks[first:], range(230 - first))
                assert U.err(torch.cat((a, b)), ref) < TOL[dt], (first, attn, rec)
    nat.lib.vui_lm_block_from(nat.handle, 0, 0)


@BOTH
def test_batch_of_unequal_rows_against_each_alone(dt):
    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 17)
    eng = U.engine(cfg, sd, dt, max_rows=7)
    lens = [1, 40, 3, 16, 129, 77, 15]
    seqs = [U.tokens(n + 9, cfg["vocab"], 20 + n) for n in lens]
    rows = [eng.new_row() for _ in lens]
    order = [4, 0, 6, 2, 5, 1, 3]
    for i in order:
        rows[i].extend(seqs[i][:lens[i]])
    got = [[] for _ in lens]
    for t in range(9):
        some = [i for i in order if (i + t) % 3]  # members change from step to step
        some = some if t % 2 else list(reversed(some))
        nxt = torch.tensor([seqs[i][lens[i] + len(got[i])] for i in some], device="cuda")
        L = eng.decode_step([rows[i] for i in some], nxt)
        for k, i in enumerate(some):
            got[i].append(L[k].clone())
    close = 0
    for i, n in enumerate(lens):
        ref, margins = oracle(cfg, sd, seqs[i][:n + len(got[i])])
        for t, g in enumerate(got[i]):
            if dt == BF16 and min(m[n + t] for m in margins) < 0.05:
                close += 1
                continue
            assert U.err(g[None], ref[n + t:n + t + 1]) < TOL[dt], (i, t)
    assert close < sum(map(len, got)) / 2


@BOTH
def test_slots_used_again(dt):
    """A slot that held a long sequence serves short ones; nothing of the old keys, values or states shows."""
    cfg = U.sandwich([(U.sig(), U.dense()), (U.gla(), None), (U.sig(heads=2), U.dense())], loop=(0, 3, 2))
    sd = U.sandwich_weights(cfg, 18)
    eng = U.engine(cfg, sd, dt, max_rows=2)
    a, b = eng.new_row(), eng.new_row()
    a.extend(U.tokens(200, cfg["vocab"], 6))
    b.extend(U.tokens(90, cfg["vocab"], 7))
    for first in (1, 2, 30, 80):
        a.close()
        a = eng.new_row()
        assert a.idx == 0 and a.offset == 0
        toks = U.tokens(first + 4, cfg["vocab"], first)
        outs = [a.extend(toks[:first], range(first)).clone()] + [a.extend([t], [0]).clone() for t in toks[first:]]
        assert U.err(torch.cat(outs), O.forward(cfg, sd, toks)) < TOL[dt], first
    more = U.tokens(90, cfg["vocab"], 7) + [3]
    assert U.err(b.extend([3], [0]), O.forward(cfg, sd, more)[-1:]) < TOL[dt]  # the neighbour is untouched


def test_every_run_of_a_looped_layer_has_a_cache_of_its_own():
    cfg = U.sandwich([(U.gla(), None), (U.sig(), None), (U.gla(), None)], loop=(1, 3, 3))
    eng = U.engine(cfg, U.sandwich_weights(cfg, 19), BF16)
    c = eng.model.cache
    assert sorted(c.k) == [1, 3, 5] and sorted(c.state) == [0, 2, 4, 6]
    assert len({t.data_ptr() for t in list(c.k.values()) + list(c.v.values()) + list(c.state.values())}) == 10
    assert all(t.dtype == F32 for t in c.state.values())
    eng.new_row().extend(U.tokens(20, cfg["vocab"]))
    assert not torch.equal(c.k[1], c.k[3]) and not torch.equal(c.state[2], c.state[4])


def needle_model(width=64, q_temp=None, vocab=12):
    """One attention layer whose single head looks for one token: token 10 asks, token 11 answers, 0..9 carry neither
    mark.  Weights of other keys are about e^-7."""
    cfg = U.sandwich([(U.sig(heads=1, kv_heads=1, dim=width, vdim=width, scale=0.5, bias_max=40, buckets=8, q_temp=q_temp), None)],
                     width=width, vocab=vocab, groups=2, scale=1.0)
    sd = U.sandwich_weights(cfg, 20)
    emb = torch.randn(vocab, width, generator=torch.Generator().manual_seed(21)) * 0.3
    emb[:, -2:] = 0.0
    emb[10, -2] = emb[11, -1] = 3.0
    eye = torch.eye(width)
    find = torch.zeros(width, width)
    find[-1, -2] = 1.0
    sd["embed"] = emb.to(BF16)
    sd["l0.mix.q"], sd["l0.mix.k"], sd["l0.mix.v"], sd["l0.mix.o"] = find.to(BF16), eye.to(BF16), eye.to(BF16), eye.to(BF16)
    for n in ("q.b", "k.b", "v.b", "o.b", "rel"):
        sd["l0.mix." + n].zero_()
    for n in ("l0.mix.q.norm", "l0.mix.k.norm", "l0.norm1"):
        sd[n].fill_(1.0)
    sd["l0.mix.pb"].fill_(-7.0)
    sd["l0.mix.g"].zero_()
    return cfg, sd


@BOTH
def test_one_key_among_hundreds(dt):
    """The needle at the first tokens, at borders of 16-, 32- and 64-key tiles and of pieces, and right before the query,
    seen from a prompt and from a decoded token."""
    cfg, sd = needle_model()
    eng = U.engine(cfg, sd, dt, max_seq=420)
    base = [t % 10 for t in U.tokens(400, 10, 8)]
    worst = 0.0
    without = O.forward(cfg, sd, base[:399] + [10])[-1:]
    for at in (0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 255, 256, 335, 383, 384, 397, 398):
        toks = list(base)
        toks[at], toks[399] = 11, 10
        ref = O.forward(cfg, sd, toks)[-1:]
        assert U.err(without, ref) > 0.3  # losing the needle would show
        with eng.new_row() as row:
            worst = max(worst, U.err(row.extend(toks, [399]), ref))
        with eng.new_row() as row:
            row.extend(toks[:399])
            worst = max(worst, U.err(row.extend(toks[399:], [0]), ref))
        with eng.new_row() as row:
            row.extend(toks[:at + 1])
            row.extend(toks[at + 1:398]) if at < 397 else None
            worst = max(worst, U.err(row.extend(toks[row.offset:], [399 - row.offset]), ref))
    assert worst < TOL[dt], worst


@BOTH
def test_a_key_of_the_future_is_not_seen(dt):
    cfg, sd = needle_model()
    eng = U.engine(cfg, sd, dt, max_seq=160)
    toks = [t % 10 for t in U.tokens(150, 10, 9)]
    for q in (14, 15, 16, 31, 62, 63, 64, 100):
        s = list(toks)
        s[q], s[q + 1] = 10, 11  # the needle comes one position after its query
        with eng.new_row() as row:
            assert U.err(run_all(row, s), O.forward(cfg, sd, s)) < TOL[dt], q


@BOTH
def test_distances_at_every_border_of_a_bucket(dt):
    """Scores are the bias alone and one bucket is open: the output is the sum of the values at its distances.  Prompts
    and decoded tokens."""
    cfg, sd = needle_model(vocab=200)
    sd["l0.mix.q"].zero_()
    eng0 = None
    toks = U.tokens(130, 200, 10)
    for b in range(8):
        sd["l0.mix.rel"].fill_(-20.0)
        sd["l0.mix.rel"][b] = 8.0
        ref = O.forward(cfg, sd, toks)
        eng0 = U.engine(cfg, sd, dt, max_seq=140)
        with eng0.new_row() as row:
            assert U.err(run_all(row, toks), ref) < TOL[dt], b
        with eng0.new_row() as row:
            row.extend(toks[:90])
            got = torch.cat([row.extend([t], [0]).clone() for t in toks[90:]])
            assert U.err(got, ref[90:]) < TOL[dt], b


def test_query_temperature_steps():
    """A steep temperature: the weight of a key depends on which side of a multiple of `every` the query is (fp32)."""
    for every, coef in ((1, 0.3), (5, 2.0), (64, 3.0)):
        cfg = U.sandwich([(U.sig(q_temp=(coef, every)), None)])
        sd = U.sandwich_weights(cfg, 22)
        eng = U.engine(cfg, sd, max_seq=330)
        toks = U.tokens(320, cfg["vocab"], 11)
        ref = O.forward(cfg, sd, toks)
        with eng.new_row() as row:
            got = torch.cat([run_all(row, toks[:250])] + [row.extend([t], [0]).clone() for t in toks[250:]])
            assert U.err(got, ref) < TOL[F32], (every, coef)


@BOTH
def test_long_decoding_keeps_the_state(dt):
    """Decays within a percent of one, 300 decoded tokens: what entered early is still there."""
    cfg = U.sandwich([(U.gla(tau=16.0), None), (U.gla(heads=2, dim=17, vdim=9, tau=16.0), None)])
    sd = U.sandwich_weights(cfg, 23)
    for i in range(2):
        sd[f"l{i}.mix.a2.b"].fill_(4.0)
    toks = U.tokens(310, cfg["vocab"], 12)
    ref = O.forward(cfg, sd, toks)
    eng = U.engine(cfg, sd, dt, max_seq=320)
    with eng.new_row() as row:
        outs = [row.extend(toks[:10], range(10)).clone()] + [row.extend([t], [0]).clone() for t in toks[10:]]
        assert U.err(torch.cat(outs), ref) < TOL[dt]


def test_a_fresh_slot_starts_from_zero_state():
    cfg = U.sandwich([(U.gla(), None)])
    sd = U.sandwich_weights(cfg, 24)
    eng = U.engine(cfg, sd, BF16)
    toks = U.tokens(20, cfg["vocab"], 12)
    with eng.new_row() as row:
        a = row.extend(toks, [19]).clone()
    for n in (20, 3, 1):  # chunks, steps, a single position
        eng.model.cache.state[0].fill_(1e6)
        with eng.new_row() as row:
            got = row.extend(toks[:n], [n - 1]).clone()
            assert U.err(got, O.forward(cfg, sd, toks[:n])[-1:]) < TOL[BF16]
            assert n < 20 or torch.equal(a, got)


@BOTH
def test_all_tokens_to_few_experts(dt):
    """A router whose bias sends everything to the last experts: whole tiles of one expert and none of the others."""
    cfg = U.sandwich([(U.gla(heads=1, dim=4, vdim=4), U.moe(experts=20, top=2))])
    sd = U.sandwich_weights(cfg, 25)
    sd["l0.mlp.router.b"].zero_()
    sd["l0.mlp.router.b"][18:] = 50.0
    eng = U.engine(cfg, sd, dt, max_seq=160)
    for T in (1, 15, 16, 17, 31, 32, 33, 150):
        toks = U.tokens(T, cfg["vocab"], T)
        with eng.new_row() as row:
            assert U.err(run_all(row, toks), O.forward(cfg, sd, toks)) < TOL[dt], T


@BOTH
def test_captured_step_replayed(dt):
    """The bucketed graph against the oracle, several replays with other work of the engine in between."""
    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 26)
    eng = U.engine(cfg, sd, dt, max_rows=2)
    toks = U.tokens(30, cfg["vocab"], 13)
    ref, margins = oracle(cfg, sd, toks)
    a = eng.new_row()
    a.extend(toks[:20])
    for t in range(20, 30):
        got = a.extend([toks[t]], [0]).clone()
        assert (dt == BF16 and min(m[t] for m in margins) < 0.05) or U.err(got, ref[t:t + 1]) < TOL[dt], t
        with eng.new_row() as b:
            b.extend(U.tokens(5 + t, cfg["vocab"], t))
        torch.cuda.synchronize()


def test_rewind_restores_positions_and_states():
    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 27)
    eng = U.engine(cfg, sd)
    toks = U.tokens(60, cfg["vocab"], 14)
    row = eng.new_row()
    row.extend(toks[:40])
    assert row.mark_prompt() == 40
    a = row.extend(toks[40:], range(20)).clone()
    row.extend([1, 2, 3])
    assert row.rewind() == 40
    assert torch.equal(a, row.extend(toks[40:], range(20)))
    assert row.reset() == 0
    assert U.err(run_all(row, toks[:9]), O.forward(cfg, sd, toks[:9])) < TOL[F32]


def test_greedy_generation_through_the_scheduler():
    """More requests than rows, unequal prompts and lengths, stops; fp32, token for token."""
    from vui_amd.lm_engine import TokenRequest

    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 28)
    eng = U.engine(cfg, sd, max_rows=3, max_seq=120)
    reqs = [TokenRequest(U.tokens(n, cfg["vocab"], 30 + n), max_new=m) for n, m in ((5, 12), (70, 3), (1, 20), (33, 1), (17, 9), (2, 15))]
    ref = [O.greedy(cfg, sd, r.tokens, r.max_new) for r in reqs]
    assert eng.generate(reqs) == ref
    assert len(eng._free) == 3 and eng.generate(reqs) == ref
    stops = [TokenRequest(r.tokens, r.max_new, frozenset({o[len(o) // 2]})) for r, o in zip(reqs, ref)]
    assert eng.generate(stops) == [o[:o.index(o[len(o) // 2]) + 1] for o in ref]
    assert list(eng.stream(reqs[0])) == ref[0]


def test_generation_in_bf16_and_sampled():
    from vui_amd.engine import GenConfig
    from vui_amd.lm_engine import TokenRequest

    cfg = U.sandwich([(U.sig(), U.dense()), (U.gla(), U.dense())], loop=(0, 2, 2))
    sd = U.sandwich_weights(cfg, 29)
    eng = U.engine(cfg, sd, BF16, max_rows=4, max_seq=120)
    reqs = [TokenRequest(U.tokens(n, cfg["vocab"], 40 + n), max_new=10) for n in (3, 90, 20, 7, 11)]
    for r, o in zip(reqs, eng.generate(reqs)):
        L = O.forward(cfg, sd, list(r.tokens) + o)[len(r.tokens) - 1:-1]
        for t, tok in enumerate(o):  # the oracle's choice or within the tolerance of it
            assert L[t].max() - L[t][tok] <= 2 * TOL[BF16] * L[t].pow(2).mean().sqrt()
    c = GenConfig(temperature=0.9, top_k=20, rep_penalty=1.2, rep_window=6, seed=5)
    a, b = eng.generate(reqs, c), eng.generate(reqs, c)
    assert a == b and all(0 <= t < cfg["vocab"] for o in a for t in o)


def test_checkpoint_folder_and_programs(tmp_path):
    """A folder on disk through the registry, the replay program and the command line, in processes of their own."""
    import os
    import subprocess
    import sys

    import numpy as np
    from safetensors.torch import save_file

    from tests.conftest import ROOT

    cfg = U.sandwich_mixed()
    sd = U.sandwich_weights(cfg, 30)
    (tmp_path / "m").mkdir()
    (tmp_path / "out").mkdir()
    (tmp_path / "m" / "config.json").write_text(json.dumps(cfg))
    save_file(sd, str(tmp_path / "m" / "model.safetensors"))
    toks = U.tokens(30, cfg["vocab"], 50)
    steps = [{"step": 0, "entries": [{"id": "x", "tokens": toks[:21], "want": [0, 20]}], "end": []},
             {"step": 1, "entries": [{"id": "x", "tokens": toks[21:22], "want": [0]}], "end": []},
             {"step": 2, "entries": [{"id": "x", "tokens": toks[22:], "want": []}], "end": ["x"]},
             {"step": 3, "entries": [{"id": "y", "tokens": toks[:2], "want": [1]}], "end": ["y"]}]
    p = subprocess.run([sys.executable, os.path.join(ROOT, "bin", "trace_run"), "--model", str(tmp_path / "m"), "--dtype", "float32",
                        "--out", str(tmp_path / "out"), "--max-tokens", "30"], input="\n".join(json.dumps(s) for s in steps) + "\n",
                       capture_output=True, text=True, timeout=100)
    assert p.returncode == 0, p.stderr[-2000:]
    assert [ln for ln in p.stdout.splitlines() if ln.startswith("done")] == [f"done {i}" for i in range(4)]
    ref = O.forward(cfg, sd, toks)
    for step, want in ((0, [0, 20]), (1, [21]), (3, [1])):
        got = torch.from_numpy(np.fromfile(tmp_path / "out" / f"{step}.f32", dtype="<f4").reshape(len(want), -1).copy())
        assert U.err(got, ref[want]) < TOL[F32]
    p = subprocess.run([sys.executable, "-m", "vui_amd", "generate", "--model", str(tmp_path / "m"), "--dtype", "float32", "--tokens", "5,9,2",
                        "--tokens", "7", "--max-new", "4"], capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    got = [json.loads(ln) for ln in p.stdout.splitlines() if ln.startswith("{")]
    assert got == [{"prompt": t, "tokens": O.greedy(cfg, sd, t, 4)} for t in ([5, 9, 2], [7])]


def test_lengths_of_several_thousand():
    """Scores far out and many pieces: 2100 positions, the last ones decoded (bf16 and fp32, one layer of each mixer)."""
    cfg = U.sandwich([(U.sig(heads=2, kv_heads=1, bias_max=900, buckets=32), None), (U.gla(heads=1), None)], width=48)
    sd = U.sandwich_weights(cfg, 31)
    toks = U.tokens(2104, cfg["vocab"], 16)
    ref = O.forward(cfg, sd, toks)[-5:]
    assert math.isfinite(float(ref.sum()))
    for dt in (F32, BF16):
        eng = U.engine(cfg, sd, dt, max_seq=2112)
        with eng.new_row() as row:
            outs = [row.extend(toks[:2100], [2099]).clone()] + [row.extend([t], [0]).clone() for t in toks[2100:]]
            assert U.err(torch.cat(outs), ref) < 2 * TOL[dt]
