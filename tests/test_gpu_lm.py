"""Token language models on the GPU against the plain oracle (float64), fp32 and bf16."""
import dataclasses

import pytest
import torch

from oracle import lm_oracle as O
from tests import lm_util as U

pytestmark = pytest.mark.gpu
F32, BF16 = torch.float32, torch.bfloat16
BOTH = pytest.mark.parametrize("dt", [F32, BF16])


def run_all(row, toks):
    return row.extend(toks, range(len(toks)))


SINGLE = {
    "attention": lambda: U.config([U.attn()], ff=None),
    "attention_partial_rotation": lambda: U.config([U.attn(rot_dim=12, dims=6, base=50.0)], ff=None),
    "attention_shared_latent": lambda: U.config([U.attn(), U.attn(heads=4, dim=9, vdim=7, kv_from=0, scale=0.7)], ff=None),
    "mingru": lambda: U.config([U.gru()], ff=None),
    "feed_forward": lambda: U.config([U.gru(16)], ff=150, limit=0.8),
    "parallel_layer": lambda: U.config([U.attn()], ff=90),
    "mixed": U.mixed,
    "ones": lambda: U.config([U.attn(heads=1, dim=1, rot_dim=2, vdim=1, kv_rank=1), U.gru(1)], width=3, vocab=2, ff=1, eps=1e-2),
    "equal_sizes": lambda: U.config([U.attn(heads=2, dim=16, rot_dim=16, vdim=16, kv_rank=16), U.gru(16)], width=16, vocab=16, ff=16),
    "many_heads": lambda: U.config([U.attn(heads=21, dim=12, rot_dim=6, vdim=20, kv_rank=72)], width=144, ff=200),
    "wide_heads": lambda: U.config([U.attn(heads=2, dim=70, rot_dim=40, vdim=100, kv_rank=200), U.gru(300)], width=192, ff=260),
    "no_expanded_form": lambda: U.config([U.attn(heads=2, dim=140, rot_dim=70, vdim=150, kv_rank=560)], width=160, ff=None),
}


@BOTH
@pytest.mark.parametrize("name", sorted(SINGLE))
def test_prompts_of_many_lengths(name, dt):
    """Each mechanism alone and together; lengths on both sides of 16-row tiles, of the scan's chunks and of the switch
    to expanded keys."""
    cfg = SINGLE[name]()
    sd = U.weights(cfg, 11)
    if name == "feed_forward":
        sd["l0.mix.o"].zero_()
    if name == "ones":  # one channel: keep the logits away from zero
        sd["embed"].add_(1.0)
    eng = U.engine(cfg, sd, dt, max_seq=160)
    for T in (1, 2, 16, 17, 33, 64, 150):
        toks = U.tokens(T, cfg["vocab"], T)
        with eng.new_row() as row:
            e = U.err(run_all(row, toks), O.forward(cfg, sd, toks))
            assert e < U.TOL[dt], (name, T, e)


def test_residual_stream_of_every_layer():
    cfg = U.mixed()
    sd = U.weights(cfg, 12)
    eng = U.engine(cfg, sd)
    toks = U.tokens(41, cfg["vocab"], 3)
    ref = []
    O.forward(cfg, sd, toks, layers_out=ref)
    buf = torch.zeros(len(ref), 41, cfg["width"], device="cuda")
    nat = eng.model._native
    nat.lib.vui_lm_debug_layers(nat.handle, buf.data_ptr())
    eng.new_row().extend(toks)
    torch.cuda.synchronize()
    nat.lib.vui_lm_debug_layers(nat.handle, None)
    for i, r in enumerate(ref):
        assert U.err(buf[i], r) < 1e-5, i


@BOTH
def test_prompt_against_token_by_token_and_portions(dt):
    cfg = U.mixed()
    sd = U.weights(cfg, 13, q_gain=3.0)
    toks = U.tokens(139, cfg["vocab"], 4)
    ref = O.forward(cfg, sd, toks)
    eng = U.engine(cfg, sd, dt)
    tol = U.TOL[dt] * 2  # sharper attention passes on more of the rounding
    for cuts in ([1] * 139, [2] * 69 + [1], [3, 2, 5, 129], [64, 75], [70, 2, 67], [31, 1, 32, 1, 15, 16, 17, 26], [5, 134], [137, 2]):
        assert sum(cuts) == 139
        with eng.new_row() as row:
            at, outs = 0, []
            for n in cuts:
                outs.append(row.extend(toks[at:at + n], range(n)).clone())
                at += n
            e = U.err(torch.cat(outs), ref)
            assert e < tol, (cuts[:4], e)


@BOTH
def test_prompts_longer_than_one_native_call(dt, monkeypatch):
    """Wanted places in any order, in several calls of at most 40 positions, some calls without any."""
    from vui_amd.lm import TokenLM

    monkeypatch.setattr(TokenLM, "PREFILL_CHUNK", 40)
    cfg = U.mixed()
    sd = U.weights(cfg, 28)
    toks = U.tokens(131, cfg["vocab"], 15)
    want = [130, 0, 79, 80, 39, 3]
    eng = U.engine(cfg, sd, dt)
    with eng.new_row() as row:
        assert U.err(row.extend(toks, want), O.forward(cfg, sd, toks)[want]) < U.TOL[dt]
        with pytest.raises(ValueError):
            row.extend([1, 2], [2])
        with pytest.raises(ValueError):
            row.extend([], [])
        with pytest.raises(ValueError):
            row.extend(U.tokens(140, cfg["vocab"]))


def test_both_forms_of_attention_agree():
    """Expanded keys against the latent space, from the same cache, for portions behind a long prefix (bf16)."""
    cfg = U.config([U.attn(), U.attn(heads=4, dim=40, vdim=24, kv_from=0)], ff=64)
    sd = U.weights(cfg, 14, q_gain=2.0)
    toks = U.tokens(230, cfg["vocab"], 5)
    ref = O.forward(cfg, sd, toks)
    eng = U.engine(cfg, sd, BF16)
    nat = eng.model._native
    for first in (1, 130, 199):
        for rows in (2, 1000):
            nat.lib.vui_lm_expand_from(nat.handle, rows)
            with eng.new_row() as row:
                a = row.extend(toks[:first], range(first)).clone()
                b = row.extend(toks[first:], range(230 - first))
                assert U.err(torch.cat((a, b)), ref) < 0.08, (first, rows)
    nat.lib.vui_lm_expand_from(nat.handle, 0)


@BOTH
def test_batch_of_unequal_rows_against_each_alone(dt):
    cfg = U.mixed()
    sd = U.weights(cfg, 15)
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
    for i, n in enumerate(lens):
        ref = O.forward(cfg, sd, seqs[i][:n + len(got[i])])[n:]
        assert len(got[i]) >= 5 and U.err(torch.stack(got[i]), ref) < U.TOL[dt], i


@BOTH
def test_slots_used_again(dt):
    """A slot that held a long sequence serves short ones; nothing of the old keys, latents or state shows."""
    cfg = U.mixed()
    sd = U.weights(cfg, 16)
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
        assert U.err(torch.cat(outs), O.forward(cfg, sd, toks)) < U.TOL[dt], first
    more = U.tokens(90, cfg["vocab"], 7) + [3]
    assert U.err(b.extend([3], [0]), O.forward(cfg, sd, more)[-1:]) < U.TOL[dt]  # the neighbour is untouched


def needle_model(width=64):
    """One attention layer whose single head looks for one token: keys and values are the (normed) latent itself, and
    W_q turns the query token's own mark (the last coordinate but one) into the needle's (the last).  Tokens 0..9 carry
    neither mark, token 10 is the query, 11 the needle."""
    cfg = U.config([U.attn(heads=1, dim=width, rot_dim=4, vdim=width, kv_rank=width, scale=0.6)], width=width, vocab=12, ff=None)
    sd = U.weights(cfg, 17)
    g = torch.Generator().manual_seed(18)
    emb = torch.randn(12, width, generator=g) * 0.3
    emb[:, -2:] = 0.0
    emb[10, -2] = emb[11, -1] = 3.0
    eye = torch.eye(width)
    find = torch.zeros(width, width)
    find[-1, -2] = 1.0
    sd["embed"] = emb.to(BF16)
    sd["l0.mix.q"] = torch.cat((find, torch.zeros(4, width))).to(BF16)
    sd["l0.mix.dkv"] = torch.cat((eye, torch.zeros(4, width))).to(BF16)
    sd["l0.mix.dkv.norm"] = torch.ones(width, dtype=BF16)
    sd["l0.mix.uk"], sd["l0.mix.uv"], sd["l0.mix.o"] = eye.to(BF16), eye.to(BF16), (4 * eye).to(BF16)
    sd["l0.norm1"] = torch.tensor(1.0, dtype=BF16)
    return cfg, sd


@BOTH
def test_one_key_among_hundreds(dt):
    """The needle at the first tokens, at borders of 16-, 32- and 64-key tiles and of splits, and right before the query,
    seen from a prompt and from a decoded token."""
    cfg, sd = needle_model()
    eng = U.engine(cfg, sd, dt, max_seq=420)
    base = [t % 10 for t in U.tokens(400, 10, 8)]
    worst = 0.0
    for at in (0, 1, 15, 16, 31, 32, 63, 64, 127, 128, 255, 256, 335, 383, 384, 397, 398):
        toks = list(base)
        toks[at], toks[399] = 11, 10
        ref, without = O.forward(cfg, sd, toks)[-1:], O.forward(cfg, sd, base[:399] + [10])[-1:]
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
    assert worst < U.TOL[dt], worst


@BOTH
def test_a_key_of_the_future_is_not_seen(dt):
    cfg, sd = needle_model()
    eng = U.engine(cfg, sd, dt, max_seq=160)
    toks = [t % 10 for t in U.tokens(150, 10, 9)]
    for q in (14, 15, 16, 31, 62, 63, 64, 100):
        s = list(toks)
        s[q], s[q + 1] = 10, 11  # the needle comes one position after its query
        with eng.new_row() as row:
            assert U.err(row.extend(s, range(150)), O.forward(cfg, sd, s)) < U.TOL[dt], q


def test_rotation_far_out():
    """Scores from the rotated part alone, hundreds of positions in, decoded and from a prompt (fp32)."""
    cfg = U.config([U.attn(heads=2, dim=8, rot_dim=16, vdim=16, kv_rank=24, base=40.0, scale=1.0)], ff=None)
    sd = U.weights(cfg, 19, q_gain=2.0)
    sd["l0.mix.uk"].zero_()
    eng = U.engine(cfg, sd, max_seq=700)
    toks = U.tokens(660, cfg["vocab"], 10)
    ref = O.forward(cfg, sd, toks)
    with eng.new_row() as row:
        a = row.extend(toks[:640], range(640)).clone()
        b = [row.extend([t], [0]).clone() for t in toks[640:]]
        assert U.err(torch.cat([a] + b), ref) < 1e-4


def test_long_decoding_keeps_the_state():
    """Slow gates (update around 2%), 300 decoded tokens: what entered early is still there (fp32 state in both)."""
    cfg = U.config([U.gru(40), U.gru(21)], ff=None)
    sd = U.weights(cfg, 20)
    for i in range(2):
        sd[f"l{i}.mix.z.b"].fill_(-4.0)
    toks = U.tokens(310, cfg["vocab"], 11)
    ref = O.forward(cfg, sd, toks)
    for dt in (F32, BF16):
        eng = U.engine(cfg, sd, dt, max_seq=320)
        with eng.new_row() as row:
            outs = [row.extend(toks[:10], range(10)).clone()] + [row.extend([t], [0]).clone() for t in toks[10:]]
            assert U.err(torch.cat(outs), ref) < U.TOL[dt]


def test_recurrent_state_is_fp32_in_bf16_contexts():
    cfg = U.config([U.gru(40)], ff=None)
    eng = U.engine(cfg, U.weights(cfg, 21), BF16)
    assert eng.model.cache.state[0].dtype == F32
    # fresh slots start from zero whatever the memory holds
    toks = U.tokens(20, cfg["vocab"], 12)
    with eng.new_row() as row:
        a = row.extend(toks, [19]).clone()
    eng.model.cache.state[0].fill_(1e6)
    with eng.new_row() as row:
        assert torch.equal(a, row.extend(toks, [19]))
    eng.model.cache.state[0].fill_(1e6)
    with eng.new_row() as row:
        first = row.extend(toks[:1], [0]).clone()
        assert U.err(first, O.forward(cfg, U.weights(cfg, 21), toks[:1])) < U.TOL[BF16]


@BOTH
def test_captured_step_replayed(dt):
    """The bucketed graph against fresh steps, several replays with other work of the engine in between."""
    cfg = U.mixed()
    sd = U.weights(cfg, 22)
    eng = U.engine(cfg, sd, dt, max_rows=2)
    toks = U.tokens(30, cfg["vocab"], 13)
    ref = O.forward(cfg, sd, toks)
    a = eng.new_row()
    a.extend(toks[:20])
    for t in range(20, 30):
        got = a.extend([toks[t]], [0]).clone()
        assert U.err(got, ref[t:t + 1]) < U.TOL[dt], t
        with eng.new_row() as b:
            b.extend(U.tokens(5 + t, cfg["vocab"], t))
        torch.cuda.synchronize()


def test_rewind_restores_positions_and_state():
    cfg = U.mixed()
    sd = U.weights(cfg, 23)
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
    assert U.err(run_all(row, toks[:9]), O.forward(cfg, sd, toks[:9])) < U.TOL[F32]


def margin_ok(cfg, sd, prompt, drawn, dt):
    """Every drawn token is the oracle's choice or within the tolerance of it."""
    L = O.forward(cfg, sd, list(prompt) + drawn)[len(prompt) - 1:-1]
    for t, tok in enumerate(drawn):
        if L[t].max() - L[t][tok] > 2 * U.TOL[dt] * L[t].pow(2).mean().sqrt():
            return False
    return True


def test_greedy_generation_through_the_scheduler():
    """More requests than rows, unequal prompts and lengths, stops; fp32, token for token."""
    from vui_amd.lm_engine import TokenRequest

    cfg = U.mixed()
    sd = U.weights(cfg, 24)
    eng = U.engine(cfg, sd, max_rows=3, max_seq=120)
    reqs = [TokenRequest(U.tokens(n, cfg["vocab"], 30 + n), max_new=m) for n, m in ((5, 12), (70, 3), (1, 20), (33, 1), (17, 9), (2, 15))]
    ref = [O.greedy(cfg, sd, r.tokens, r.max_new) for r in reqs]
    got = eng.generate(reqs)
    assert got == ref
    assert len(eng._free) == 3 and eng.generate(reqs) == ref
    # a stop token ends the answer with itself
    stops = [TokenRequest(r.tokens, r.max_new, frozenset({o[len(o) // 2]})) for r, o in zip(reqs, ref)]
    assert eng.generate(stops) == [o[:o.index(o[len(o) // 2]) + 1] for o in ref]
    assert list(eng.stream(reqs[0])) == ref[0]
    # the slot's end ends the answer
    full = eng.generate([TokenRequest(U.tokens(110, cfg["vocab"], 1), max_new=50)])[0]
    assert len(full) == 11
    with pytest.raises(ValueError):
        eng.generate([TokenRequest(U.tokens(121, cfg["vocab"], 1))])
    assert len(eng._free) == 3


def test_generation_in_bf16_and_sampled():
    from vui_amd.engine import GenConfig
    from vui_amd.lm_engine import TokenRequest

    cfg = U.mixed()
    sd = U.weights(cfg, 25)
    eng = U.engine(cfg, sd, BF16, max_rows=4, max_seq=120)
    reqs = [TokenRequest(U.tokens(n, cfg["vocab"], 40 + n), max_new=10) for n in (3, 90, 20, 7, 11)]
    for r, o in zip(reqs, eng.generate(reqs)):
        assert len(o) == 10 and margin_ok(cfg, sd, r.tokens, o, BF16)
    c = GenConfig(temperature=0.9, top_k=20, rep_penalty=1.2, rep_window=6, seed=5)
    a, b = eng.generate(reqs, c), eng.generate(reqs, c)
    assert a == b and a != eng.generate(reqs, dataclasses.replace(c, seed=6))
    assert all(0 <= t < cfg["vocab"] for o in a for t in o)
    # top-k 1 under a penalty: no token of the window comes back while another is close; greedy stays deterministic
    g = GenConfig(temperature=1.0, top_k=1, rep_penalty=50.0, rep_window=4)
    for o in eng.generate(reqs, g):
        assert all(o[i] not in o[max(0, i - 4):i] for i in range(len(o)))
    n = GenConfig(temperature=1.0, top_k=0, top_p=0.5, rep_penalty=1.0, seed=1)
    assert eng.generate(reqs, n) == eng.generate(reqs, n)


def test_checkpoint_folder_and_trace_program(tmp_path):
    """A folder on disk through the registry and the replay program, in a process of its own."""
    import json
    import os
    import subprocess
    import sys

    import numpy as np
    from safetensors.torch import save_file

    from tests.conftest import ROOT

    cfg = U.mixed()
    sd = U.weights(cfg, 26)
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
        assert U.err(got, ref[want]) < U.TOL[F32]
    assert not (tmp_path / "out" / "2.f32").exists()
    p = subprocess.run([sys.executable, "-m", "vui_amd", "generate", "--model", str(tmp_path / "m"), "--dtype", "float32", "--tokens", "5,9,2",
                        "--tokens", "7", "--max-new", "4"], capture_output=True, text=True, timeout=100, cwd=ROOT)
    assert p.returncode == 0, p.stderr[-2000:]
    got = [json.loads(ln) for ln in p.stdout.splitlines() if ln.startswith("{")]
    assert got == [{"prompt": t, "tokens": O.greedy(cfg, sd, t, 4)} for t in ([5, 9, 2], [7])]


def sample(logits, temperature, top_k, top_p, seed, frame, keep_ties=True, counts=None, penalty=1.0):
    import ctypes as C

    from vui_amd import _lib
    from vui_amd.model import make_sample_params

    lib = _lib.load(lm_only=True)
    B, V = logits.shape
    x = logits.float().cuda().contiguous()
    ctr = torch.tensor([frame], dtype=torch.int32, device="cuda")
    out = torch.full((B,), -1, dtype=torch.long, device="cuda")
    sp = make_sample_params(temperature, top_k, seed, ctr, keep_ties=keep_ties, top_p=top_p or 0.0)
    c = counts.cuda() if counts is not None else None
    _lib.check(lib.vui_sample_tokens(x.data_ptr(), V, _lib.ptr(c), None, None, float(penalty), 0, C.byref(sp), out.data_ptr(), B,
                                     torch.cuda.current_stream().cuda_stream), "vui_sample_tokens")
    torch.cuda.synchronize()
    return out.cpu().tolist(), c


@pytest.mark.parametrize("V", [3000, 8193, 50257])
def test_sampler_of_any_vocabulary(V):
    """The register form up to 8192 entries and the re-reading form beyond, under the same rules: greedy (lowest index of
    the maximum), top-k with ties kept and cut to exactly k, nucleus, both together, a penalty; heavy ties."""
    from oracle import vui_oracle as VO

    g = torch.Generator().manual_seed(V)
    logits = torch.randn(12, V, generator=g) * 3
    logits[4:8] = (logits[4:8] * 2).round() / 2  # many equal values
    logits[0, [77, V - 1]] = 40.0
    assert sample(logits, 1.0, 1, None, 0, 0)[0] == [int(r.argmax()) for r in logits]
    agree = total = 0
    for frame, (temp, k, p) in enumerate([(0.9, 50, None), (1.3, 0, None), (0.7, 0, 0.9), (1.0, 40, 0.8), (1.0, 5000 if V > 5000 else 900, 0.3), (1.0, 7, 0.999)]):
        got, _ = sample(logits, temp, k, p, 99, frame)
        for b, tok in enumerate(got):
            u = VO.uniform01(99, frame, b, 0)
            kept = VO.sample_codes_probs(logits[b], temp, k if k > 0 else None, p)
            assert kept[tok] > 0, (V, temp, k, p, b)
            agree += tok == VO._inverse_cdf(kept, u)
            total += 1
        if p is None and k > 0:
            got, _ = sample(logits, temp, k, None, 7, frame, keep_ties=False)
            for b, tok in enumerate(got):
                kept = VO.cb0_probs(logits[b], temp, k)
                assert kept[tok] > 0 and (kept > 0).sum() == k
                agree += tok == VO._inverse_cdf(kept, VO.uniform01(7, frame, b, 0))
                total += 1
    assert agree >= 0.97 * total, (agree, total)
    counts = torch.zeros(12, V)
    counts[0, 77] = 3.0
    got, after = sample(logits, 1.0, 1, None, 0, 0, counts=counts, penalty=2.0)
    assert got[0] == V - 1 and after[0, V - 1] == 1.0 and after.sum() == 3.0 + 12


def test_generation_with_a_large_vocabulary():
    from vui_amd.lm_engine import TokenRequest

    cfg = U.config([U.attn(), U.gru()], vocab=9001)
    sd = U.weights(cfg, 27)
    eng = U.engine(cfg, sd, max_rows=2, max_seq=40)
    reqs = [TokenRequest(U.tokens(n, 9001, n), max_new=5) for n in (3, 20, 9)]
    assert eng.generate(reqs) == [O.greedy(cfg, sd, r.tokens, 5) for r in reqs]
