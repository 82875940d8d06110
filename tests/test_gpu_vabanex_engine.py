"""The sequence engine on small random Vabanex models against oracle/vabanex.py: whole prompts with the stream after every layer,
decoding through the caches, portions, mixed batches, reuse of pages and slots, the first tokens, a far token that decides the
logits pages later, long decoding, generation through the scheduler, graph replays, a checkpoint
folder served by its configuration."""
import json
import struct

import numpy as np
import pytest
import torch

from oracle import vabanex as ov
from tests.conftest import load_pkg
from tests.seq_helpers import make_engine, rel_err, rows_close, run_portions, run_whole

pytestmark = pytest.mark.gpu

CONFIGS = {
    # every kind of feed-forward, layers that differ in every size, rescaled frequencies and plain ones
    "mixed": dict(layers=[(None, ("dense",)), ({"scaling": None}, ("moe",)), (dict(heads=5, dim=8, rot_dim=12, vdim=10, kv_rank=30, q_rank=20), None),
                          (None, ("moe", dict(experts=8, count=4, keep=2, top=3, ff=33, scale=0.8)))]),
    # sizes that are no multiples of 4 or 8, one head, one pair rotated, one expert per group, a single choice, no groups, no cap
    "odd": dict(width=50, vocab=61, eps=1e-3, embed_scale=1.3, softcap=None,
                layers=[(dict(heads=1, dim=12, rot_dim=2, vdim=9, kv_rank=10, q_rank=6), ("moe", dict(experts=4, count=4, keep=2, top=1, ff=10, scale=1.0))),
                        (dict(heads=3, dim=5, rot_dim=6, vdim=7, kv_rank=13, q_rank=11, scale=0.4), ("dense", dict(ff=33, limit=0.5))),
                        (dict(heads=1, dim=3, rot_dim=4, vdim=1, kv_rank=5, q_rank=1), ("moe", dict(experts=3, count=0, top=3, ff=6)))]),
    # sizes of the matrix-core tiles: latent + rotated part of exactly one 64-element row, and of 96 in a padded row
    "tiles": dict(width=64, vocab=130, embed_scale=1.0, softcap=4.0,
                  layers=[(dict(heads=4, dim=32, rot_dim=16, vdim=32, kv_rank=48, q_rank=32, base=100.0), ("moe", dict(experts=8, count=2, keep=1, top=4, ff=32))),
                          (dict(heads=8, dim=16, rot_dim=16, vdim=64, kv_rank=72, q_rank=16, base=300.0), ("dense", dict(ff=96, limit=1.0)))]),
}

# rows of a 16-bit engine that must lie within the tolerance: a rounding can tip a narrow choice of experts, which swaps the
# feed-forward output of that row (and, weakly, of the rows that read it)
SHARE = {"odd": 0.8, "mixed": 0.9}


def model(name, seed=0):
    rng = np.random.default_rng(seed)
    cfg, t = ov.random_vabanex(rng, **CONFIGS[name])
    return cfg, t, rng


@pytest.mark.parametrize("name", list(CONFIGS))
def test_whole_prompt_f32_and_bf16(name):
    cfg, t, rng = model(name)
    tokens = rng.integers(0, cfg["vocab"], 150).tolist()
    streams = []
    want = ov.forward(cfg, t, tokens, streams)
    assert len(streams) == len(cfg["layers"])
    eng = make_engine(cfg, t, torch.float32)
    taps = {}
    got = eng.step([("a", tokens, list(range(len(tokens))))], taps=taps).cpu().numpy()
    for i, s in enumerate(streams):
        assert rel_err(taps[i].cpu().numpy(), s) < 2e-5, f"layer {i}"
    assert rel_err(got, want) < 5e-5
    eng.release("a")
    eng16 = make_engine(cfg, t, torch.bfloat16)
    assert rows_close(run_whole(eng16, "a", tokens), want, 0.08, SHARE.get(name, 0.95))


@pytest.mark.parametrize("name", list(CONFIGS))
def test_prefill_against_token_by_token_decoding(name):
    cfg, t, rng = model(name, 1)
    tokens = rng.integers(0, cfg["vocab"], 200).tolist()      # decoding runs over three pages
    want = ov.forward(cfg, t, tokens)
    eng = make_engine(cfg, t, torch.float32)
    whole = run_whole(eng, "w", tokens)
    dec = run_portions(eng, "d", tokens, [1])
    assert rel_err(whole, want) < 5e-5 and rel_err(dec, want) < 5e-5
    mixed = run_portions(eng, "m", tokens, [70, 1])           # a prompt, then its last tokens one by one
    assert rel_err(mixed, dec) < 2e-5
    eng16 = make_engine(cfg, t, torch.bfloat16)
    w16 = run_whole(eng16, "w", tokens)
    d16 = run_portions(eng16, "d", tokens, [120, 1])          # decode steps replay graphs; the key walks are split
    assert rows_close(d16, w16, 0.04, SHARE.get(name, 0.95)) and rows_close(d16, want, 0.08, SHARE.get(name, 0.95))


@pytest.mark.parametrize("sizes", [[2], [3, 2, 64, 1, 5, 63, 2], [64], [65, 2, 2, 1, 127], [1, 2, 128, 2], [130, 2]])
def test_portions_of_any_size(sizes):
    cfg, t, rng = model("mixed", 2)
    tokens = rng.integers(0, cfg["vocab"], 201).tolist()
    eng = make_engine(cfg, t, torch.float32)
    whole = run_whole(eng, "w", tokens)
    assert rel_err(run_portions(eng, "p", tokens, sizes), whole) < 2e-5
    eng16 = make_engine(cfg, t, torch.bfloat16)
    w16 = run_whole(eng16, "w", tokens)
    assert rows_close(run_portions(eng16, "p", tokens, sizes), w16, 0.04, SHARE["mixed"])


@pytest.mark.parametrize("name", ["mixed", "tiles"])
def test_batches_of_unequal_requests_against_each_alone(name):
    cfg, t, rng = model(name, 3)
    lens = [1, 23, 97, 190]
    toks = [rng.integers(0, cfg["vocab"], n).tolist() for n in lens]
    for dtype, tol in ((torch.float32, 2e-5), (torch.bfloat16, None)):
        eng = make_engine(cfg, t, dtype, max_tokens=1024)
        alone = [run_whole(eng, ("a", i), tk) for i, tk in enumerate(toks)]
        got = [[] for _ in toks]
        at = [0] * len(toks)
        plan = [[20, 20, 20, 20], [0, 1, 40, 2], [0, 1, 1, 64], [0, 1, 36, 1], [0, 0, 0, 103]]
        for step in plan:
            ent, who = [], []
            for i, n in enumerate(step):
                n = min(n, lens[i] - at[i])
                if n > 0:
                    ent.append((("b", i), toks[i][at[i]:at[i] + n], list(range(n))))
                    who.append((i, n))
            out = eng.step(ent).cpu().numpy()
            o = 0
            for i, n in who:
                got[i].append(out[o:o + n])
                o, at[i] = o + n, at[i] + n
        for i in range(len(toks)):
            assert at[i] == lens[i]
            if tol is None:
                assert rows_close(np.concatenate(got[i]), alone[i], 0.04, SHARE.get(name, 0.95)), f"request {i}"
            else:
                assert rel_err(np.concatenate(got[i]), alone[i]) < tol, f"request {i}"


def test_pages_and_slots_that_are_freed_and_used_again():
    cfg, t, rng = model("odd", 4)
    toks = [rng.integers(0, cfg["vocab"], n).tolist() for n in (150, 100, 120, 64, 30)]
    fresh = [run_whole(make_engine(cfg, t, torch.float32, max_tokens=256, max_slots=2), "f", tk) for tk in toks]
    eng = make_engine(cfg, t, torch.float32, max_tokens=320, max_slots=2)      # 5 pages, 2 slots
    assert eng.state.num_pages == 5
    a = run_portions(eng, "a", toks[0], [64, 1, 85])                           # 3 pages, released
    assert eng.state.used_pages() == 0
    b = eng.step([("b", toks[1][:90], list(range(90))), ("c", toks[2][:40], list(range(40)))]).cpu().numpy()
    b2 = eng.step([("b", toks[1][90:], list(range(10))), ("c", toks[2][40:], list(range(80)))]).cpu().numpy()
    assert eng.state.used_pages() == 4
    with pytest.raises(RuntimeError):
        eng.step([("d", toks[3], [])])                                         # no slot left
    eng.release("b")
    d = eng.step([("d", toks[3], list(range(64))), ("c", [], [])]).cpu().numpy()   # b's slot and pages, dirty from b
    eng.release("c")
    e = run_whole(eng, "e", toks[4])
    eng.release("d")
    assert eng.state.used_pages() == 0 and len(eng.state.free_slots) == 2
    assert rel_err(a, fresh[0]) < 2e-5 and rel_err(np.concatenate([b[:90], b2[:10]]), fresh[1]) < 2e-5
    assert rel_err(np.concatenate([b[90:], b2[10:]]), fresh[2]) < 2e-5
    assert rel_err(d, fresh[3]) < 2e-5 and rel_err(e, fresh[4]) < 2e-5


def test_the_first_tokens_of_a_sequence():
    cfg, t, rng = model("tiles", 5)
    tokens = rng.integers(0, cfg["vocab"], 6).tolist()
    want = ov.forward(cfg, t, tokens)
    for dtype, tol in ((torch.float32, 5e-5), (torch.bfloat16, 0.08)):
        eng = make_engine(cfg, t, dtype)
        assert rel_err(run_whole(eng, "a", tokens[:1]), want[:1]) < tol      # one key
        got = run_portions(eng, "b", tokens, [1, 2, 3])
        assert rel_err(got, want) < tol if dtype == torch.float32 else rows_close(got, want, tol, 0.8)
    second = run_whole(eng, "c", tokens[1:2])
    assert rel_err(got[1:2], second) > 1e-3                                  # a token at position 1 is not that token at position 0


def test_far_tokens_decide_the_logits_pages_later():
    """sharp scores: the logits of the last rows change visibly when tokens more than 230 positions (three pages and more) back are
    others"""
    rng = np.random.default_rng(8)
    cfg, t = ov.random_vabanex(rng, [({"scale": 1.5}, None), ({"scale": 1.5, "heads": 2, "vdim": 8}, ("moe",))])
    a = [int(x) for x in rng.integers(0, cfg["vocab"], 330)]
    b = [int(x) for x in rng.integers(0, cfg["vocab"], 100)] + a[100:]
    wa, wb = ov.forward(cfg, t, a)[-20:], ov.forward(cfg, t, b)[-20:]
    assert rel_err(wa, wb) > 1e-2
    eng = make_engine(cfg, t, torch.float32)
    ga = run_portions(eng, "a", a, [310, 1])[-20:]                            # the last 20 tokens decoded alone, 5 pages on
    gb = run_portions(eng, "b", b, [2, 150, 158, 1])[-20:]
    assert rel_err(ga, wa) < 5e-5 and rel_err(gb, wb) < 5e-5
    eng16 = make_engine(cfg, t, torch.bfloat16)
    assert rows_close(run_portions(eng16, "a", a, [310, 1])[-20:], wa, 0.08, 0.8)


def test_long_decoding():
    cfg, t, rng = model("mixed", 10)
    tokens = rng.integers(0, cfg["vocab"], 170).tolist()
    want = ov.forward(cfg, t, tokens)
    eng16 = make_engine(cfg, t, torch.bfloat16)
    got = run_portions(eng16, "d", tokens, [10, 1])                           # 160 decoded tokens, three pages
    assert rows_close(got, want, 0.08, SHARE["mixed"])
    eng = make_engine(cfg, t, torch.float32)
    assert rel_err(run_portions(eng, "d", tokens, [10, 1]), want) < 5e-5


def test_greedy_generation_through_the_scheduler():
    cfg, t, rng = model("mixed", 6)
    prompts = [rng.integers(0, cfg["vocab"], n).tolist() for n in (5, 41, 18)]
    new = 12
    want = []
    for p in prompts:
        seq = list(p)
        for _ in range(new):
            seq.append(int(np.argmax(ov.forward(cfg, t, seq)[-1])))
        want.append(seq[len(p):])
    eng = make_engine(cfg, t, torch.float32, max_tokens=192, max_slots=2)      # the third prompt waits for a slot
    got = eng.generate(prompts, max_new_tokens=new, token_budget=24, max_chunk=16)
    assert got == want
    assert eng.state.used_pages() == 0 and not eng.state.live
    sampled = eng.generate(prompts[:2], max_new_tokens=4, sampling={"top_k": 5, "top_p": 0.9, "temperature": 0.8, "seed": 3})
    assert all(len(s) == 4 and all(0 <= x < cfg["vocab"] for x in s) for s in sampled)


def test_decode_steps_replayed_as_graphs_equal_eager_steps(monkeypatch):
    cfg, t, rng = model("tiles", 7)
    toks = [rng.integers(0, cfg["vocab"], n).tolist() for n in (90, 150, 40)]

    def run(eng):
        out = []
        eng.step([("a", toks[0][:50], []), ("b", toks[1][:100], [])])
        for i in range(25):
            out.append(eng.step([("a", [toks[0][50 + i]], [0]), ("b", [toks[1][100 + i]], [0])]).cpu().numpy().copy())
            if i == 10:
                torch.cuda.synchronize()
                eng.step([("c", toks[2][:30], [])])      # a prompt's portion between two replays
        for i in range(10):
            out.append(eng.step([("a", [toks[0][75 + i]], [0]), ("b", [toks[1][125 + i]], [0]), ("c", [toks[2][30 + i]], [0])]).cpu().numpy().copy())
        return out
    graphed = make_engine(cfg, t, torch.bfloat16)
    assert graphed.use_graphs
    got = run(graphed)
    assert any(g["graph"] is not None for g in graphed._graphs.values())
    monkeypatch.setenv("DIHIP_SEQ_GRAPH", "0")
    eager = make_engine(cfg, t, torch.bfloat16)
    assert not eager.use_graphs
    want = run(eager)
    for a, b in zip(got, want):
        assert np.array_equal(a, b)


def test_a_checkpoint_folder_is_served(tmp_path):
    """config.json + model.safetensors (bf16) of a folder -> the class by its architecture, the engine, the oracle's logits"""
    cfg, t, rng = model("mixed", 9)
    head, blob = {}, b""
    for k, v in t.items():
        raw = (np.ascontiguousarray(v, np.float32).view(np.uint32) >> 16).astype("<u2").tobytes()
        head[k] = {"dtype": "BF16", "shape": list(v.shape), "data_offsets": [len(blob), len(blob) + len(raw)]}
        blob += raw
    meta = json.dumps(head).encode()
    (tmp_path / "model.safetensors").write_bytes(struct.pack("<Q", len(meta)) + meta + blob)
    (tmp_path / "config.json").write_text(json.dumps(cfg))
    load_pkg()
    from dash_infer_amd.engine import SeqEngine
    eng = SeqEngine.from_pretrained(str(tmp_path), dtype=torch.float32, max_tokens=256, max_slots=2)
    tokens = rng.integers(0, cfg["vocab"], 70).tolist()
    assert rel_err(run_whole(eng, "a", tokens), ov.forward(cfg, t, tokens)) < 5e-5
    bad = json.loads(json.dumps(cfg))
    bad["layers"][0]["mixer"]["rot"]["dims"] = 4
    (tmp_path / "config.json").write_text(json.dumps(bad))
    with pytest.raises(ValueError):
        SeqEngine.from_pretrained(str(tmp_path), dtype=torch.float32, max_tokens=256, max_slots=2)
