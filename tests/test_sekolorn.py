"""Sekolorn on the CPU: configuration, checkpoint files, engine bookkeeping, and the plain implementation against itself
(cut sequences, planted mistakes). The kernels are in test_sekolorn_gpu.py."""
import json
import struct

import numpy as np
import pytest
import torch

import sekolorn_models as S
import sekolorn_oracle as O
from nats_llm_studio_amd.models.registry import checkpoint_kind, stack_arch, supported_architectures
from nats_llm_studio_amd.models.stack_config import StackConfig, is_stack_dir
from nats_llm_studio_amd.safetensors_io import SafetensorsReader, write_safetensors


def test_safetensors_round_trip(tmp_path):
    p = str(tmp_path / "a.safetensors")
    t = {"a": torch.randn(3, 5).to(torch.bfloat16), "b": torch.arange(7, dtype=torch.int32), "c": torch.randn(2, 2, 2)}
    write_safetensors(p, t)
    r = SafetensorsReader(p)
    assert set(r.keys()) == set(t)
    for k, v in t.items():
        assert r.shape(k) == tuple(v.shape) and torch.equal(r.tensor(k), v)
    raw = open(p, "rb").read()
    n = struct.unpack("<Q", raw[:8])[0]
    head = json.loads(raw[8:8 + n])
    head["a"]["data_offsets"][1] += 2
    bad = json.dumps(head).encode()
    open(p, "wb").write(struct.pack("<Q", len(bad)) + bad + raw[8 + n:])
    with pytest.raises(ValueError, match="data_offsets"):
        SafetensorsReader(p)
    open(p, "wb").write(struct.pack("<Q", 1 << 40))
    with pytest.raises(ValueError, match="header"):
        SafetensorsReader(p)


@pytest.mark.parametrize("name", S.CONFIGS)
def test_config(name):
    cfg = S.CONFIGS[name]
    W = S.make_weights(cfg)
    shape = lambda n: tuple(W[n].shape) if n in W else None     # noqa: E731
    c = StackConfig.from_json(cfg, shape)
    assert (c.d_model, c.vocab, c.eps, c.n_layer) == (cfg["width"], cfg["vocab"], cfg["norm"]["eps"], len(cfg["layers"]))
    for L, l in zip(cfg["layers"], c.layers):
        assert l.mixer.kind == L["type"] and l.mixer.heads == L["mixer"]["heads"]
        assert (l.mlp is None) == (L.get("mlp") is None)
        if l.mixer.kind == "latent_attention":
            assert l.mixer.kv_from == L["mixer"].get("kv_from") and l.mixer.scale == L["mixer"]["scale"]
        if l.mlp:
            g = L["mlp"]["router"].get("groups", {"count": 1, "keep": 1})
            assert (l.mlp.groups, l.mlp.keep) == (g["count"], g["keep"])
            assert l.mlp.shared_ff == (L["mlp"]["shared"]["ff"] if L["mlp"].get("shared") else 0)
    # sizes that the config leaves out come from the tensors
    lean = json.loads(json.dumps(cfg))
    for k in ("width", "vocab"):
        lean.pop(k)
    for L in lean["layers"]:
        for k in ("dim", "vdim", "kv_rank", "q_rank"):
            L["mixer"].pop(k, None)
        if L.get("mlp"):
            L["mlp"]["router"].pop("experts")
            L["mlp"]["expert"].pop("ff")
    c2 = StackConfig.from_json(lean, shape)
    for a, b in zip(c.layers, c2.layers):
        if a.mixer.kind == "latent_attention":
            assert a.mixer == b.mixer and a.mlp == b.mlp


def test_config_refusals():
    base = S.CONFIGS["uneven"]

    def bad(edit, exc=ValueError):
        c = json.loads(json.dumps(base))
        edit(c)
        with pytest.raises(exc):
            StackConfig.from_json(c)
    bad(lambda c: c.update(architecture="Nothing"), NotImplementedError)
    bad(lambda c: c["layers"][0].update(type="other"), NotImplementedError)
    bad(lambda c: c["layers"][0]["mlp"].update(kind="dense9"), NotImplementedError)
    bad(lambda c: c["layers"][2]["mixer"].update(kv_from=1))          # not a latent layer
    bad(lambda c: c["layers"][2]["mixer"].update(kv_from=3))          # not an earlier layer
    bad(lambda c: c["layers"][2]["mixer"].update(kv_rank=41))         # another latent size
    bad(lambda c: c["layers"][0]["mixer"]["rot"].update(dims=6))      # a part of the rotated part
    bad(lambda c: c["layers"][0]["mlp"]["router"].update(top=9))      # more than the kept groups hold


def test_registry(tmp_path):
    cfg = S.CONFIGS["ones"]
    d = S.write_model(str(tmp_path / "m"), cfg, S.make_weights(cfg))
    assert is_stack_dir(d) and checkpoint_kind(d) == "stack" and checkpoint_kind(d + "/config.json") == "stack"
    assert stack_arch(d) == "Sekolorn" and "Sekolorn" in supported_architectures()
    with pytest.raises(FileNotFoundError):
        checkpoint_kind(str(tmp_path))
    json.dump({"architecture": "Nothing"}, open(d + "/config.json", "w"))
    assert stack_arch(d) is None


def test_service_registry_lists_folder_models(tmp_path):
    from nats_llm_studio_amd.service.registry import Registry
    cfg = S.CONFIGS["ones"]
    d = S.write_model(str(tmp_path / "pub" / "Tiny-Seko"), cfg, S.make_weights(cfg))
    reg = Registry(str(tmp_path))
    (e,) = reg.scan()
    assert e.id == "tiny-seko" and e.arch == "Sekolorn" and e.quantization == "BF16" and e.path == d
    api = reg.list_api()["data"][0]
    assert api["compatibility_type"] == "safetensors" and api["size_bytes"] > 1000
    assert reg.resolve("pub/Tiny-Seko") is not None


def test_id_tokenizer():
    from nats_llm_studio_amd.tokenizer.ids import IdTokenizer
    t = IdTokenizer(50)
    assert t.encode("3 17\n49") == [3, 17, 49] and t.decode([3, 17, 49]) == "3 17 49"
    assert all(0 <= i < 50 for i in t.encode("hello 99"))       # words become bytes, folded into the vocabulary
    from nats_llm_studio_amd.tokenizer.bpe import StreamDecoder
    sd = StreamDecoder(t)
    assert "".join(sd.push(i) or "" for i in (3, 17)).split() == ["3", "17"]


def test_state_slots():
    from nats_llm_studio_amd.engine.engine import StateSlots
    s = StateSlots(2)
    a, b = s.alloc(), s.alloc()
    assert {a, b} == {0, 1} and s.alloc() is None
    s.release(a)
    assert s.alloc() == a


class _FakeRecurrent:
    """A stand-in model: checks what the engine hands a recurrent model, and answers with a counter as the token."""
    recurrent, prefill_graphs, ep, format = True, False, False, "safetensors"
    kv_token_bytes = 4

    def __init__(self, vocab=64):
        from types import SimpleNamespace
        from nats_llm_studio_amd.models.llama import ShardSpec
        self.cfg = SimpleNamespace(ctx=256, vocab=vocab, n_layer=1, n_expert=0, n_expert_used=0, arch="fake")
        self.device, self.shard, self.comm = torch.device("cpu"), ShardSpec(), None
        self.vocab_lo, self.vocab_hi, self.ended = 0, vocab, []

    def n_splits(self, T):
        return 1

    def kv_cache(self, nb, bs):
        self.rows = {}
        return {}, None

    def state_pool(self, n):
        return {"last": [None] * n}

    def step_buffers(self, cap, ms, mb, logit_rows=None):
        from types import SimpleNamespace
        pad = (cap + 63) // 64 * 64
        meta = torch.zeros(6 * pad + ms * mb + 4 * ms, dtype=torch.int32)
        s = [meta[i * pad:(i + 1) * pad] for i in range(6)]
        return SimpleNamespace(pad=pad, meta=meta, ids=s[0], pos=s[1], slot=s[2], tok_seq=s[3], ctx_len=s[4], use_prev=s[5],
                               block_tables=meta[6 * pad:6 * pad + ms * mb].view(ms, mb),
                               runs=meta[6 * pad + ms * mb:].view(ms, 4), logits=torch.zeros(max(64, logit_rows or 0), self.cfg.vocab),
                               next_ids=torch.zeros(pad, dtype=torch.int32))

    def forward(self, b, kc, vc, T, bs, ns=1, logit_rows=None, n_logits=None, qblocks=None, nqb=0, feed_prev=False,
                need_logits=True, state=None, nruns=None):
        if feed_prev:
            b.ids[:T] = torch.where(b.use_prev[:T] != 0, b.next_ids[:T], b.ids[:T])
        last = state["last"]
        vals = torch.zeros(T, dtype=torch.int64)
        seen = 0
        for r in range(nruns):
            t0, n, slot, p0 = b.runs[r].tolist()
            if slot < 0 or n == 0:
                continue
            seen += n
            assert b.tok_seq[t0:t0 + n].eq(r).all() and b.pos[t0:t0 + n].tolist() == list(range(p0, p0 + n))
            h = (0, 0) if p0 == 0 else last[slot]
            assert h is not None and h[0] == p0, (h, p0)           # the slot holds this sequence up to p0
            for t in range(t0, t0 + n):
                h = (h[0] + 1, (h[1] * 31 + int(b.ids[t])) % 1009)
                vals[t] = h[1]
            last[slot] = h
        assert seen == T or feed_prev
        pick = torch.arange(T) if logit_rows is None else logit_rows[:n_logits].long()
        b.logits[:len(pick)] = 0
        b.logits[torch.arange(len(pick)), vals[pick] % self.cfg.vocab] = 1.0
        b.next_ids[:len(pick)] = b.logits[:len(pick)].argmax(1).int()
        return len(pick)


def _fake_next(toks, vocab=64):
    h = 0
    for t in toks:
        h = (h * 31 + t) % 1009
    return h % vocab


@pytest.mark.parametrize("blocks", [200, 8])
def test_engine_state_slots_follow_sequences(blocks):
    """Many requests over few slots (and, with 8 blocks, preemptions): every run starts where its slot's state ends."""
    from nats_llm_studio_amd.engine.engine import Engine, GenRequest
    from nats_llm_studio_amd.engine.sampling import SamplingParams
    m = _FakeRecurrent()
    eng = Engine(m, None, max_batch=3, num_blocks=blocks, max_prefill_tokens=24, ctx=128, use_graphs=False)
    assert eng.slots is not None and not eng.alloc.cache_enabled
    eng.gen_ratio = 0.0                  # admit on the prompts alone
    reqs = [(S.tokens(5 + 13 * i, 64, i), 20 + 3 * i) for i in range(6)]
    futs = [eng.submit(GenRequest(p, SamplingParams(max_tokens=n, ignore_eos=True))) for p, n in reqs]
    for _ in range(2000):
        if all(f.done() for f in futs):
            break
        eng.step()
    for (p, n), f in zip(reqs, futs):
        want = list(p)
        for _ in range(n):
            want.append(_fake_next(want))
        assert f.result().token_ids == want[len(p):]
    assert len(eng.slots.free) == 3 and eng.alloc.n_free == blocks
    assert blocks == 200 or eng.counters["preemptions"] > 0


def test_engine_feed_bookkeeping():
    from nats_llm_studio_amd.engine.engine import Engine
    m = _FakeRecurrent()
    eng = Engine(m, None, max_batch=2, num_blocks=8, max_prefill_tokens=16, ctx=96, use_graphs=False, max_logit_rows=3)
    a, b = S.tokens(70, 64, 1), S.tokens(20, 64, 2)
    (la,) = eng.feed([("a", a[:40], list(range(40)))])           # larger than a row batch and than its wanted rows
    assert [int(r.argmax()) for r in la] == [_fake_next(a[:i + 1]) for i in range(40)]
    la, lb = eng.feed([("a", a[40:41], [0]), ("b", b[:9], [8, 2])])
    assert int(la[0].argmax()) == _fake_next(a[:41])
    assert [int(r.argmax()) for r in lb] == [_fake_next(b[:9]), _fake_next(b[:3])]
    la, lb = eng.feed([("a", a[41:42], [0]), ("b", b[9:10], [])])    # a decode step
    assert int(la[0].argmax()) == _fake_next(a[:42]) and lb.shape[0] == 0
    with pytest.raises(RuntimeError, match="live"):
        eng.feed([("c", [1], [])])
    (lb,) = eng.feed([("b", b[10:11], [0])])                          # "a" is left out
    assert int(lb[0].argmax()) == _fake_next(b[:11])
    eng.feed_end("a")
    (lc,) = eng.feed([("c", a[:50], [49])])                           # a's slot and blocks again
    assert int(lc[0].argmax()) == _fake_next(a[:50])
    with pytest.raises(RuntimeError, match="pool"):
        eng.feed([("c", a[:46], []), ("b", a[:40], [])])
    for r in "bc":
        eng.feed_end(r)
    assert eng.alloc.n_free == 8 and len(eng.slots.free) == 2
    with pytest.raises(ValueError, match="vocabulary"):
        eng.feed([("d", [64], [])])


# ---- the plain implementation against itself

def test_oracle_cut_sequences():
    """Every mixer fed in pieces, with its carried state or cached rows, equals one pass."""
    cfg = S.CONFIGS["uneven"]
    W = {k: v.double() for k, v in S.make_weights(cfg).items()}
    eps = cfg["norm"]["eps"]
    h = torch.randn(23, cfg["width"], generator=torch.Generator().manual_seed(3), dtype=torch.float64)
    mix = cfg["layers"][1]["mixer"]
    whole, _ = O.wkv_mixer(h, W, "l1.mix.", mix, eps)
    st, out = None, []
    for a, b in ((0, 1), (1, 3), (3, 16), (16, 23)):
        y, st = O.wkv_mixer(h[a:b], W, "l1.mix.", mix, eps, st)
        out.append(y)
    assert torch.allclose(torch.cat(out), whole, atol=1e-10)
    mix = cfg["layers"][0]["mixer"]
    pos = torch.arange(23)
    c, kr = O.latent_rows(h, W, "l0.mix.", mix, pos, eps)
    whole = O.latent_mixer(h, W, "l0.mix.", mix, pos, eps, c, kr)
    out = [O.latent_mixer(h[a:b], W, "l0.mix.", mix, pos[a:b], eps, c[:b], kr[:b]) for a, b in ((0, 2), (2, 17), (17, 23))]
    assert torch.allclose(torch.cat(out), whole, atol=1e-10)


def test_oracle_known_values():
    """Hand-computed cases."""
    assert torch.allclose(O.layer_norm(torch.tensor([1.0, 3.0]), torch.tensor([2.0, 5.0]), 0.0), torch.tensor([-2.0, 5.0]))
    x = torch.tensor([[3.0, 4.0]])
    assert torch.allclose(O.rms_norm(x, None, 0.5), x / (13.0 ** 0.5))
    r = O.rotate(torch.tensor([[1.0, 0.0, 1.0, 0.0]], dtype=torch.float64), torch.tensor([2]), 100.0, 4)
    a = torch.tensor([2.0, 0.2], dtype=torch.float64)
    assert torch.allclose(r[0], torch.stack([a.cos(), a.sin()], 1).reshape(-1))
    z = torch.logit(torch.tensor([.9, .1, .5, .45, .8, .05, .3, .2], dtype=torch.float64))
    # pairs: 1.0, .95, .85, .5 -> groups 0 and 1; experts 0 (.9) and 2 (.5), not 4 (.8)
    got = O.route(z, 2, 3.0, 4, 2)
    assert [e for e, _ in got] == [0, 2] and abs(float(got[0][1]) - 2.7) < 1e-9
    assert [e for e, _ in O.route(z, 2, 3.0, 1, 1)] == [0, 4]
    o, Sx = O.wkv_scan(torch.ones(2, 1, 1), torch.tensor([[[2.0]], [[3.0]]]), torch.tensor([[[5.0]], [[7.0]]]),
                       torch.tensor([[[.5]], [[.25]]]), torch.tensor([[4.0]]))
    assert o.flatten().tolist() == [40.0, 10.0 + 84.0] and float(Sx) == 2.5 + 21.0


MISTAKES = {
    "a key is missed": lambda m: m.setattr(O, "latent_rows", _drop_key(O.latent_rows)),
    "the shared key part is not rotated": lambda m: m.setattr(O, "rotate", lambda x, *a: x),
    "the token shift is lost": lambda m: m.setattr(O, "token_shift", lambda h, prev: h),
    "no bonus for the current token": lambda m: m.setattr(O, "wkv_scan", _no_bonus(O.wkv_scan)),
    "groups are ignored": lambda m: m.setattr(O, "route", lambda z, t, s, g, k, f=O.route: f(z, t, s, 1, 1)),
    "weights are renormalized": lambda m: m.setattr(O, "route", _renorm(O.route)),
}


def _drop_key(f):
    def g(*a):
        c, kr = f(*a)
        return torch.cat([c[:7], c[6:7], c[8:]]), torch.cat([kr[:7], kr[6:7], kr[8:]])
    return g


def _no_bonus(f):
    return lambda r, k, v, w, u, state=None: f(r, k, v, w, torch.zeros_like(u), state)


def _renorm(f):
    def g(*a):
        out = f(*a)
        t = sum(w for _, w in out)
        return [(e, w / t) for e, w in out]
    return g


@pytest.mark.parametrize("mistake", MISTAKES)
def test_weights_show_mistakes(mistake, monkeypatch):
    """The tests' weights make each mistake visible well above what bf16 rounding does (test_sekolorn_gpu.BF16)."""
    cfg = S.CONFIGS["uneven"]
    W, toks = S.make_weights(cfg), S.tokens(48, cfg["vocab"])
    good = O.forward(cfg, W, toks)
    MISTAKES[mistake](monkeypatch)
    assert S.error(O.forward(cfg, W, toks), good) > 0.2


def test_bench_option_parses():
    import bench
    a = bench.parse([])
    assert a.stack is None and a.model == "llama-3-8b" and a.steps == 200
    assert bench.parse(["--stack", "decode"]).stack == "decode"
    assert np.prod(bench.parse(["--stack", "all"]).gpus) == 1
