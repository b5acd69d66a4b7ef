"""Cases for the token language models, run on the kernel simulator (test_tlm_sim.py) and on the GPU (test_d_tlm_gpu.py): the engine
against the plain oracle (oracle/token_lm_oracle.py) on small random networks of this file's own sizes."""
from __future__ import annotations

from dataclasses import replace

import numpy as np
import torch

from moshi_amd.config import (BigramConfig, ChannelDeltaConfig, DenseGLUConfig, GroupedAttentionConfig, LatentAttentionConfig, LightningConfig, MinGRUConfig,
                              MoEConfig, TokenLayerConfig, TokenLMConfig, tiny_bibapel_config, tiny_token_lm_config)
from moshi_amd.tlm import TokenLM
from moshi_amd.token_batcher import TokenBatcher
from moshi_amd.weights import random_token_lm_state_dict
from oracle.token_lm_oracle import TokenLMOracle, rms_norm

F32, BF16 = torch.float32, torch.bfloat16
TOL = {F32: 2e-5, BF16: 4e-2}           # of the logits' RMS (mean removed), worst position

ATT = LatentAttentionConfig(heads=3, dim=24, vdim=20, rot_dim=12, q_rank=40, kv_rank=36, scale=0.17, rot_base=5000.0, window=37)
MOE = MoEConfig(experts=5, top=2, ff=44)


def one_layer(mixer, mlp=None, **kw):
    base = dict(architecture="Kesirax", vocab=67, width=48, norm_groups=2, norm_eps=1e-5, logit_scale=1.3, layers=[TokenLayerConfig(mixer, mlp)])
    base.update(kw)
    return TokenLMConfig(**base)


MECHANISMS = {
    "mingru": one_layer(MinGRUConfig(40)),
    "mingru_wide": one_layer(MinGRUConfig(272)),
    "mingru_experts": one_layer(MinGRUConfig(16), MOE),
    "every_expert": one_layer(MinGRUConfig(16), MoEConfig(experts=3, top=3, ff=16)),
    "one_expert": one_layer(MinGRUConfig(16), MoEConfig(experts=1, top=1, ff=8)),
    "attention": one_layer(ATT),
    "attention_experts": one_layer(ATT, MOE),
    "one_head": one_layer(replace(ATT, heads=1, vdim=16, rot_dim=2)),
    "many_heads": one_layer(replace(ATT, heads=18, dim=8, vdim=12)),
    "window_one": one_layer(replace(ATT, window=1)),
    "no_window": one_layer(replace(ATT, window=0)),
    "wide_latent": one_layer(replace(ATT, kv_rank=200, q_rank=17, rot_dim=40)),
    "widest_latent": one_layer(replace(ATT, kv_rank=500, q_rank=33, rot_dim=128, heads=2)),
    "latent_of_eight_tiles": one_layer(replace(ATT, kv_rank=120, rot_dim=66, heads=5)),
    "latent_of_one_tile": one_layer(replace(ATT, kv_rank=16, dim=32, vdim=32, rot_dim=32)),
    "one_group": one_layer(MinGRUConfig(24), norm_groups=1),
    "six_groups": one_layer(MinGRUConfig(24), norm_groups=6),
    "odd_width": one_layer(ATT, MOE, width=42, norm_groups=7),
    "repeated": one_layer(None, layers=[TokenLayerConfig(MinGRUConfig(24), MOE), TokenLayerConfig(ATT, None)], loop_start=0, loop_stop=2, loop_times=3),
    "repeated_one": one_layer(None, layers=[TokenLayerConfig(MinGRUConfig(24), None), TokenLayerConfig(ATT, MOE), TokenLayerConfig(MinGRUConfig(32), MOE)],
                              loop_start=1, loop_stop=2, loop_times=2),
    "two_windows": one_layer(None, layers=[TokenLayerConfig(ATT, None), TokenLayerConfig(replace(ATT, window=5, heads=2, rot_base=300.0, rot_dim=8), MOE)]),
    "mixed": tiny_token_lm_config(),
}

GQA = GroupedAttentionConfig(heads=6, kv_heads=2, dim=24, vdim=20, scale=0.3, window=37, keep_first=5, sink=True)
DELTA = ChannelDeltaConfig(heads=4, kv_heads=2, dim=20, vdim=24, conv=3, decay_rank=10, gate_rank=14)
LIGHT = LightningConfig(heads=3, dim=18, vdim=28, decay=[0.7, 0.93, 0.995])
GLU = DenseGLUConfig(ff=44, limit=1.2)


def plain_layer(mixer, mlp=None, **kw):
    """One layer of the two-norm kind: no layer scales, the head is the embedding table."""
    base = dict(architecture="Bibapel", vocab=67, width=48, norm_eps=1e-5, layers=[TokenLayerConfig(mixer, mlp)], norms=2, layer_scales=False, tied_head=True,
                loop_inject="project")
    base.update(kw)
    return TokenLMConfig(**base)


MECHANISMS.update({
    "grouped_attention": plain_layer(GQA),
    "grouped_attention_own_heads": plain_layer(replace(GQA, heads=3, kv_heads=3, keep_first=0, sink=False)),
    "grouped_attention_one_kv_head": plain_layer(replace(GQA, heads=5, kv_heads=1, vdim=33)),
    "grouped_attention_one_head": plain_layer(replace(GQA, heads=1, kv_heads=1, window=1, keep_first=1)),
    "grouped_attention_no_window": plain_layer(replace(GQA, window=0, keep_first=0)),
    "grouped_attention_keeps_more_than_it_sees": plain_layer(replace(GQA, window=3, keep_first=40)),
    "grouped_attention_wide": plain_layer(replace(GQA, heads=4, kv_heads=2, dim=100, vdim=72, scale=0.1)),
    "grouped_attention_widest": plain_layer(replace(GQA, heads=2, kv_heads=1, dim=200, vdim=256, scale=0.07)),
    "delta": plain_layer(DELTA),
    "delta_own_heads_no_conv": plain_layer(replace(DELTA, heads=3, kv_heads=3, conv=1, vdim=16, dim=16)),
    "delta_wide_long_conv": plain_layer(replace(DELTA, heads=2, kv_heads=1, dim=72, vdim=40, conv=7, decay_rank=1, gate_rank=70)),
    "delta_widest": plain_layer(replace(DELTA, heads=1, kv_heads=1, dim=256, vdim=208, conv=2)),
    "lightning": plain_layer(LIGHT),
    "lightning_decay_ends": plain_layer(replace(LIGHT, decay=[0.0, 1.0, 0.5])),
    "lightning_wide": plain_layer(LightningConfig(heads=2, dim=136, vdim=100, decay=[0.9, 0.97])),
    "glu": plain_layer(LIGHT, GLU),
    "glu_odd": plain_layer(replace(LIGHT, heads=1, decay=[0.8]), DenseGLUConfig(ff=37, limit=0.5), width=42),
    "bigram": plain_layer(LIGHT, None, bigram=BigramConfig(buckets=13, mul_prev=5, mul_cur=3), embed_scale=0.5),
    "positions": plain_layer(LIGHT, None, max_positions=200, embed_scale=2.0),
    "projected_passes": plain_layer(None, layers=[TokenLayerConfig(DELTA, GLU), TokenLayerConfig(GQA, None)], loop_start=0, loop_stop=2, loop_times=3),
    "projected_pass_of_one": plain_layer(None, layers=[TokenLayerConfig(LIGHT, GLU), TokenLayerConfig(GQA, GLU), TokenLayerConfig(DELTA, GLU)], width=40,
                                         loop_start=1, loop_stop=2, loop_times=1, max_positions=150, bigram=BigramConfig(buckets=29, mul_prev=7, mul_cur=2)),
    "two_kept_windows": plain_layer(None, layers=[TokenLayerConfig(GQA, None), TokenLayerConfig(replace(GQA, window=9, keep_first=70, heads=4, kv_heads=4), GLU)]),
    "bibapel": tiny_bibapel_config(),
})


def make(cfg, dev, lib, dtype=F32, seed=5, **kw):
    sd = random_token_lm_state_dict(cfg, seed=seed)
    args = dict(max_slots=6, max_tokens=1024)
    args.update(kw)
    return TokenLM(sd, cfg, device=dev, dtype=dtype, lib=lib, **args), TokenLMOracle(sd, cfg)


def tokens_of(cfg, n, seed=0):
    return np.random.default_rng(seed).integers(0, cfg.vocab, n).tolist()


def rel(got, want):
    """Worst position: RMS of the difference over the vocabulary (means removed) / RMS of all the wanted logits."""
    got, want = np.asarray(got, np.float64), np.asarray(want, np.float64)
    d = got - want
    d -= d.mean(axis=-1, keepdims=True)
    w = want - want.mean(axis=-1, keepdims=True)
    return float(np.sqrt((d * d).mean(axis=-1)).max() / np.sqrt((w * w).mean()))


def run_cut(lm, toks, cuts, slot=None):
    """Logits of every token, the prompt fed in portions of the given sizes (the last size repeats)."""
    own = slot is None
    slot = lm.open() if own else slot
    out, at, i = [], 0, 0
    while at < len(toks):
        n = min(cuts[min(i, len(cuts) - 1)], len(toks) - at)
        out.append(lm.step([(slot, toks[at:at + n], list(range(n)))]).cpu().numpy().copy())
        at += n
        i += 1
    if own:
        lm.close(slot)
    return np.concatenate(out)


# ---- one mechanism at a time ---------------------------------------------------------------------------------------------------
def check_mechanism(name, dev, lib, dtype=F32, n=90):
    """Whole prompt (tiled kernels), its short head (row kernels), and the residual stream after every layer run."""
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype)
    toks = tokens_of(cfg, n)
    want_taps = []
    want = orc.logits(toks, want_taps)
    assert rel(run_cut(lm, toks, [n]), want) < TOL[dtype]
    assert rel(run_cut(lm, toks[:21], [21]), want[:21]) < TOL[dtype]
    if cfg.width % 16 == 0:
        slot = lm.open()
        _, taps = lm.step_with_taps([(slot, toks, [0])])
        lm.close(slot)
        for got, ref in zip(taps.cpu().numpy(), want_taps):
            assert np.abs(got - ref).max() < TOL[dtype] * np.sqrt((ref * ref).mean()) * 8
    assert lm.free_pages == lm.total_pages and lm.free_slots == 6


def check_activation_branches(dev, lib):
    """Both branches of the candidate (u >= 0 and u < 0), gates near 0 and near 1, inputs of squared ReLU on both sides of zero: biases
    push whole channels to each side."""
    cfg = MECHANISMS["mingru_experts"]
    sd = random_token_lm_state_dict(cfg, seed=9)
    sd["l0.mix.x.b"] = torch.linspace(-6, 6, 16).to(BF16)
    sd["l0.mix.z.b"] = torch.linspace(5, -5, 16).to(BF16)
    lm = TokenLM(sd, cfg, device=dev, dtype=F32, lib=lib, max_slots=2, max_tokens=256)
    toks = tokens_of(cfg, 70)
    assert rel(run_cut(lm, toks, [70]), TokenLMOracle(sd, cfg).logits(toks)) < TOL[F32]


# ---- how a sequence is fed -----------------------------------------------------------------------------------------------------
def check_portions(dev, lib, dtype=F32, n=132, cut_sets=((2,), (3, 2, 61, 7), (64,), (65, 1), (127, 2), (33,)), name="mixed"):
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype)
    toks = tokens_of(cfg, n, seed=1)
    want = orc.logits(toks)
    whole = run_cut(lm, toks, [n])
    assert rel(whole, want) < TOL[dtype]
    for cuts in cut_sets:
        assert rel(run_cut(lm, toks, list(cuts)), want) < TOL[dtype], cuts


def check_prompt_then_decode(dev, lib, dtype=F32, n=110, tail=30, name="mixed"):
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype)
    toks = tokens_of(cfg, n, seed=2)
    assert rel(run_cut(lm, toks, [n - tail, 1]), orc.logits(toks)) < TOL[dtype]


def check_unequal_batch(dev, lib, dtype=F32, name="mixed"):
    """Requests of different lengths, portions beside single tokens, requests left out of steps: each as if it were alone."""
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype, max_tokens=2048)
    rng = np.random.default_rng(3)
    seqs = [tokens_of(cfg, n, seed=10 + i) for i, n in enumerate((131, 1, 64, 40, 97, 66))]
    slots = [lm.open() for _ in seqs]
    at, got = [0] * len(seqs), [[] for _ in seqs]
    while any(a < len(s) for a, s in zip(at, seqs)):
        entries, who = [], []
        for i in rng.permutation(len(seqs)):
            left = len(seqs[i]) - at[i]
            if left == 0 or rng.random() < 0.25:
                continue
            k = min(left, int(rng.choice([1, 1, 2, 5, 17, 64, 70])))
            entries.append((slots[i], seqs[i][at[i]:at[i] + k], list(range(k))))
            who.append((i, k))
            at[i] += k
        if not entries:
            continue
        rows = lm.step(entries).cpu().numpy()
        for i, k in who:
            got[i].append(rows[:k].copy())
            rows = rows[k:]
    for g, s in zip(got, seqs):
        assert rel(np.concatenate(g), orc.logits(s)) < TOL[dtype]


def check_batched_decode(dev, lib, dtype=F32, B=5, steps=12, name="mixed"):
    """Pure decode steps at a fixed batch (captured launches): every replay against the oracle."""
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype, max_tokens=2048)
    seqs = [tokens_of(cfg, 20 + 9 * i + steps, seed=30 + i) for i in range(B)]
    want = [orc.logits(s) for s in seqs]
    slots = [lm.open() for _ in seqs]
    for s, t in zip(slots, seqs):
        lm.step([(s, t[:-steps], [])])
    for k in range(steps):
        rows = lm.step([(s, [t[len(t) - steps + k]], [0]) for s, t in zip(slots, seqs)]).cpu().numpy()
        for r, t, w in zip(rows, seqs, want):
            assert rel(r[None], w[len(t) - steps + k][None]) < 2 * TOL[dtype]


def check_reuse(dev, lib, dtype=F32, name="mixed"):
    """Pages and slots go from request to request: a pool that holds one request at a time, earlier owners with other tokens, closed in
    the middle of a page; the last request's logits equal a fresh engine's, bit for bit."""
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype, max_slots=2, max_tokens=192)
    fresh, _ = make(cfg, dev, lib, dtype, max_slots=2, max_tokens=192)
    for i, n in enumerate((192, 70, 129)):
        run_cut(lm, tokens_of(cfg, n, seed=50 + i), [50])
    other = lm.open()
    lm.step([(other, tokens_of(cfg, 40, seed=60), [])])
    toks = tokens_of(cfg, 100, seed=61)
    got = run_cut(lm, toks, [30, 1, 69])
    assert rel(got, orc.logits(toks)) < TOL[dtype]
    assert np.array_equal(got, run_cut(fresh, toks, [30, 1, 69]))
    lm.close(other)
    assert lm.free_pages == lm.total_pages == 3


def check_long_decode(dev, lib, dtype=F32, n=330, pool=256, name="two_windows", held=2):
    """A sequence longer than the pool: pages behind every window are given back and come round again (but those with kept positions)."""
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype, max_slots=2, max_tokens=pool)
    toks = tokens_of(cfg, n, seed=4)
    slot = lm.open()
    got = run_cut(lm, toks, [130, 1], slot)
    assert rel(got, orc.logits(toks)) < TOL[dtype]
    assert lm.position(slot) == n and lm.info(5, slot) <= held          # a window of 37 spans at most two pages
    lm.close(slot)
    assert lm.free_pages == lm.total_pages


# per bound of the attention kernels' latent, heads enough for their key-staging form
WIDE_PROMPTS = {
    "latent_36": one_layer(replace(ATT, heads=26)),
    "latent_128": one_layer(replace(ATT, heads=26, kv_rank=128, rot_dim=40, window=300)),
    "latent_200": one_layer(replace(ATT, heads=26, kv_rank=200, rot_dim=80, window=0)),
    "latent_500": one_layer(replace(ATT, heads=14, kv_rank=500, rot_dim=64, window=129)),
}


# the same for grouped attention (per head-size bound of its kernels), the delta rule and lightning attention over many chunks
WIDE_PROMPTS_2 = {
    "gqa_24": plain_layer(replace(GQA, heads=26, kv_heads=2, window=90)),
    "gqa_128": plain_layer(replace(GQA, heads=28, kv_heads=4, dim=128, vdim=96, window=300, keep_first=100, scale=0.1)),
    "gqa_256": plain_layer(replace(GQA, heads=26, kv_heads=13, dim=160, vdim=256, window=0, keep_first=0, scale=0.08)),
    "delta_128": plain_layer(replace(DELTA, heads=4, kv_heads=2, dim=128, vdim=128, conv=4)),
    "delta_lightning": plain_layer(None, layers=[TokenLayerConfig(DELTA, GLU), TokenLayerConfig(replace(LIGHT, dim=128, vdim=64), None)]),
}


def check_long_prompt(dev, lib, dtype=F32, n=1300, cfg=None):
    """Enough rows for the large product tile, for attention with one column tile per wave and for scans over many segments; then
    decoding with the keys split over workgroups (no window: every key is visible)."""
    cfg = cfg or one_layer(None, layers=[TokenLayerConfig(MinGRUConfig(24), MOE), TokenLayerConfig(replace(ATT, window=0, heads=14, dim=8, vdim=8), None)])
    lm, orc = make(cfg, dev, lib, dtype, max_tokens=n + 64)
    toks = tokens_of(cfg, n, seed=6)
    want = orc.logits(toks)
    slot = lm.open()
    pick = [0, 1, 31, 32, 33, 63, 64, 65, n // 2, n - 12, n - 11]
    got = lm.step([(slot, toks[:n - 10], pick)]).cpu().numpy()
    assert rel(got, want[pick]) < TOL[dtype]
    assert rel(run_cut(lm, toks[n - 10:], [1], slot), want[n - 10:]) < TOL[dtype]
    lm.close(slot)


def check_long_prompt_beside_decoding(dev, lib, dtype=F32, n=340, name="many_kv_heads"):
    """A long portion beside single tokens and short portions of other sequences in one step: the two forms of the attention kernel and of
    the recurrences share a step, and leave each other's rows alone."""
    cfg = BESIDE[name]
    lm, orc = make(cfg, dev, lib, dtype, max_tokens=2048)
    lens = (90, 33, 70, 12)
    seqs = [tokens_of(cfg, k + 7, seed=20 + i) for i, k in enumerate(lens)]
    long = tokens_of(cfg, n, seed=30)
    slots = [lm.open() for _ in seqs]
    for s, t, k in zip(slots, seqs, lens):
        lm.step([(s, t[:k], [])])
    ls = lm.open()
    want = [orc.logits(t) for t in seqs]
    wl = orc.logits(long)
    pick = [0, 63, 64, n // 2, n - 6]
    counts = (1, 4, 1, 5)
    entries = [(s, t[k:k + c], list(range(c))) for s, t, k, c in zip(slots, seqs, lens, counts)]
    entries.insert(2, (ls, long[:n - 5], pick))
    rows = lm.step(entries).cpu().numpy()
    at = 0
    for i in (0, 1, None, 2, 3):
        m = len(pick) if i is None else counts[i]
        ref = wl[pick] if i is None else want[i][lens[i]:lens[i] + m]
        assert rel(rows[at:at + m], ref) < TOL[dtype], i
        at += m
    entries = [(s, t[k + c:k + c + 2], [0, 1]) for s, t, k, c in zip(slots, seqs, lens, counts)] + [(ls, long[n - 5:], list(range(5)))]
    rows = lm.step(entries).cpu().numpy()
    ref = np.concatenate([w[k + c:k + c + 2] for w, k, c in zip(want, lens, counts)] + [wl[n - 5:]])
    assert rel(rows, ref) < TOL[dtype]
    for s in slots + [ls]:
        lm.close(s)


BESIDE = {
    "many_kv_heads": plain_layer(replace(GQA, heads=26, kv_heads=13, window=150)),
    "all": plain_layer(None, layers=[TokenLayerConfig(DELTA, GLU), TokenLayerConfig(replace(GQA, heads=26, kv_heads=13, window=100), GLU), TokenLayerConfig(LIGHT, None)],
                       bigram=BigramConfig(buckets=29, mul_prev=7, mul_cur=2), max_positions=2000, loop_start=1, loop_stop=3, loop_times=2),
}


# ---- single keys ---------------------------------------------------------------------------------------------------------------
def _pair_that_stands_out(orc, cfg):
    """(query token, key token, plain token): of all pairs the one whose un-rotated score beats the plain token's by most."""
    w, m, p = orc.w, cfg.layers[0].mixer, "l0.mix."
    h = rms_norm(w["embed"], w["l0.norm1"], cfg.norm_eps, cfg.norm_groups)
    q = (rms_norm(h @ w[p + "dq"].T, w[p + "dq.norm"], cfg.norm_eps) @ w[p + "uq"].T).reshape(cfg.vocab, m.heads, -1)[:, :, :m.dim]
    c = rms_norm((h @ w[p + "dkv"].T)[:, :m.kv_rank], w[p + "dkv.norm"], cfg.norm_eps)
    k = (c @ w[p + "uk"].T).reshape(cfg.vocab, m.heads, m.dim)
    s = np.einsum("ahd,bhd->abh", q, k)
    low = s.min(axis=1)                                                  # the least attractive token of every (query, head)
    own = s[np.arange(cfg.vocab), np.arange(cfg.vocab)]
    gap = s - np.maximum(low, own)[:, None, :]                           # the query itself is always visible, too
    query, key, head = np.unravel_index(np.argmax(gap), gap.shape)
    return int(query), int(key), int(np.argmin(s[query, :, head]))


def check_single_keys(dev, lib, window=70, dtype=F32):
    """One key that dominates the softmax, everywhere else tokens whose score is low: at chosen distances from the query - itself, the
    neighbour, page borders, the last position inside the window, the first one outside - the logits must be the oracle's, must differ
    from a prompt without that key while it is visible, and must be bit-identical to it once it is not.  In the prompt and decoded."""
    cfg = one_layer(replace(ATT, window=window, scale=1.1, rot_dim=4, rot_base=1e6))
    sd = random_token_lm_state_dict(cfg, seed=5)
    sd["l0.ls1"] = torch.full((cfg.width,), 2.0).to(BF16)
    lm, orc = TokenLM(sd, cfg, device=dev, dtype=dtype, lib=lib, max_slots=2, max_tokens=512), TokenLMOracle(sd, cfg)
    query, key, plain = _pair_that_stands_out(orc, cfg)
    assert key not in (query, plain)
    n = 3 * 64 + 9
    for at in (n - 1, 128, 191, 64):                     # the query's position: past a page border, first of a page, last of a page
        base = [plain] * (at + 1)
        base[at] = query
        without = {mode: run_cut(lm, base, cuts)[at] for mode, cuts in (("prompt", [at + 1]), ("decoded", [at, 1]), ("two", [at - 1, 2]))}
        ref0 = orc.logits(base)[at]
        dists = [d for d in (1, 2, at % 64, at % 64 + 1, window - 2, window - 1, window, window + 1, at) if 0 < d <= at]
        for d in dists:
            toks = list(base)
            toks[at - d] = key
            ref = orc.logits(toks)[at]
            shows = window == 0 or d < window
            assert (rel(ref[None], ref0[None]) > 0.05) == shows, (at, d, "the key must show in the oracle while it is visible")
            for mode, cuts in (("prompt", [at + 1]), ("decoded", [at, 1]), ("two", [at - 1, 2])):
                got = run_cut(lm, toks, cuts)[at]
                assert rel(got[None], ref[None]) < TOL[dtype], (at, d, mode)
                if shows:
                    assert rel(got[None], without[mode][None]) > 0.05, (at, d, mode)
                else:
                    assert np.array_equal(got, without[mode]), (at, d, mode)


def check_far_state(dev, lib, dtype=F32):
    """What the recurrence remembers: with gates nearly shut the first token still shows 150 tokens later, through portions and single
    tokens."""
    cfg = MECHANISMS["mingru"]
    sd = random_token_lm_state_dict(cfg, seed=3)
    sd["l0.mix.z.b"] = torch.full((40,), -6.0).to(BF16)
    lm, orc = TokenLM(sd, cfg, device=dev, dtype=dtype, lib=lib, max_slots=2, max_tokens=512), TokenLMOracle(sd, cfg)
    a = tokens_of(cfg, 160, seed=8)
    b = [(a[0] + 1) % cfg.vocab] + a[1:]
    wa, wb = orc.logits(a), orc.logits(b)
    effect = np.abs(wa[-1] - wb[-1]).max()
    assert effect > 1e-5
    for cuts in ([160], [31, 2, 97, 1], [1]):
        diff = run_cut(lm, a, cuts)[-1].astype(np.float64) - run_cut(lm, b, cuts)[-1]
        assert np.abs(diff - (wa[-1] - wb[-1])).max() < 0.05 * effect, cuts


def check_first_tokens(dev, lib, dtype=F32, name="mixed"):
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype)
    for seed in range(3):
        toks = tokens_of(cfg, 5, seed=70 + seed)
        want = orc.logits(toks)
        for cuts in ([5], [1], [2, 3]):
            assert rel(run_cut(lm, toks, cuts), want) < TOL[dtype]


def _attention_pair(orc, cfg):
    """(query token, key token, plain token) of grouped attention over bare token embeddings: the pair whose score stands out most in some
    head, and the token that head cares least for."""
    w, m, p = orc.w, cfg.layers[0].mixer, "l0.mix."
    h = rms_norm(w["embed"] * cfg.embed_scale, w["l0.norm1"], cfg.norm_eps)
    q = (h @ w[p + "q"].T).reshape(cfg.vocab, m.heads, m.dim)
    k = np.repeat((h @ w[p + "k"].T).reshape(cfg.vocab, m.kv_heads, m.dim), m.heads // m.kv_heads, axis=1)
    s = np.matmul(q.transpose(1, 0, 2), k.transpose(1, 2, 0)).transpose(1, 2, 0)        # [query, key, head]
    own = s[np.arange(cfg.vocab), np.arange(cfg.vocab)]
    gap = s - np.maximum(np.maximum(s.min(axis=1), own), 0.0)[:, None, :]
    query, key, head = np.unravel_index(np.argmax(gap), gap.shape)
    return int(query), int(key), int(np.argmin(s[query, :, head]))


def check_single_kept_keys(dev, lib, window=70, keep=7, dtype=F32, queries=(200, 128, 191, 97)):
    """One dominating key at chosen places: around the window's edge, page borders, the last kept position and the one after it.  While it is
    visible the logits are the oracle's and differ from a prompt without it; otherwise they are bit-identical to that."""
    cfg = plain_layer(replace(GQA, window=window, keep_first=keep, scale=1.0))
    sd = random_token_lm_state_dict(cfg, seed=5)
    lm, orc = TokenLM(sd, cfg, device=dev, dtype=dtype, lib=lib, max_slots=2, max_tokens=512), TokenLMOracle(sd, cfg)
    query, key, plain = _attention_pair(orc, cfg)
    assert key not in (query, plain)
    for at in queries:                                   # the query's position
        base = [plain] * (at + 1)
        base[at] = query
        modes = (("prompt", [at + 1]), ("decoded", [at, 1]), ("two", [at - 1, 2]))
        without = {mode: run_cut(lm, base, cuts)[at] for mode, cuts in modes}
        ref0 = orc.logits(base)[at]
        places = {0, 1, keep - 1, keep, keep + 1, 31, 32, 63, 64, at - 1, at - 2, at - window + 1, at - window, at - window - 1, at - at % 64}
        for j in sorted(x for x in places if 0 <= x < at):
            toks = list(base)
            toks[j] = key
            ref = orc.logits(toks)[at]
            shows = window == 0 or at - j < window or j < keep
            assert (rel(ref[None], ref0[None]) > 0.05) == shows, (at, j)
            for mode, cuts in modes:
                got = run_cut(lm, toks, cuts)[at]
                assert rel(got[None], ref[None]) < TOL[dtype], (at, j, mode)
                if shows:
                    assert rel(got[None], without[mode][None]) > 0.05, (at, j, mode)
                else:
                    assert np.array_equal(got, without[mode]), (at, j, mode)


def check_sink(dev, lib):
    """Weak scores: the one in the denominator takes a share that leaving it out would show.  Strong negative ones: nearly all of it."""
    for scale, n in ((0.01, 3), (0.01, 90), (-3.0, 40), (3.0, 40)):
        cfg = plain_layer(replace(GQA, scale=scale))
        sd = random_token_lm_state_dict(cfg, seed=7)
        lm, orc = TokenLM(sd, cfg, device=dev, dtype=F32, lib=lib, max_slots=2, max_tokens=256), TokenLMOracle(sd, cfg)
        without = TokenLMOracle(sd, plain_layer(replace(GQA, scale=scale, sink=False)))
        toks = tokens_of(cfg, n)
        want = orc.logits(toks)
        assert rel(without.logits(toks)[:3], want[:3]) > 0.02
        for cuts in ([n], [1], [n - 2, 2]):
            assert rel(run_cut(lm, toks, cuts), want) < TOL[F32], (scale, n, cuts)


def check_matrix_state_far(dev, lib, dtype=F32):
    """What the matrix states remember: with decays of nearly one the first token still shows 200 tokens later, however it was fed."""
    for name in ("delta", "lightning"):
        cfg = plain_layer(DELTA if name == "delta" else replace(LIGHT, decay=[0.9995, 0.999, 0.9999]))
        sd = random_token_lm_state_dict(cfg, seed=3)
        if name == "delta":
            sd["l0.mix.A_log"] = torch.full((DELTA.heads,), -7.0).to(BF16)
        lm, orc = TokenLM(sd, cfg, device=dev, dtype=dtype, lib=lib, max_slots=2, max_tokens=512), TokenLMOracle(sd, cfg)
        a = tokens_of(cfg, 200, seed=8)
        b = [(a[0] + 1) % cfg.vocab] + a[1:]
        wa, wb = orc.logits(a), orc.logits(b)
        effect = np.abs(wa[-1] - wb[-1]).max()
        assert effect > 1e-3, (name, effect)
        for cuts in ([200], [31, 2, 97, 1], [4]):
            diff = run_cut(lm, a, cuts)[-1].astype(np.float64) - run_cut(lm, b, cuts)[-1]
            assert np.abs(diff - (wa[-1] - wb[-1])).max() < 0.05 * effect, (name, cuts)


def check_decay_extremes(dev, lib):
    """Channels that forget everything at one token and nothing at the next, in one chunk: the running products lose no precision.  Keys that
    repeat with step sizes near one: the triangular system at its stiffest."""
    cfg = plain_layer(replace(DELTA, heads=2, kv_heads=2, dim=32, vdim=16))
    for amp, alog in ((40.0, 3.0), (8.0, 0.0)):
        sd = random_token_lm_state_dict(cfg, seed=4)
        sd["l0.mix.A_log"] = torch.full((2,), alog).to(BF16)
        sd["l0.mix.a2"] = (sd["l0.mix.a2"].float() * amp).to(BF16)
        sd["l0.mix.b"] = (sd["l0.mix.b"].float() * 5).to(BF16)
        lm, orc = TokenLM(sd, cfg, device=dev, dtype=F32, lib=lib, max_slots=2, max_tokens=512), TokenLMOracle(sd, cfg)
        toks = tokens_of(cfg, 60, seed=9) + [5] * 50 + [5, 9] * 20
        want = orc.logits(toks)
        for cuts in ([150], [1], [70, 3, 77]):
            assert rel(run_cut(lm, toks, cuts), want) < TOL[F32], (amp, cuts)


def check_glu_limits(dev, lib):
    """Gate above its limit (and far below zero: unlimited), up beyond both of its limits."""
    cfg = MECHANISMS["glu"]
    sd = random_token_lm_state_dict(cfg, seed=6)
    for n in ("gate", "up"):
        sd[f"l0.mlp.{n}"] = (sd[f"l0.mlp.{n}"].float() * 4).to(BF16)
    lm, orc = TokenLM(sd, cfg, device=dev, dtype=F32, lib=lib, max_slots=2, max_tokens=256), TokenLMOracle(sd, cfg)
    toks = tokens_of(cfg, 80)
    want = orc.logits(toks)
    for cuts in ([80], [30, 1]):
        assert rel(run_cut(lm, toks, cuts), want) < TOL[F32]


def check_previous_token(dev, lib):
    """The bigram row needs the token before a portion: cut everywhere, with another sequence in between, on a slot used before."""
    cfg = MECHANISMS["bigram"]
    sd = random_token_lm_state_dict(cfg, seed=2)
    sd["bigram"] = (sd["bigram"].float() * 6).to(BF16)
    lm, orc = TokenLM(sd, cfg, device=dev, dtype=F32, lib=lib, max_slots=2, max_tokens=256), TokenLMOracle(sd, cfg)
    for seed in range(2):
        a, b = tokens_of(cfg, 20, seed=seed), tokens_of(cfg, 20, seed=seed + 40)
        wa, wb = orc.logits(a), orc.logits(b)
        sa, sb = lm.open(), lm.open()
        got, at = [], 0
        for n in (1, 1, 5, 2, 1, 10):
            if at % 2:
                rows = lm.step([(sb, b[at:at + n], list(range(n))), (sa, a[at:at + n], list(range(n)))]).cpu().numpy()
                assert rel(rows[:n], wb[at:at + n]) < TOL[F32]
                rows = rows[n:]
            else:
                rows = lm.step([(sa, a[at:at + n], list(range(n)))]).cpu().numpy()
                assert rel(lm.step([(sb, b[at:at + n], list(range(n)))]).cpu().numpy(), wb[at:at + n]) < TOL[F32]
            got.append(rows.copy())
            at += n
        assert rel(np.concatenate(got), wa) < TOL[F32]
        lm.close(sa)
        lm.close(sb)


def check_last_position(dev, lib):
    import pytest
    cfg = plain_layer(LIGHT, None, max_positions=70)
    lm, orc = make(cfg, dev, lib, max_slots=2, max_tokens=256)
    toks = tokens_of(cfg, 70)
    slot = lm.open()
    assert rel(run_cut(lm, toks, [69, 1], slot), orc.logits(toks)) < TOL[F32]
    with pytest.raises(AssertionError):
        lm.step([(slot, [1], [0])])
    assert lm.position(slot) == 70
    lm.close(slot)
    with pytest.raises(ValueError):
        TokenBatcher(lm).submit(toks, 2)
    assert TokenBatcher(lm).submit(toks, 1)


# ---- entry points --------------------------------------------------------------------------------------------------------------
def check_generation(dev, lib, dtype=F32, name="mixed"):
    """Greedy generation through the scheduler: more requests than slots, prompts cut by the step budget, a pool they must share;
    each request as the oracle generates it alone."""
    cfg = MECHANISMS[name]
    lm, orc = make(cfg, dev, lib, dtype, max_slots=3, max_tokens=320)
    prompts = [tokens_of(cfg, n, seed=80 + i) for i, n in enumerate((50, 3, 120, 1, 66))]
    batcher = TokenBatcher(lm, step_tokens=48)
    got = batcher.generate(prompts, max_new_tokens=9)
    for p, g in zip(prompts, got):
        assert g == orc.greedy(p, 9)
    assert batcher.stats() == {"waiting": 0, "live": 0, "free_pages": lm.total_pages, "free_slots": 3, "reserved_pages": 0}
    stop = got[0][4]
    want = got[0][:got[0].index(stop) + 1]
    assert batcher.generate([prompts[0]], 9, stop=[stop])[0] == want


def check_sampling(dev, lib):
    """top_k = 1 is greedy whatever the temperature; a seed reproduces its stream; only tokens of the top-k set are drawn, and all of a
    flat pair are."""
    cfg = MECHANISMS["mingru"]
    lm, _ = make(cfg, dev, lib)
    prompts = [tokens_of(cfg, 12, seed=90 + i) for i in range(3)]
    greedy = TokenBatcher(lm).generate(prompts, 6)
    slots = [lm.open() for _ in prompts]
    logits = lm.step([(s, p, [len(p) - 1]) for s, p in zip(slots, prompts)])
    assert lm.sample(logits, slots).tolist() == [g[0] for g in greedy]
    assert lm.sample(logits.to(BF16).float(), slots, temp=0.9, top_k=1).tolist() == lm.sample(logits.to(BF16).float(), slots).tolist()
    flat = torch.full((3, cfg.vocab), -30.0, device=logits.device)
    flat[:, 5] = flat[:, 66] = 2.0
    drawn = {t for seed in range(24) for t in lm.sample(flat, slots, temp=1.0, top_k=10, seed=seed).tolist()}
    assert drawn == {5, 66}
    mixed = lm.sample(flat, slots, temp=[0.0, 1.0, 0.0], top_k=[0, 2, 0]).tolist()
    assert mixed[0] == 5 and mixed[2] == 5 and mixed[1] in (5, 66)
    for s in slots:
        lm.close(s)
    a = TokenBatcher(make(cfg, dev, lib)[0], seed=11).generate(prompts, 8, temp=1.0)
    b = TokenBatcher(make(cfg, dev, lib)[0], seed=11).generate(prompts, 8, temp=1.0)
    assert a == b and all(0 <= t < cfg.vocab for r in a for t in r)


def check_limits(dev, lib):
    import pytest
    from moshi_amd.errors import UnknownChannel
    cfg = MECHANISMS["attention"]
    lm, orc = make(cfg, dev, lib, max_slots=2, max_tokens=128, max_step_tokens=100)
    a, b = lm.open(), lm.open()
    with pytest.raises(BufferError):
        lm.open()
    toks = tokens_of(cfg, 90)
    lm.step([(a, toks[:60], []), (b, toks[:10], [])])
    with pytest.raises(BufferError):                      # both want a second page, none is free: nothing happens
        lm.step([(a, toks[60:], [29])])
    assert lm.position(a) == 60 and lm.free_pages == 0
    lm.close(b)
    got = lm.step([(a, toks[60:], [29])]).cpu().numpy()
    assert rel(got, orc.logits(toks)[89:]) < TOL[F32]
    with pytest.raises(UnknownChannel):
        lm.step([(b, [1], [])])
    with pytest.raises(UnknownChannel):
        lm.close(b)
    with pytest.raises(ValueError):
        lm.step([(a, [cfg.vocab], [])])
    with pytest.raises(ValueError):
        lm.step([(a, [1], []), (a, [2], [])])
    with pytest.raises(AssertionError):
        lm.step([(a, toks + toks, [])])
    with pytest.raises(KeyError):
        sd = random_token_lm_state_dict(cfg)
        del sd["l0.mix.uk"]
        TokenLM(sd, cfg, device=dev, lib=lib)
    with pytest.raises(AssertionError):
        sd = random_token_lm_state_dict(cfg)
        sd["l0.mix.uk"] = sd["l0.mix.uk"][:-1]
        TokenLM(sd, cfg, device=dev, lib=lib)
    with pytest.raises(BufferError):
        TokenBatcher(lm).submit(toks, 60)
    # wanted rows in any order, and a step that wants nothing
    lm.close(a)
    a = lm.open()
    rows = lm.step([(a, toks[:20], [7, 3, 3])]).cpu().numpy()
    want = orc.logits(toks[:20])
    assert rel(rows, want[[7, 3, 3]]) < TOL[F32]


def check_replay(dev, lib, tmp_path):
    """bin/trace_run's loop: names instead of slots, admission at the first entry, slots given back, files per step."""
    import json
    from moshi_amd.trace_run import replay
    cfg = MECHANISMS["mixed"]
    lm, orc = make(cfg, dev, lib, max_slots=2, max_tokens=256)
    seqs = {n: tokens_of(cfg, k, seed=i) for i, (n, k) in enumerate({"a": 70, "b": 30, "c": 41}.items())}
    plan = [[("a", 0, 50)], [("b", 0, 30), ("a", 50, 51)], [("a", 51, 70)], [("c", 0, 41)]]
    lines, done = [], []
    for i, step in enumerate(plan):
        entries = [{"id": n, "tokens": seqs[n][x:y], "want": [0, y - x - 1] if y - x > 1 else [0]} for n, x, y in step]
        if i == 0:
            entries[0]["want"] = []
        lines.append(json.dumps({"step": i, "entries": entries, "end": [n for n, _, y in step if y == len(seqs[n])]}))
    replay(lm, lines, tmp_path, done.append)
    assert done == [f"done {i}" for i in range(4)] and not (tmp_path / "0.f32").exists()
    read = lambda i: np.fromfile(tmp_path / f"{i}.f32", dtype="<f4").reshape(-1, cfg.vocab)
    wa, wb, wc = (orc.logits(seqs[n]) for n in "abc")
    assert rel(read(1), np.stack([wb[0], wb[29], wa[50]])) < TOL[F32]
    assert rel(read(2), wa[[51, 69]]) < TOL[F32] and rel(read(3), wc[[0, 40]]) < TOL[F32]
    assert lm.free_slots == 2 and lm.free_pages == lm.total_pages
