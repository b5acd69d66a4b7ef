"""Host side of the token language models: binding against the header, configuration, registry, loading, command line, scheduler."""
import ctypes
import json
import re
import subprocess

import numpy as np
import pytest
import torch

from moshi_amd import _capi, loaders
from moshi_amd.config import (BigramConfig, ChannelDeltaConfig, DenseGLUConfig, GroupedAttentionConfig, LatentAttentionConfig, LightningConfig, MinGRUConfig,
                              MoEConfig, TokenLayerConfig, tiny_bibapel_config, tiny_token_lm_config)
from moshi_amd.token_batcher import TokenBatcher
from moshi_amd.weights import random_token_lm_state_dict, token_lm_state_spec
from oracle.token_lm_oracle import TokenLMOracle
from tests import tlm_cases as tc
from tests.conftest import ROOT
from tests.test_tlm_sim import tlm_lib  # noqa: F401  (fixture)

RAW = {
    "architecture": "Kesirax", "vocab": 53, "width": 60, "logit_scale": 0.25, "norm": {"eps": 1e-5, "groups": 5},
    "layers": [
        {"type": "latent_attention",
         "mixer": {"heads": 2, "dim": 18, "vdim": 14, "rot_dim": 10, "q_rank": 22, "kv_rank": 26, "scale": 0.2, "mask": {"size": 19}, "rot": {"base": 777.0, "dims": 10}},
         "mlp": None},
        {"type": "mingru", "mixer": {"width": 34},
         "mlp": {"kind": "moe", "router": {"experts": 3, "top": 2}, "expert": {"ff": 21}}}]}

BIBAPEL = {
    "architecture": "Bibapel", "vocab": 59, "width": 44, "norm": {"eps": 1e-4}, "max_positions": 90,
    "embedding": {"scale": 0.7, "bigram": {"buckets": 23, "mul_prev": 13, "mul_cur": 4}}, "loop": {"start": 1, "stop": 3, "times": 2},
    "layers": [
        {"type": "lightning", "mixer": {"heads": 2, "dim": 12, "vdim": 20, "decay": [0.5, 0.99]}, "mlp": None},
        {"type": "channel_delta", "mixer": {"heads": 4, "kv_heads": 2, "dim": 14, "vdim": 18, "conv": 3}, "mlp": {"kind": "dense", "ff": 30, "limit": 1.5}},
        {"type": "attention", "mixer": {"heads": 3, "kv_heads": 1, "dim": 22, "vdim": 10, "scale": 0.3, "mask": {"size": 17, "keep_first": 2}},
         "mlp": {"kind": "dense", "ff": 26, "limit": 0.8}}]}


def _header():
    return re.sub(r"/\*.*?\*/", "", (ROOT / "include" / "moshi_tlm.h").read_text(), flags=re.S)


def test_binding_covers_the_header_and_the_library_exports_it():
    declared = set(re.findall(r"\b(mmi_tlm_[a-z0-9_]+)\s*\(", _header()))
    assert declared == {n for n in _capi.TLM_SIGNATURES if n.startswith("mmi_tlm_")}
    from moshi_amd import build
    build.build(verbose=False, which="tlm")
    lib = _capi.load_tlm()
    assert all(hasattr(lib.cdll, n) for n in declared) and lib.mmi_version() == 3


def test_header_compiles_alone_and_structs_equal_the_binding(tmp_path):
    structs = {"mmi_tlm_layer": _capi.TLMLayer, "mmi_tlm_cfg": _capi.TLMCfg}
    consts = sorted(set(re.findall(r"#define (MMI_TLM_\w+)", _header())))
    lines = ['#include "moshi_tlm.h"', "#include <stdio.h>", "#include <stddef.h>", "int main(void) {"]
    for s, cls in structs.items():
        lines.append(f'  printf("{s} . %zu\\n", sizeof({s}));')
        lines += [f'  printf("{s} {f} %zu\\n", offsetof({s}, {f}));' for f, _ in cls._fields_]
    lines += [f'  printf("const {c} %d\\n", {c});' for c in consts] + ["  return 0;", "}"]
    (tmp_path / "t.c").write_text("\n".join(lines) + "\n")
    subprocess.check_call(["gcc", "-std=c99", "-Wall", "-Werror", f"-I{ROOT / 'include'}", str(tmp_path / "t.c"), "-o", str(tmp_path / "t")])
    for line in subprocess.run([str(tmp_path / "t")], capture_output=True, text=True, check=True).stdout.splitlines():
        s, f, v = line.split()
        if s == "const":
            assert getattr(_capi, f[len("MMI_"):]) == int(v), f
        else:
            assert int(v) == (ctypes.sizeof(structs[s]) if f == "." else getattr(structs[s], f).offset), (s, f)


def test_missing_library_and_cpu_device_fail_loudly(monkeypatch, tmp_path):
    monkeypatch.setattr(_capi, "TLM_LIB", tmp_path / "nope.so")
    monkeypatch.setattr(_capi, "_default_tlm", None)
    with pytest.raises(RuntimeError, match="no CPU/PyTorch fallback"):
        _capi.load_tlm()
    from moshi_amd import TokenLM
    with pytest.raises(RuntimeError, match="no CPU path"):
        TokenLM({}, tiny_token_lm_config(), device="cpu")


def test_configuration_is_read_not_assumed():
    cfg = loaders.token_lm_config_from_dict(RAW)
    assert cfg.layers == [TokenLayerConfig(LatentAttentionConfig(heads=2, dim=18, vdim=14, rot_dim=10, q_rank=22, kv_rank=26, scale=0.2, rot_base=777.0, window=19), None),
                          TokenLayerConfig(MinGRUConfig(34), MoEConfig(experts=3, top=2, ff=21))]
    assert (cfg.vocab, cfg.width, cfg.norm_groups, cfg.norm_eps, cfg.logit_scale) == (53, 60, 5, 1e-5, 0.25)
    assert cfg.layer_runs == [0, 1]
    looped = loaders.token_lm_config_from_dict({**RAW, "loop": {"start": 1, "stop": 2, "times": 4}})
    assert looped.layer_runs == [0, 1, 1, 1, 1]
    for bad in ({**RAW, "architecture": "Other"}, {**RAW, "layers": [{"type": "conv", "mixer": {}, "mlp": None}]},
                {**RAW, "layers": [{**RAW["layers"][1], "mlp": {**RAW["layers"][1]["mlp"], "kind": "glu"}}]},
                {**RAW, "layers": [{**RAW["layers"][0], "mixer": {**RAW["layers"][0]["mixer"], "rot": {"base": 10.0, "dims": 4}}}]}):
        with pytest.raises(ValueError):
            loaders.token_lm_config_from_dict(bad)


def test_bibapel_configuration_is_read_not_assumed():
    cfg = loaders.token_lm_config_from_dict(BIBAPEL, {"l1.mix.a1": (9, 44), "l1.mix.g1": (11, 44)})
    assert cfg.layers == [
        TokenLayerConfig(LightningConfig(heads=2, dim=12, vdim=20, decay=[0.5, 0.99]), None),
        TokenLayerConfig(ChannelDeltaConfig(heads=4, kv_heads=2, dim=14, vdim=18, conv=3, decay_rank=9, gate_rank=11), DenseGLUConfig(ff=30, limit=1.5)),
        TokenLayerConfig(GroupedAttentionConfig(heads=3, kv_heads=1, dim=22, vdim=10, scale=0.3, window=17, keep_first=2, sink=True), DenseGLUConfig(ff=26, limit=0.8))]
    assert (cfg.vocab, cfg.width, cfg.norm_eps, cfg.max_positions, cfg.embed_scale, cfg.bigram) == (59, 44, 1e-4, 90, 0.7, BigramConfig(23, 13, 4))
    assert cfg.layer_runs == [0, 1, 2, 1, 2] and cfg.tied_head and cfg.norms == 2 and not cfg.layer_scales and cfg.loop_inject == "project"
    bare = loaders.token_lm_config_from_dict({**BIBAPEL, "embedding": {}, "loop": None, "max_positions": 0,
                                              "layers": [{**BIBAPEL["layers"][2], "mixer": {**BIBAPEL["layers"][2]["mixer"], "mask": None}}]})
    assert bare.bigram is None and bare.embed_scale == 1.0 and bare.layer_runs == [0] and bare.layers[0].mixer.window == 0
    for bad in ({**BIBAPEL, "embedding": {"scale": 1.0, "trigram": {}}}, {**BIBAPEL, "layers": [{**BIBAPEL["layers"][1], "type": "mingru"}]},
                {**BIBAPEL, "layers": [{**BIBAPEL["layers"][0], "mixer": {"heads": 3, "dim": 4, "vdim": 4, "decay": [0.5, 0.9]}}]},
                {**BIBAPEL, "layers": [{**BIBAPEL["layers"][1], "mlp": {"kind": "moe", "ff": 3, "limit": 1.0}}]}):
        with pytest.raises(ValueError):
            loaders.token_lm_config_from_dict(bad)


def test_spec_covers_every_tensor_of_every_layer():
    cfg = tiny_token_lm_config()
    spec = {n: s for n, s, _ in token_lm_state_spec(cfg)}
    assert spec["embed"] == (101, 96) and spec["l1.mix.uq"] == (3 * 36, 40) and spec["l1.mlp.table"] == (101, 2)
    assert "l2.ls2" not in spec and "l2.mlp.table" not in spec and "l2.ls1" in spec
    cfg2 = tiny_bibapel_config()
    spec2 = {n: s for n, s, _ in token_lm_state_spec(cfg2)}
    assert spec2["bigram"] == (38, 80) and spec2["pos"] == (1500, 80) and spec2["loop.in"] == (80, 160) and spec2["loop.step"] == (2, 80)
    assert spec2["l1.mix.v.conv"] == (96, 3) and spec2["l1.mix.a2"] == (80, 10) and "l3.norm2" not in spec2 and "head" not in spec2 and "l0.ls1" not in spec2
    table = random_token_lm_state_dict(cfg)["l1.mlp.table"]
    assert table.dtype == torch.int32 and all(len(set(row)) == 2 for row in table.tolist())


def _save(tmp_path, raw, seed=4):
    from safetensors.torch import save_file
    sd = random_token_lm_state_dict(loaders.token_lm_config_from_dict(raw), seed=seed)
    save_file(sd, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(raw))
    return sd


def test_registry_loads_a_directory(tlm_lib, tmp_path):  # noqa: F811
    sd = _save(tmp_path, RAW)
    assert loaders.is_token_lm(tmp_path) and loaders.is_token_lm(tmp_path / "config.json")
    with pytest.raises(ValueError, match="get_token_lm"):
        loaders.CheckpointInfo.from_local(tmp_path)
    moshi = tmp_path / "moshi"
    moshi.mkdir()
    (moshi / "config.json").write_text(json.dumps({"dim": 4096}))
    assert not loaders.is_token_lm(moshi)
    lm = loaders.get_token_lm(tmp_path, device="cpu", dtype=torch.float32, max_slots=2, max_tokens=128, lib=tlm_lib)
    toks = tc.tokens_of(lm.config, 40)
    assert tc.rel(tc.run_cut(lm, toks, [33, 1, 6]), TokenLMOracle(sd, lm.config).logits(toks)) < tc.TOL[tc.F32]


def test_registry_takes_sizes_from_the_tensors(tlm_lib, tmp_path):  # noqa: F811
    from safetensors.torch import save_file
    shapes = {"l1.mix.a1": (9, 44), "l1.mix.g1": (11, 44)}
    sd = random_token_lm_state_dict(loaders.token_lm_config_from_dict(BIBAPEL, shapes), seed=4)
    save_file(sd, str(tmp_path / "model.safetensors"))
    (tmp_path / "config.json").write_text(json.dumps(BIBAPEL))
    assert loaders.is_token_lm(tmp_path)
    lm = loaders.get_token_lm(tmp_path, device="cpu", dtype=torch.float32, max_slots=2, max_tokens=128, lib=tlm_lib)
    assert lm.config.layers[1].mixer.decay_rank == 9 and lm.config.layers[1].mixer.gate_rank == 11
    toks = tc.tokens_of(lm.config, 40)
    assert tc.rel(tc.run_cut(lm, toks, [33, 1, 6]), TokenLMOracle(sd, lm.config).logits(toks)) < tc.TOL[tc.F32]


@pytest.mark.parametrize("raw", [RAW, BIBAPEL], ids=["kesirax", "bibapel"])
def test_command_line_generates(tlm_lib, tmp_path, monkeypatch, raw):  # noqa: F811
    from moshi_amd import run_inference
    sd = _save(tmp_path, raw)
    load = loaders.get_token_lm
    monkeypatch.setattr(loaders, "get_token_lm", lambda path, **kw: load(path, **{**kw, "device": "cpu", "lib": tlm_lib}))
    cfg = loaders.token_lm_config_from_dict(raw)
    prompts = [tc.tokens_of(cfg, n, seed=n) for n in (7, 40, 2)]
    (tmp_path / "in.txt").write_text("\n".join(" ".join(map(str, p)) for p in prompts) + "\n")
    run_inference.main(["--checkpoint-dir", str(tmp_path), "--greedy", "--dtype", "float32", "--batch-size", "2", "--step-tokens", "16", "--max-new-tokens", "5",
                        str(tmp_path / "in.txt"), str(tmp_path / "out.txt")])
    got = [[int(t) for t in ln.split()] for ln in (tmp_path / "out.txt").read_text().splitlines()]
    orc = TokenLMOracle(sd, cfg)
    assert got == [orc.greedy(p, 5) for p in prompts]


class _FakeLM:
    """Slots and pages only: what the scheduler asks of a model."""
    vocab, max_step_tokens, page = 50, 64, 64

    def __init__(self, slots, pages):
        self.total_pages, self.slots, self.pos, self.steps = pages, slots, {}, []
        self.next = 0

    free_slots = property(lambda self: self.slots - len(self.pos))
    free_pages = property(lambda self: self.total_pages - sum(-(-p // self.page) for p in self.pos.values()))

    def pages_needed(self, slot, n):
        return -(-n // self.page)

    def open(self):
        self.next += 1
        self.pos[self.next] = 0
        return self.next

    def close(self, slot):
        del self.pos[slot]

    def step(self, entries):
        assert sum(len(t) for _, t, _ in entries) <= self.max_step_tokens
        for s, t, _ in entries:
            self.pos[s] += len(t)
        assert self.free_pages >= 0
        self.steps.append([(s, len(t), len(w)) for s, t, w in entries])
        return np.zeros((sum(len(w) for _, _, w in entries), self.vocab))

    def sample(self, logits, slots, temp, top_k, seed=0):
        assert len(logits) == len(slots)
        return torch.full((len(slots),), 7, dtype=torch.int32)


def test_scheduler_mixes_decoding_with_prompt_portions_within_its_budget():
    lm = _FakeLM(slots=4, pages=10)
    b = TokenBatcher(lm, step_tokens=20)
    first = b.submit([1] * 5, 6)
    b.step()
    second = b.submit([2] * 50, 3)
    while b.step():
        pass
    assert b.pop(first) == [7] * 6 and b.pop(second) == [7] * 3
    assert lm.steps[1] == [(1, 1, 1), (2, 19, 0)] and lm.steps[3][1] == (2, 12, 1)      # 19 + 19 + 12 beside single tokens
    assert lm.free_slots == 4 and lm.free_pages == 10


def test_scheduler_admits_only_what_the_pool_can_finish():
    lm = _FakeLM(slots=8, pages=4)
    b = TokenBatcher(lm)
    ids = [b.submit([3] * 60, 40) for _ in range(4)]             # two pages each: two at a time
    b.step()
    assert b.stats()["live"] == 2 and b.stats()["waiting"] == 2
    b.cancel(ids[3])
    while b.step():
        pass
    assert all(len(b.pop(i)) == 40 for i in ids[:3]) and b.stats()["reserved_pages"] == 0
    from moshi_amd.errors import UnknownChannel
    with pytest.raises(UnknownChannel):
        b.pop(ids[3])
    with pytest.raises(ValueError):
        b.submit([], 3)
    with pytest.raises(BufferError):
        b.submit([1] * 300, 3)
