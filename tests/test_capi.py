"""The C-ABI library loads and exports exactly what include/skyrl_hip.h declares (no GPU needed)."""

import ctypes
import os
import re

import pytest

from skyrl_amd import _ffi

ROOT = os.path.dirname(os.path.dirname(os.path.abspath(__file__)))


def header_functions(name="skyrl_hip.h"):
    src = open(os.path.join(ROOT, "include", name)).read()
    src = re.sub(r"/\*.*?\*/", "", src, flags=re.S)
    return sorted(set(re.findall(r"^\s*(?:const\s+)?\w+\*?\s+\*?(skyrl_\w+)\s*\(", src, flags=re.M)))


def test_header_parsed():
    names = header_functions()
    assert "skyrl_grpo_advantage" in names and "skyrl_logprob_fwd" in names and len(names) >= 18


def test_library_exports_every_declared_symbol():
    lib = _ffi.load()
    missing = [n for n in header_functions() if not hasattr(lib, n)]
    assert not missing, f"declared in skyrl_hip.h but not exported: {missing}"


def test_ffi_signatures_cover_header():
    assert sorted(_ffi.SIGNATURES) == header_functions()


def test_layers_library_matches_its_header():
    """The layer libraries export what include/skyrl_layers.h declares, and are bound name by name."""
    names = header_functions("skyrl_layers.h")
    assert "skyrl_latent_attend" in names and "skyrl_delta_scan" in names and sorted(_ffi.LAYERS_SIGNATURES) == names
    assert not [n for n in names if not hasattr(_ffi.load_layers(_ffi.layer_lib_of(n)), n)]
    assert {_ffi.layer_lib_of(n) for n in names} == set(_ffi.LAYER_LIBS)
    assert not set(names) & set(header_functions())


def test_recurrent_layers_entries_validate_on_host():
    p = ctypes.c_void_p(16)
    q = ctypes.c_void_p(20)  # not aligned to 16 bytes
    attn = lambda *a: ctypes.byref(_ffi.AttnShape(*a, 0.5, 1e-5))  # noqa: E731
    ssd = lambda *a: ctypes.byref(_ffi.SSDShape(*a))  # noqa: E731
    sec = (_ffi.ConvSection * 4)(_ffi.ConvSection(2, 8, 8, 16, None), _ffi.ConvSection(1, 4, 2, 16, None))
    seqs = (p, 1, p, p, p)
    for name, args, msg in (
            ("skyrl_norm_add", (p, None, None, None, 0.5, p, p, 1, None, 0, 1, 9000, 1e-5, p, _ffi.BF16, None), "H must be"),
            ("skyrl_norm_add", (p, None, None, None, 0.5, p, p, 7, None, 0, 1, 64, 1e-5, p, _ffi.BF16, None), "1 or H"),
            ("skyrl_norm_add", (p, None, p, None, 0.5, p, p, 1, None, 0, 1, 64, 1e-5, p, _ffi.BF16, None), "null"),
            ("skyrl_xielu", (p, 7, 1, 8, p, p, 8, _ffi.F32, None), "bad sizes"),
            ("skyrl_gated_norm", (p, 8, p, 8, p, 1, 8, 3, 1e-5, p, 8, _ffi.F32, None), "bad sizes"),
            ("skyrl_embed", (p, p, 1, 8, 1.0, None, p, p, None, _ffi.F32, None), "null"),
            ("skyrl_conv_chunk", (p, 32, 20, 4, p, None, 0, *seqs, p, sec, 2, _ffi.BF16, None), "bad section"),
            ("skyrl_conv_chunk", (p, 32, 20, 4, p, None, 0, *seqs, p, sec, 1, _ffi.BF16, None), "cover"),
            ("skyrl_conv_chunk", (p, 32, 20, 4, p, None, 0, *seqs, p, sec, 4, _ffi.BF16, None), "sections"),
            ("skyrl_conv_chunk", (p, 32, 16, 4, q, None, 0, *seqs, p, sec, 1, _ffi.BF16, None), "alignment"),
            ("skyrl_rglru_step", (p, 20, 10, 3, 4, p, p, p, p, p, p, p, 1, p, p, p, 10, _ffi.BF16, None), "multiple of blocks"),
            ("skyrl_rglru_step", (p, 10, 10, 2, 4, p, p, p, p, p, p, p, 1, p, p, p, 10, _ffi.BF16, None), "bad sizes"),
            ("skyrl_rglru_step", (p, 8192, 4096, 1, 4, p, p, p, p, p, p, p, 1, p, p, p, 4096, _ffi.BF16, None), "too large"),
            ("skyrl_rglru_prompt", (p, 20, 10, 2, p, p, p, p, p, 1, p, 2, p, 0, 1, p, p, p, p, p, p, p, p, 10, _ffi.F32, None),
             "bad sizes"),
            ("skyrl_attn_write", (attn(3, 2, 8, 8, 0), p, 99, p, p, p, None, 0, 1, p, p, p, _ffi.BF16, None), "multiple of kv_heads"),
            ("skyrl_attn_write", (attn(2, 1, 9, 8, 0), p, 99, p, p, p, p, 0, 1, p, p, p, _ffi.BF16, None), "runs need"),
            ("skyrl_attn_attend", (attn(2, 1, 8, 8, 4), p, p, 16, p, p, p, 1, p, p, 1, 64, 3, p, 16, None, _ffi.BF16, None), "workspace"),
            ("skyrl_attn_attend", (attn(2, 1, 8, 8, 4), p, p, 15, p, p, p, 1, p, p, 1, 64, 1, p, 16, None, _ffi.BF16, None), "bad sizes"),
            ("skyrl_attn_prefill", (attn(2, 1, 300, 8, 4), p, p, 16, p, p, p, 1, p, 1, p, 16, None), "dim, vdim"),
            ("skyrl_ssd_scan", (ssd(3, 8, 8, 2, 4), p, 99, p, p, p, p, p, p, p, p, 1, p, p, 0, p, 24, _ffi.BF16, None), "multiple of groups"),
            ("skyrl_ssd_scan", (ssd(2, 1024, 1024, 1, 4), p, 9999, p, p, p, p, p, p, p, p, 1, p, p, 0, p, 2048, _ffi.BF16, None), "too large"),
            ("skyrl_ssd_prompt", (ssd(2, 8, 300, 1, 4), p, p, p, p, p, 2, p, p, p, p, 1, p, 1, p, 0, p, 0, p, p, p, p, p, p, p, p,
                                  16, None), "at most 256")):
        with pytest.raises(_ffi.SkyrlHipError, match=msg):
            _ffi.call(name, *args)


def test_layers_entries_validate_on_host():
    p, sh = ctypes.c_void_p(16), _ffi.DeltaShape(3, 2, 8, 8, 4, 1e-5)
    diff = lambda *a: ctypes.byref(_ffi.DiffShape(*a, 0.5, 0.3, 1e-5))  # noqa: E731
    good = diff(4, 2, 12, 8, 4, 3, 1)
    rows = (p, p, p, p, p, p)
    for name, args, msg in (
            ("skyrl_add_norm", (None, p, None, p, 0.0, 1, 9000, 1e-5, 0, p, _ffi.BF16, None), "H must be"),
            ("skyrl_add_norm", (None, p, None, p, 0.0, 1, 64, 1e-5, 0, p, _ffi.I64, None), "dtype"),
            ("skyrl_gate_mul", (p, 16, 1, 8, 7, 1.0, 0.0, p, 8, _ffi.F32, None), "activation"),
            ("skyrl_gate_mul", (p, 15, 1, 8, 2, 1.0, 0.0, p, 8, _ffi.F32, None), "sizes"),
            ("skyrl_embed", (p, p, 1, 0, 1.0, None, None, p, None, _ffi.F32, None), "sizes"),
            ("skyrl_conv_save", (p, 7, 8, 3, p, p, p, 1, p, _ffi.F32, None), "sizes"),
            ("skyrl_latent_write", (p, 10, 1, 1, 4, 4, 0, 0, None, 8, 8, p, 1e-5, p, p, p, p, 32, _ffi.F32, None), "proj_stride"),
            ("skyrl_latent_write", (p, 100, 1, 1, 4, 4, 0, 0, None, 40, 8, p, 1e-5, p, p, p, p, 40, _ffi.F32, None), "multiple of 32"),
            ("skyrl_latent_write", (p, 100, 1, 1, 4, 4, 1, 8, p, 8, 8, p, 1e-5, p, p, p, p, 32, _ffi.F32, None), "not both"),
            ("skyrl_latent_write", (p, 100, 1, 0, 0, 4, 1, 8, None, 8, 8, p, 1e-5, p, p, p, p, 32, _ffi.F32, None), "null"),
            ("skyrl_latent_attend", (p, p, 8, 8, p, 64, p, 4, p, p, 1, 1, 32, 16, 1.0, 0, 8, 1, None, None, 0, p, p, _ffi.BF16, None),
             "part_min"),
            ("skyrl_latent_attend", (p, p, 8, 8, p, 64, p, 4, p, p, 1, 1, 32, 16, 1.0, 0, 64, 2, None, None, 0, p, None, _ffi.BF16, None),
             "workspace"),
            ("skyrl_latent_attend", (p, p, 8, 8, p, 64, p, 4, p, p, 1, 2, 32, 16, 1.0, 0, 64, 1, None, p, 1, p, None, _ffi.BF16, None),
             "gate_stride"),
            ("skyrl_latent_prefill", (p, 8, p, 8, p, p, 65, p, 1, 1, 16, 16, 16, 1.0, 0, None, None, 0, p, 16, None), "vt_stride"),
            ("skyrl_latent_prefill", (p, 8, p, 8, p, p, 64, p, 1, 1, 250, 16, 16, 1.0, 0, None, None, 0, p, 16, None), "256"),
            ("skyrl_delta_scan", (ctypes.byref(sh), p, 100, p, p, p, p, p, p, p, 1, p, p, 1, p, 24, _ffi.F32, None),
             "multiple of kv_heads"),
            ("skyrl_diff_write", (diff(3, 2, 8, 8, 4, 3, 1), p, 100, p, *rows, p, 0, 0, 1, p, p, p, _ffi.F32, None),
             "multiple of kv_heads"),
            ("skyrl_diff_write", (diff(4, 2, 8, 8, 10, 3, 1), p, 100, p, *rows, p, 0, 0, 1, p, p, p, _ffi.F32, None),
             "rot_dims"),
            ("skyrl_diff_write", (good, p, 100, p, *rows, p, 0, 0, 1, p, p, p, _ffi.F32, None), "sizes"),
            ("skyrl_diff_write_runs", (good, p, 160, p, *rows, p, p, 1, p, p, p, None), "multiples of 8"),
            ("skyrl_diff_attend", (good, p, p, 4, p, p, p, 8, p, p, 1, p, 8, 1, p, 32, p, _ffi.BF16, None), "part_min"),
            ("skyrl_diff_attend", (good, p, p, 4, p, p, p, 8, p, p, 1, p, 64, 2, p, 32, None, _ffi.BF16, None),
             "workspace"),
            ("skyrl_diff_attend", (good, p, p, 4, p, p, p, 8, p, p, 1, p, 64, 1, p, 31, None, _ffi.F32, None), "sizes"),
            ("skyrl_diff_prefill", (diff(4, 2, 130, 8, 4, 3, 1), p, p, 4, p, p, p, 8, p, 1, p, p, 32, None), "dim <= 128"),
            ("skyrl_diff_prefill", (good, p, p, 3, p, p, p, 8, p, 1, p, p, 32, None), "sizes")):
        with pytest.raises(_ffi.SkyrlHipError, match=msg):
            _ffi.call(name, *args)


def test_routed_entries_validate_on_host():
    p = ctypes.c_void_p(16)
    gd = lambda *a: ctypes.byref(_ffi.GeneralDeltaShape(*a, 1e-5))  # noqa: E731
    moe = lambda *a: ctypes.byref(_ffi.MoeShape(*a))  # noqa: E731
    ok = moe(64, 32, 8, 2, 2, 1)
    for name, args, msg in (
            ("skyrl_gate_norm_add", (p, None, 1, None, 0, None, p, 1, 1e-5, 1.0, p, 0, p, 1, 9000, p, _ffi.BF16, None), "H must be"),
            ("skyrl_gate_norm_add", (p, None, 1, None, 0, None, p, 3, 1e-5, 1.0, p, 0, p, 1, 64, p, _ffi.BF16, None), "multiple of groups"),
            ("skyrl_gate_norm_add", (p, None, 1, p, 64, None, p, 4, 1e-5, 1.0, p, 0, p, 1, 64, p, _ffi.BF16, None), "bias"),
            ("skyrl_tanh", (p, 7, 1, 8, p, _ffi.F32, None), "sizes"),
            ("skyrl_gdelta_scan", (gd(2, 300), p, 9999, p, 9999, p, p, p, p, p, p, 1, p, p, 9999, _ffi.BF16, None), "256"),
            ("skyrl_gdelta_scan", (gd(2, 8), p, 79, p, 16, p, p, p, p, p, p, 1, p, p, 16, _ffi.BF16, None), "strides"),
            ("skyrl_gdelta_chunk", (gd(2, 8), p, 80, p, 15, p, p, p, 1, p, p, p, p, _ffi.F32, None), "strides"),
            ("skyrl_gdelta_chain", (gd(2, 8), p, p, -1, 1, p, p, p, p, p, p, p, None), "sizes"),
            ("skyrl_gdelta_out", (gd(2, 8), p, 1, p, p, p, p, 15, p, p, 16, _ffi.F32, None), "sizes"),
            ("skyrl_moe_route", (moe(64, 32, 8, 2, 3, 1), p, 1, p, p, p, p, _ffi.F32, None), "multiple of groups"),
            ("skyrl_moe_route", (moe(64, 32, 8, 5, 2, 1), p, 1, p, p, p, p, _ffi.F32, None), "top must be"),
            ("skyrl_moe_route", (moe(64, 32, 2048, 2, 1, 1), p, 1, p, p, p, p, _ffi.F32, None), "1024"),
            ("skyrl_moe_sort", (p, 20, 8, 16, 8, None, p, p, None), "too few tiles"),
            ("skyrl_moe_sort", (p, 20000, 8, 16, 9999, None, p, p, None), "counts"),
            ("skyrl_moe_sort", (p, 20, 8, 20, 99, None, p, p, None), "sizes"),
            ("skyrl_moe_gate_up", (ok, p, p, p, p, 24, 4, p, _ffi.F32, None), "plain form"),
            ("skyrl_moe_down", (ok, p, p, p, p, 16, 4, None, p, _ffi.F32, None), "null pointer")):
        with pytest.raises(_ffi.SkyrlHipError, match=msg):
            _ffi.call(name, *args)
    assert [_ffi.query("skyrl_moe_tiles", *a) for a in ((8, 20, 16), (8, 3, 16), (8, 0, 16), (4, 1000, 128))] == [9, 3, 0, 11]


def test_abi_version_and_error_path():
    lib = _ffi.load()
    assert lib.skyrl_abi_version() == 12
    # argument validation happens on the host before any launch: no GPU needed
    with pytest.raises(_ffi.SkyrlHipError, match="temperature"):
        _ffi.call("skyrl_logprob_fwd", ctypes.c_void_p(16), _ffi.BF16, 8, 8, 1, 1, 8, ctypes.c_void_p(16), 1, 1,
                  -1.0, ctypes.c_void_p(16), None, None, None)
    assert "temperature" in lib.skyrl_last_error().decode()


def test_workspace_queries():
    assert _ffi.query("skyrl_ppo_loss_workspace_bytes", 512, 1024) >= 512 * 5 * 4
    assert _ffi.query("skyrl_sample_workspace_bytes", 512, 151936) > 0
    assert _ffi.query("skyrl_gae_workspace_bytes", 512) >= 512 * 24


def test_workspace_queries_degenerate_sizes():
    """Host-only size queries must not trap (e.g. divide by zero) on empty batches."""
    for name, args in (("skyrl_sample_workspace_bytes", (0, 7)), ("skyrl_sample_workspace_bytes", (1, 1)),
                       ("skyrl_gae_workspace_bytes", (0,)), ("skyrl_ppo_loss_workspace_bytes", (0, 0)),
                       ("skyrl_reward_kl_workspace_bytes", (0,)), ("skyrl_critic_loss_workspace_bytes", (0, 0)),
                       ("skyrl_policy_train_workspace_bytes", (0, 0)), ("skyrl_sumsq_workspace_bytes", (0,))):
        assert _ffi.query(name, *args) > 0, name


def test_oracle_sampler_builds():
    path = os.path.join(ROOT, "oracle", "_build", "libsampler_ref.so")
    assert os.path.exists(path), "oracle C restatement not built (make -C oracle)"
    ctypes.CDLL(path).sampler_ref


def test_cpu_tensor_is_rejected_not_computed():
    import torch

    from skyrl_amd import ops

    with pytest.raises(RuntimeError, match="no CPU fallback"):
        ops.approx_kl(torch.zeros(4), torch.zeros(4))


def test_grpo_ppo_loss_entry_validates_on_host():
    """skyrl_grpo_ppo_loss_fwd checks its layout before any launch: no GPU needed."""
    params = _ffi.PPOParams(0.2, 0.2, 3.0, 0, 0, 0.0, 1, 3, 0.001, 0, 0.0, 0)
    p = ctypes.c_void_p(16)
    args = lambda ng, mdt: (p, None, p, mdt, ng, 1e-6, 1, p, p, p, p, None, p, 512, 1024,  # noqa: E731
                            ctypes.byref(params), p, p, p, p, None, 0, p, None)
    with pytest.raises(_ffi.SkyrlHipError, match="n % num_groups"):
        _ffi.call("skyrl_grpo_ppo_loss_fwd", *args(7, _ffi.I64))
    with pytest.raises(_ffi.SkyrlHipError, match="mask dtype"):
        _ffi.call("skyrl_grpo_ppo_loss_fwd", *args(64, 99))
    with pytest.raises(_ffi.SkyrlHipError, match="params is null"):
        a = list(args(64, _ffi.I64))
        a[15] = None
        _ffi.call("skyrl_grpo_ppo_loss_fwd", *a)
    with pytest.raises(_ffi.SkyrlHipError, match="unknown flags"):
        a = list(args(64, _ffi.I64))
        a[21] = 6
        _ffi.call("skyrl_grpo_ppo_loss_fwd", *a)
    with pytest.raises(_ffi.SkyrlHipError, match="null pointer"):
        a = list(args(64, _ffi.I64))
        a[0] = None  # neither rewards nor scores
        _ffi.call("skyrl_grpo_ppo_loss_fwd", *a)


def test_ppo_loss_finish_validates_on_host():
    params = _ffi.PPOParams(0.2, 0.2, 3.0, 0, 0, 0.0, 1, 3, 0.001, 0, 0.0, 0)
    p = ctypes.c_void_p(16)
    with pytest.raises(_ffi.SkyrlHipError, match="ppo_loss_finish: null pointer"):
        _ffi.call("skyrl_ppo_loss_finish", None, None, None, 4, 4, ctypes.byref(params), p, p, None, None)
    with pytest.raises(_ffi.SkyrlHipError, match="grad_out needs grad_logp"):
        _ffi.call("skyrl_ppo_loss_finish", p, None, None, 4, 4, ctypes.byref(params), p, p, p, None)
    with pytest.raises(_ffi.SkyrlHipError, match="bad sizes"):
        _ffi.call("skyrl_ppo_loss_finish", None, None, None, 0, 4, ctypes.byref(params), p, p, p, None)


def test_comm_abi_host_checks():
    """The RCCL entry points validate on the host (no GPU, no RCCL call)."""
    assert _ffi.query("skyrl_comm_unique_id_bytes") == 128  # sizeof(ncclUniqueId)
    with pytest.raises(_ffi.SkyrlHipError, match="null pointer"):
        _ffi.call("skyrl_comm_init", None, 1, 0, ctypes.byref(ctypes.c_void_p()))
    with pytest.raises(_ffi.SkyrlHipError, match="rank must be"):
        _ffi.call("skyrl_comm_init", ctypes.c_void_p(16), 2, 2, ctypes.byref(ctypes.c_void_p()))
    with pytest.raises(_ffi.SkyrlHipError, match="null communicator"):
        _ffi.call("skyrl_comm_allreduce", ctypes.c_void_p(16), ctypes.c_void_p(16), 4, _ffi.F32, 0, None, None)
    with pytest.raises(_ffi.SkyrlHipError, match="dtype"):
        _ffi.call("skyrl_comm_broadcast", ctypes.c_void_p(16), ctypes.c_void_p(16), 4, 9, 0, ctypes.c_void_p(16), None)
    assert _ffi.call("skyrl_comm_destroy", None) == 0


def _exported_symbols():
    import subprocess

    out = subprocess.run(["nm", "-D", "--defined-only", _ffi.LIB_PATH], stdout=subprocess.PIPE, text=True, check=True)
    return sorted({ln.split()[-1] for ln in out.stdout.splitlines() if " T " in ln and ln.split()[-1].startswith("skyrl_")})


def test_no_process_state_setters_exported():
    """reentrant entry points, no global mutable state. The A/B
    knobs are a caller-owned skyrl_variant passed to one *_ex call; nothing exported stores state:
    no skyrl_tune, no test hook, and every exported C symbol is an entry point of skyrl_hip.h."""
    syms = _exported_symbols()
    assert syms == header_functions(), set(syms) ^ set(header_functions())
    assert not [s for s in syms if "tune" in s or "occupy" in s or s.startswith("skyrl_set")]
    assert all(n + "_ex" in syms for n in _ffi.EX_FORMS)


def test_variant_applies_to_its_call_only():
    """A variant changes the decision of the call it is passed to and of no other call: the
    fused-pass support query (host-only, no GPU) with the 4 x 256 split shape at V = 200,000 says
    no; the plain call before and after, and an _ex call with NULL or an all-default variant, say
    yes. A bad field fails that call alone."""
    lib = _ffi.load()
    V = 200_000
    v = _ffi.Variant(train_split_shape=2)
    d = _ffi.Variant()
    lib.skyrl_variant_init(ctypes.byref(d))
    assert all(getattr(d, f) == _ffi.VARIANT_DEFAULT for f in _ffi.VARIANT_FIELDS)
    assert lib.skyrl_policy_train_supports(V, 1, 1.0) == 1
    assert lib.skyrl_policy_train_supports_ex(V, 1, 1.0, ctypes.byref(v)) == 0
    assert lib.skyrl_policy_train_supports(V, 1, 1.0) == 1
    assert lib.skyrl_policy_train_supports_ex(V, 1, 1.0, None) == 1
    assert lib.skyrl_policy_train_supports_ex(V, 1, 1.0, ctypes.byref(d)) == 1
    bad = _ffi.Variant(sampler_split_nt=300)
    assert lib.skyrl_policy_train_supports_ex(V, 1, 1.0, ctypes.byref(bad)) == -1
    with pytest.raises(_ffi.SkyrlHipError, match="bad value for sampler_split_nt"):
        _ffi.call("skyrl_sample_ex", ctypes.c_void_p(16), _ffi.BF16, 8, 1, 8, 1.0, -1, 1.0, 0.0, 0, None, 0,
                  ctypes.c_void_p(16), None, ctypes.c_void_p(16), None, ctypes.byref(bad))
    # the host-side scope: nested scopes override fields, leaving restores the enclosing one
    with _ffi.variant(train_split_shape=2):
        assert _ffi.query("skyrl_policy_train_supports", V, 1, 1.0) == 0
        with _ffi.variant(train_split_shape=5):
            assert _ffi.query("skyrl_policy_train_supports", V, 1, 1.0) == 1
        assert _ffi.query("skyrl_policy_train_supports", V, 1, 1.0) == 0
    assert _ffi.query("skyrl_policy_train_supports", V, 1, 1.0) == 1 and _ffi.current_variant() is None
