"""Building and loading the HIP kernel library (gfx950).

The sources under ``csrc/`` are compiled with hipcc into one shared object with a
plain C interface, loaded through ctypes.  ``load()`` uses the built library if
its recorded digest matches the sources, and builds otherwise (first call in a
fresh checkout); ``build()`` always compiles.  There is no other implementation
behind these entry points: without the library every op raises.
"""
import ctypes
import fcntl
import hashlib
import os
import shutil
import stat
import subprocess
import sys
import tempfile
import time
from pathlib import Path

CSRC = Path(__file__).resolve().parent.parent / 'csrc'
ARCH = 'gfx950'
# packed-fp32 off: hipcc may otherwise form v_pk_*_f32, which must not be used on this hardware pool.
FLAGS = [f'--offload-arch={ARCH}', '-O3', '-fPIC', '-std=c++17', '-Xclang', '-target-feature', '-Xclang',
         '-packed-fp32-ops']
LIBRARY_NAME = 'libqil_hip.so'

_library = None


class KernelLibraryError(RuntimeError):
    pass


def sources():
    return sorted(CSRC.glob('*.hip'))


def digest():
    h = hashlib.sha256(' '.join(FLAGS).encode())
    for path in sorted(list(CSRC.glob('*.hip')) + list(CSRC.glob('*.h'))):
        h.update(path.name.encode())
        h.update(path.read_bytes())
    return h.hexdigest()


def _in_tree():
    return CSRC / '_build'


def _writable(folder):
    try:
        folder.mkdir(exist_ok=True)
        probe = folder / f'.probe{os.getpid()}'
        probe.write_text('')
        probe.unlink()
        return True
    except OSError:
        return False


def _private_folder():
    """The per-user folder that stands in when the package's own folder cannot be written (an installed package):
    ``$XDG_CACHE_HOME/qil_amd`` or ``~/.cache/qil_amd``; without a usable home, a folder under the temp dir."""
    base = os.environ.get('XDG_CACHE_HOME')
    if base:
        return Path(base) / 'qil_amd'
    home = Path(os.path.expanduser('~'))
    if str(home) not in ('~', '/') and home.is_dir() and os.access(home, os.W_OK | os.X_OK):
        return home / '.cache' / 'qil_amd'
    return Path(tempfile.gettempdir()) / f'qil_amd_build_{os.getuid()}'


def _trusted(folder):
    """Whether a folder outside the package may hold a library that this process loads: it is a real folder (no
    link), owned by this user, and nobody else may write to it.  A folder that someone else could have made or
    filled (a predictable name in a shared temp dir) must not be loaded from."""
    try:
        status = os.lstat(folder)
    except OSError:
        return False
    return stat.S_ISDIR(status.st_mode) and status.st_uid == os.getuid() and not status.st_mode & 0o022


def build_dir():
    """In-tree ``csrc/_build`` when writable, else the per-user folder, made for this user alone (mode 0700)."""
    local = _in_tree()
    if _writable(local):
        return local
    fallback = _private_folder()
    try:
        fallback.mkdir(mode=0o700, parents=True, exist_ok=True)
    except OSError as error:
        raise KernelLibraryError(f'no folder to build the kernel library in: {error}') from None
    if not _trusted(fallback):
        raise KernelLibraryError(f'{fallback} is not a folder of this user alone (owner, or write permission of '
                                 'others): refusing to build into it or to load a library from it')
    return fallback


def _hipcc():
    found = shutil.which('hipcc') or ('/opt/rocm/bin/hipcc' if Path('/opt/rocm/bin/hipcc').exists() else None)
    if not found:
        raise KernelLibraryError('hipcc not found: the HIP kernels cannot be built, and there is no other path')
    return found


def _say(message):
    print(f'[qil_amd build] {message}', file=sys.stderr, flush=True)


def build(verbose=True):
    """Compile every source and link the library.  Returns its path."""
    out = build_dir()
    hipcc = _hipcc()
    with open(out / '.lock', 'w') as lock:
        fcntl.flock(lock, fcntl.LOCK_EX)
        started = time.time()
        jobs = []
        for source in sources():
            obj = out / (source.stem + '.o')
            command = [hipcc, *FLAGS, '-c', str(source), '-o', str(obj)]
            jobs.append((source, obj, subprocess.Popen(command, stdout=subprocess.PIPE, stderr=subprocess.STDOUT,
                                                       text=True)))
        if verbose:
            _say(f'compiling {len(jobs)} HIP sources for {ARCH} into {out}')
        pending = list(jobs)
        last = time.time()
        while pending:
            pending = [job for job in pending if job[2].poll() is None]
            if pending and verbose and time.time() - last > 10:
                _say(f'still compiling: {", ".join(job[0].name for job in pending)} ({time.time() - started:.0f} s)')
                last = time.time()
            time.sleep(0.2)
        for source, obj, process in jobs:
            text = process.stdout.read()
            if process.returncode:
                raise KernelLibraryError(f'hipcc failed on {source.name}:\n{text}')
        target = out / LIBRARY_NAME
        scratch = out / f'.{LIBRARY_NAME}.{os.getpid()}'
        link = subprocess.run([hipcc, '-shared', '-fPIC', f'--offload-arch={ARCH}', '-o', str(scratch),
                               *[str(obj) for _, obj, _ in jobs]], stdout=subprocess.PIPE, stderr=subprocess.STDOUT,
                              text=True)
        if link.returncode:
            raise KernelLibraryError(f'linking {LIBRARY_NAME} failed:\n{link.stdout}')
        os.replace(scratch, target)
        (out / 'digest.txt').write_text(digest())
        if verbose:
            _say(f'built {target} in {time.time() - started:.0f} s')
    return target


def built_library():
    """Path of a built library whose digest matches the sources, or None.  The per-user folder is looked at only
    when the package's own folder cannot be written, and only if it belongs to this user alone."""
    folders = [_in_tree()]
    if not _writable(_in_tree()):
        fallback = _private_folder()
        if _trusted(fallback):
            folders.append(fallback)
    for folder in folders:
        target, record = folder / LIBRARY_NAME, folder / 'digest.txt'
        if target.exists() and record.exists() and record.read_text() == digest():
            return target
    return None


def load():
    global _library
    if _library is None:
        path = built_library()
        if path is None:
            _say('no built kernel library matches the sources; building now')
            path = build()
        try:
            _library = ctypes.CDLL(str(path))
        except OSError as error:
            raise KernelLibraryError(f'cannot load {path}: {error}') from None
        _declare(_library)
        _library.path = str(path)
    return _library


PLANNED_COMPUTE_UNITS, PLANNED_LDS_BYTES = 256, 160 * 1024      # the first also stands in the library (QIL_CUS)
_device_checked = False


def check_device():
    """Once per process, on the first launch: (compute units, LDS bytes a block) of the current GPU, with a warning
    if they are not what the kernels' plans were made for (results stay right, the plans do not fit)."""
    global _device_checked
    if _device_checked:
        return
    _device_checked = True
    units, lds = ctypes.c_int(0), ctypes.c_int(0)
    if load().qil_planned_compute_units() != PLANNED_COMPUTE_UNITS:
        raise RuntimeError('the kernel library and the Python side plan for different numbers of compute units')
    if load().qil_device_info(ctypes.byref(units), ctypes.byref(lds)) == 0 and \
            (units.value != PLANNED_COMPUTE_UNITS or lds.value < PLANNED_LDS_BYTES):
        _say(f'this GPU shows {units.value} compute units and {lds.value} bytes of LDS a block; the kernels\' block '
             f'shapes and splits are planned for {PLANNED_COMPUTE_UNITS} and {PLANNED_LDS_BYTES} (an MI355X as one '
             'device): results are unaffected, speed is not what was measured')


def _declare(lib):
    p, i, f, z = ctypes.c_void_p, ctypes.c_int, ctypes.c_float, ctypes.c_size_t
    lib.qil_device_info.argtypes = [ctypes.POINTER(ctypes.c_int), ctypes.POINTER(ctypes.c_int)]
    lib.qil_planned_compute_units.argtypes = []
    lib.qil_planned_compute_units.restype = i
    lib.qil_device_info.restype = i
    lib.qil_embed.argtypes = [p, p, p, i, i, f, i, p]
    lib.qil_add_rmsnorm.argtypes = [p, p, i, i, i, p, p, p, i, i, f, i, i, p]
    lib.qil_silu_mul.argtypes = [p, i, i, p, i, i, i, i, p]
    lib.qil_add_bias.argtypes = [p, p, i, i, i, p]
    lib.qil_qk_norm_rope_store.argtypes = [p, i, i, p, p, p, p, p, p, p, p, p, i, i, i, i, i, i, f, i, i, i, f, i, p, i, i, p]
    lib.qil_qk_row_norm_store.argtypes = [p, i, i, p, p, p, p, p, p, p, p, p, i, i, i, i, i, i, f, i, i, i, i, i, p]
    lib.qil_attn_rows_workspace.argtypes = [i, i, i, i]
    lib.qil_attn_rows_workspace.restype = z
    lib.qil_attn_rows.argtypes = [p, i, p, p, p, i, p, p, p, p, p, i, i, i, i, i, i, f, f, i, i, i, p, p, i, p]
    lib.qil_attn_merge.argtypes = [p, p, p, p, i, i, i, i, i, i, i, p, i, p, i, i, i, i, p]
    lib.qil_attn_decode_fused_takes.argtypes = [i, i, i, i, i]
    lib.qil_attn_decode_fused_takes.restype = i
    lib.qil_attn_decode_fused.argtypes = [p, i, p, p, f, p, p, i, i, p, p, p, i, p, p, p, p, i, i, i, i, i, i, f, i, i, i, i, i, f, i, i, p, f, i, p, i, p, i, p]
    lib.qil_attn_decode_takes.argtypes = [i, i, i, i]
    lib.qil_attn_decode_takes.restype = i
    lib.qil_attn_decode.argtypes = [p, i, p, p, p, i, p, p, p, p, p, i, i, i, i, i, i, f, i, i, i, i, f, p, p, i, p]
    lib.qil_attn_tile.argtypes = [p, i, p, p, p, i, p, p, p, i, i, i, i, i, i, i, f, f, i, p, p, i, p]
    lib.qil_gemm_f32.argtypes = [p, p, p, p, i, i, i, i, p]
    lib.qil_gemm_f32_splits.argtypes = [i, i, i]
    lib.qil_gemm_f32_waves.argtypes = [i, i, i, i]
    lib.qil_gemm_f32_waves.restype = i
    lib.qil_gemm_f32_unmerged_takes.argtypes = [i, i, i, i, i]
    lib.qil_gemm_f32_unmerged_takes.restype = i
    lib.qil_gemm_f32_unmerged.argtypes = [p, p, p, p, i, i, i, i, i, i, i, i, p]
    lib.qil_gemm_f32_unmerged.restype = i
    lib.qil_gemm_f32_gated_takes.argtypes = [i, i, i, i, i]
    lib.qil_gemm_f32_gated_takes.restype = i
    lib.qil_gemm_f32_gated.argtypes = [p, i, i, p, p, i, i, i, i, p]
    lib.qil_gemm_f32_gated.restype = i
    lib.qil_attn_rows_unmerged.argtypes = [p, i, p, p, p, i, p, p, p, i, i, i, i, i, i, f, f, i, i, i, p]
    lib.qil_attn_rows_unmerged.restype = i
    lib.qil_gemm_f32_mfma.argtypes = [p, p, p, p, i, i, i, i, p]
    lib.qil_gemm_f32_mfma_takes.argtypes = [i, i, i, i]
    lib.qil_gemm_f32_mfma_splits.argtypes = [i, i, i]
    lib.qil_gemm_f32_mfma_splits.restype = i
    lib.qil_gemm_f32_mfma_takes.restype = i
    lib.qil_gemm_f32_splits.restype = i
    lib.qil_gemm_bf16.argtypes = [p, p, p, p, i, i, i, i, i, i, i, p]
    lib.qil_gemm_bf16_splits.argtypes = [i, i, i]
    lib.qil_gemm_bf16_splits.restype = i
    lib.qil_attn_tile_bf16_takes.argtypes = [i, i, i]
    lib.qil_attn_tile_bf16_takes.restype = i
    lib.qil_attn_tile_parts.argtypes = [i, i, i, i, i, i, i, i, ctypes.POINTER(ctypes.c_int)]
    lib.qil_attn_tile_parts.restype = i
    lib.qil_attn_tile_bf16_parts.argtypes = [p, i, p, p, p, i, p, p, p, i, i, i, i, i, i, i, i, f, i, i, p]
    lib.qil_attn_tile_bf16_parts.restype = i
    lib.qil_attn_tile_key_parts.argtypes = [i, i, i, i, i, i, i, ctypes.POINTER(ctypes.c_int)]
    lib.qil_attn_tile_key_parts.restype = i
    lib.qil_attn_tile_in_parts.argtypes = [p, i, p, p, p, i, p, p, p, i, i, i, i, i, i, i, i, f, f, i, i, i, p, p]
    lib.qil_attn_tile_in_parts.restype = i
    lib.qil_attn_tile_waves.argtypes = [i]
    lib.qil_attn_tile_waves.restype = None
    lib.qil_gemm_bf16_streams.argtypes = [i, i, i, i]
    lib.qil_gemm_bf16_streams.restype = i
    lib.qil_gemm_bf16_unmerged.argtypes = [p, p, p, p, i, i, i, i, i, i, i, i, p]
    lib.qil_gemm_bf16_unmerged_takes.argtypes = [i, i, i, i, i]
    lib.qil_gemm_bf16_unmerged_takes.restype = i
    lib.qil_gemm_bf16_gated.argtypes = [p, p, p, i, i, i, i, i, i, i, p]
    lib.qil_gemm_bf16_gated_takes.argtypes = [i, i, i, i]
    lib.qil_gemm_bf16_gated_takes.restype = i
    lib.qil_gemm_bf16_normed_takes.argtypes = [i, i, i, i]
    lib.qil_gemm_bf16_normed_takes.restype = i
    lib.qil_gemm_bf16_normed.argtypes = [p, p, p, i, f, p, p, i, i, i, i, p]
    lib.qil_gemm_bf16_add_takes.argtypes = [i, i, i]
    lib.qil_gemm_bf16_add_takes.restype = i
    lib.qil_gemm_bf16_add.argtypes = [p, p, p, p, i, i, i, i, i, p]
    lib.qil_gemm_bf16_mid_splits.argtypes = [i, i, i]
    lib.qil_gemm_bf16_mid_splits.restype = i
    lib.qil_gemm_bf16_mid.argtypes = [p, p, p, i, i, i, i, i, p]
    lib.qil_gemm_bf16_mid_rows_takes.argtypes = [i, i, i]
    lib.qil_gemm_bf16_mid_rows_takes.restype = i
    lib.qil_gemm_bf16_mid_gated_takes.argtypes = [i, i, i]
    lib.qil_gemm_bf16_mid_gated_takes.restype = i
    lib.qil_gemm_bf16_mid_gated.argtypes = [p, p, p, i, i, i, i, p]
    lib.qil_gemm_bf16_wide_takes.argtypes = [i, i, i, i]
    lib.qil_gemm_bf16_wide_takes.restype = i
    lib.qil_gemm_bf16_wide.argtypes = [p, p, p, i, i, i, i, i, p]
    lib.qil_gemm_bf16_wide_gated_takes.argtypes = [i, i, i]
    lib.qil_gemm_bf16_wide_gated_takes.restype = i
    lib.qil_gemm_bf16_wide_gated.argtypes = [p, p, p, i, i, i, i, p]
    lib.qil_add_norm.argtypes = [p, p, i, i, i, f, p, p, p, p, i, i, f, i, i, i, p]
    lib.qil_gated_act.argtypes = [p, i, i, i, p, i, i, i, i, i, f, f, p]
    lib.qil_latent_prepare.argtypes = [p, i, i, i, p, p, p, p, p, p, p, p, p, i, i, i, i, i, f, i, p]
    lib.qil_head_product.argtypes = [p, i, i, i, p, i, p, i, i, i, i, i, i, i, p, i, i, i, p]
    lib.qil_gated_heads.argtypes = [p, p, i, i, i, p, i, i, i, p]
    lib.qil_gated_heads.restype = i
    lib.qil_rotate_tail.argtypes = [p, i, i, i, i, p, p, p, i, i, i, i, i, i, p]
    lib.qil_latent_attention_takes.argtypes = [i, i, i]
    lib.qil_latent_attention_takes.restype = i
    lib.qil_latent_attention.argtypes = [p, p, p, p, i, p, p, p, p, p, i, i, i, i, i, f, i, i, p]
    lib.qil_latent_mfma_takes.argtypes = [i, i, i]
    lib.qil_latent_mfma_takes.restype = i
    ip = ctypes.POINTER(ctypes.c_int)
    lib.qil_latent_mfma_plan.argtypes = [i, i, i, i, i, i, ip, ip, ip, ip]
    lib.qil_latent_mfma_plan.restype = None
    lib.qil_latent_mfma_workspace.argtypes = [i, i, i, i]
    lib.qil_latent_mfma_workspace.restype = z
    lib.qil_latent_mfma.argtypes = [p, p, p, p, i, p, p, p, p, p, p, p, i, i, i, i, i, i, i, f, i, i, i, i, i, p]
    lib.qil_latent_mfma.restype = i
    lib.qil_state_scan_slot.argtypes = [i, i, i, i]
    lib.qil_state_scan_slot.restype = z
    lib.qil_state_scan_takes.argtypes = [i, i, i]
    lib.qil_state_scan_takes.restype = i
    lib.qil_state_scan.argtypes = [p, i, i, i, i, i, p, p, f, p, p, i, f, f, p, p, p, p, p, p, i, i, i, i, i, p, i, i, i, i, i, p]
    lib.qil_head_norm_gate.argtypes = [p, p, p, i, i, p, p, i, i, i, f, i, i, p]
    lib.qil_state_scan_chunked_workspace.argtypes = [i, i, i, i, i, i]
    lib.qil_state_scan_chunked_workspace.restype = z
    lib.qil_state_scan_chunked.argtypes = [p, i, i, i, i, i, p, p, f, p, p, i, f, f, p, z, p, p, p, p, p, p, i, i, i, i, i, i, i, p, i, i, i, i, p]
    lib.qil_state_scan_chunked.restype = i
    for name in ('qil_add_norm', 'qil_gated_act', 'qil_latent_prepare', 'qil_head_product', 'qil_rotate_tail',
                 'qil_latent_attention', 'qil_state_scan', 'qil_head_norm_gate'):
        getattr(lib, name).restype = i
    lib.qil_post_norm_add_norm.argtypes = [p, p, i, i, i, p, f, p, p, p, i, i, f, i, i, p]
    lib.qil_post_norm_add_norm.restype = i
    lib.qil_post_norm_add_norm_routed.argtypes = [p, p, p, p, p, i, i, p, f, p, p, p, i, i, f, i, i, p]
    lib.qil_post_norm_add_norm_routed.restype = i
    lib.qil_moe_combine.argtypes = [p, i, p, p, p, p, i, i, i, i, p]
    lib.qil_moe_combine.restype = i
    lib.qil_moe_takes.argtypes = [i, i, i, i, i, i]
    lib.qil_moe_takes.restype = i
    lib.qil_moe_route.argtypes = [p, i, p, p, p, p, p, p, i, i, i, i, i, i, i, i, i, f, f, i, i, i, p, p, p]
    lib.qil_moe_aligns.argtypes = [i, i, i, i]
    lib.qil_moe_aligns.restype = i
    lib.qil_moe_route.restype = i
    lib.qil_scaled_sum.argtypes = [p, i, i, p, i, i, f, f, p, i, i, p]
    lib.qil_sigmoid_gate.argtypes = [p, p, i, i, i, i, p, i, i, i, p]
    lib.qil_soft_cap.argtypes = [p, f, z, p]
    lib.qil_channel_conv.argtypes = [p, i, i, i, p, p, p, p, p, p, p, p, i, i, i, i, i, i, i, p, p]
    lib.qil_selective_scan_takes.argtypes = [i, i, i]
    lib.qil_selective_scan.argtypes = [p, p, i, i, p, p, p, i, i, p, p, i, i, i, i, p, p, p, p, p, i, i, i, i, i, i, p, p]
    lib.qil_selective_scan_workspace.argtypes = [i, i, i, i]
    lib.qil_selective_scan_workspace.restype = z
    for name in ('qil_scaled_sum', 'qil_sigmoid_gate', 'qil_soft_cap', 'qil_channel_conv', 'qil_selective_scan_takes',
                 'qil_selective_scan'):
        getattr(lib, name).restype = i
    lib.qil_moe_tile_rows.argtypes = [i, i]
    lib.qil_moe_tile_rows.restype = i
    lib.qil_moe_max_tiles.argtypes = [i, i, i]
    lib.qil_moe_max_tiles.restype = i
    lib.qil_moe_experts.argtypes = [p, i, p, p, p, p, p, p, p, p, p, i, i, i, i, i, i, i, i, f, f, i, p]
    lib.qil_moe_experts.restype = i
    lib.qil_post_norm_scale_add.argtypes = [p, p, i, i, p, p, p, f, i, p, i, p, i, p, i, i, p]
    lib.qil_post_norm_scale_add.restype = i
    lib.qil_post_norm_scale_add_routed.argtypes = [p, p, p, p, p, i, i, i, p, p, p, f, i, p, i, p, i, p, i, i, p]
    lib.qil_post_norm_scale_add_routed.restype = i
    lib.qil_short_conv.argtypes = [p, p, p, p, p, p, p, p, i, i, i, i, p]
    lib.qil_short_conv.restype = i
    lib.qil_plain_act.argtypes = [p, i, i, p, i, i, i, i, p, p]
    lib.qil_plain_act.restype = i
    ll = ctypes.c_longlong
    lib.qil_embed_pairs.argtypes = [p, p, p, p, p, p, i, i, f, i, ll, ll, i, p]
    lib.qil_gated_group_norm.argtypes = [p, p, i, p, p, i, i, i, p, p, i, i, i, i, i, f, f, i, p]
    lib.qil_residual_join.argtypes = [p, p, i, i, i, f, p, i, i, i, f, p, i, i, i, p, i, i, i, p, p, p, p, p, p, i, i, i, f, i, i, p]
    lib.qil_step_scan_takes.argtypes = [i, i, i, i, i, i]
    lib.qil_step_token_takes.argtypes = [i, i]
    lib.qil_step_scan_workspace.argtypes = [i, i, i, i, i]
    lib.qil_step_scan_workspace.restype = z
    lib.qil_step_scan.argtypes = [p, i, i, i, i, p, i, i, i, p, p, p, p, p, p, p, p, i, i, i, i, i, i, i, p]
    lib.qil_step_token.argtypes = [p, i, i, i, i, i, p, i, i, i, p, p, p, p, p, p, p, i, i, i, i, i, i, p]
    for name in ('qil_step_scan_takes', 'qil_step_token_takes', 'qil_step_scan', 'qil_step_token', 'qil_embed_pairs', 'qil_gated_group_norm', 'qil_residual_join', 'qil_qk_row_norm_store'):
        getattr(lib, name).restype = i
    lib.qil_stream_join_takes.argtypes = [i]
    lib.qil_stream_join.argtypes = [p, i, p, i, i, i, p, p, p, p, i, i, p, p, p, p, p, p, p, p, i, i, i, i, i, p]
    lib.qil_embed_streams.argtypes = [p, p, p, i, i, i, f, i, p]
    lib.qil_pair_store.argtypes = [p, i, i, i, p, p, p, p, i, i, i, i, i, i, i, i, p]
    lib.qil_difference_combine.argtypes = [p, p, p, i, i, i, p, i, i, i, f, f, f, p, i, i, i, i, i, p]
    lib.qil_delta_takes.argtypes = [i, i]
    lib.qil_delta_ends.argtypes = [i]
    operands = [p, i, i, i, i, i, p, i, i, i, p, p, p, i, i, i, p, p, p, p]      # rows, raw decays, step sizes, state and sequences
    lib.qil_delta_tokens.argtypes = operands + [p, p, p, p, i, i, i, f, i, i, i, i, i, i, p]
    lib.qil_delta_end.argtypes = [p, p, p, i, i, i, f, p, i, i, i, i, p]
    lib.qil_delta_chunked_takes.argtypes = [i, i, i, i, i, i]
    lib.qil_delta_chunked_workspace.argtypes = [i, i, i, i, i]
    lib.qil_delta_chunked_workspace.restype = z
    lib.qil_delta_chunked.argtypes = operands + [p, p, i, i, i, i, i, i, i, p]
    for name in ('qil_stream_join_takes', 'qil_stream_join', 'qil_embed_streams', 'qil_pair_store', 'qil_difference_combine',
                 'qil_delta_takes', 'qil_delta_ends', 'qil_delta_tokens', 'qil_delta_end', 'qil_delta_chunked_takes',
                 'qil_delta_chunked'):
        getattr(lib, name).restype = i
    lib.qil_sample.argtypes = [p, p, p, p, p, p, p, i, i, p]
    lib.qil_sample_workspace.argtypes = [i, i]
    lib.qil_sample_workspace.restype = z
    lib.qil_sample_static.argtypes = [p, p, p, p, p, p, i, i, p]
    lib.qil_sample_static.restype = i
    lib.qil_sample_static_prepare.argtypes = []
    lib.qil_sample_static_prepare.restype = i
    for name in ('qil_embed', 'qil_add_rmsnorm', 'qil_silu_mul', 'qil_add_bias', 'qil_qk_norm_rope_store',
                 'qil_attn_rows', 'qil_attn_merge', 'qil_attn_decode', 'qil_attn_decode_fused', 'qil_attn_tile', 'qil_gemm_f32', 'qil_gemm_bf16', 'qil_gemm_bf16_gated', 'qil_gemm_bf16_unmerged', 'qil_gemm_bf16_normed', 'qil_gemm_bf16_add', 'qil_sample'):
        getattr(lib, name).restype = i
