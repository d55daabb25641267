"""The ctypes bindings match the built gfx950 kernel libraries (CPU: dlopen only, no GPU calls)."""
import ctypes

import pytest

from docagents_amd.ops import build as B
from docagents_amd.ops import kernels as K


@pytest.mark.parametrize("part", B.PARTS)
def test_every_bound_symbol_is_exported(part):
    path = B.lib_path(part)
    if not path.exists():
        pytest.skip("kernel libraries not built (python -m docagents_amd.ops.build)")
    lib = ctypes.CDLL(str(path))
    bound = [n for n in K._SIGS if K._part_of(n) == part]
    missing = [n for n in bound if not hasattr(lib, n)]
    assert bound and not missing, f"bound in kernels.py but not exported by {path.name}: {missing}"


def test_every_source_belongs_to_one_part():
    parts = [p for part in B.PARTS for p in B._sources(part)]
    assert sorted(parts) == B._sources() and len(set(parts)) == len(parts)
