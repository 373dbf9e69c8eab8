"""The argument types that Python declares for the kernel libraries' entry points are those of the sources: a pointer
that is passed as an int would lose its upper half."""
import glob
import os
import re

import pytest

from allpaca_amd.kernels import build, lib

KINDS = {"int": lib.I, "long": lib.I, "float": lib.F, "size_t": lib.Z, "unsigned": lib.I}


def declared():
    out = {}
    for path in glob.glob(os.path.join(build.CSRC, "*.hip")):
        with open(path) as f:
            text = re.sub(r"//[^\n]*", "", f.read())
        for name, args in re.findall(r"APC_EXPORT\s+int\s+(apc_\w+)\s*\(([^)]*)\)\s*\{", text):
            kinds = []
            for a in [x.strip() for x in args.split(",") if x.strip() and x.strip() != "void"]:
                if "*" in a or "hipStream_t" in a:
                    kinds.append(lib.P)
                else:
                    kinds.append(KINDS[a.replace("const ", "").split()[0]])
            out[name] = kinds
    return out


SOURCES = declared()


@pytest.mark.parametrize("library", ["plain", "tuned", "bench"])
def test_argument_types_are_those_of_the_sources(library):
    assert len(SOURCES) > 60
    for name, args in lib.SIGNATURES[library].items():
        assert name in SOURCES, name
        assert args == SOURCES[name], (name, [a.__name__ for a in args], [a.__name__ for a in SOURCES[name]])
