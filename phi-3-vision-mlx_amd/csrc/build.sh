#!/bin/bash
# Build libp3v.so (all HIP kernels + the C ABI) for gfx950, in-tree: one object per translation unit, compiled in parallel, then linked.
#
#   build.sh                      every translation unit -> ../libp3v.so
#   P3V_UNITS="a b" P3V_OUT=../libp3v_x.so build.sh   only these units (names without p3v_ / .hip): a partial library
#                                 for a program that needs no more (_lib.py binds what a partial library has)
# Extra arguments go to every hipcc compile line.
set -e
cd "$(dirname "$0")"
OUT=${P3V_OUT:-../libp3v.so}
UNITS=${P3V_UNITS:-elementwise gemm gemm256 gemm_skinny gemm_rows gemm_fp8 gemv gemv_fp8 gemv_q4 attention layered attn_mix latent latent_prompt gla lora preprocess runtime}
# packed fp32 instructions stay off: hipcc forms them from ordinary float code and some of their forms have given wrong results on this chip
FLAGS="--offload-arch=gfx950 -O3 -std=c++17 -fPIC -Wno-unused-result -Xclang -target-feature -Xclang -packed-fp32-ops"
OBJ=$(mktemp -d "${TMPDIR:-/tmp}/p3v_build.XXXXXX")
trap 'rm -rf "$OBJ"' EXIT
# attn_mix, latent, latent_prompt: no NaN reaches their maxima by design (masked scores are -inf), so they need no NaN quieting
compile() { local x=; case "$1" in attn_mix | latent | latent_prompt) x=-fno-honor-nans ;; esac; hipcc $FLAGS $x "${@:2}" -c "p3v_$1.hip" -o "$OBJ/$1.o" 2> "$OBJ/$1.log" || { cat "$OBJ/$1.log" >&2; return 1; }; grep -v "packed-fp32-ops\|^$" "$OBJ/$1.log" >&2 || true; }
PIDS=()
MAX=${MAX_JOBS:-$(nproc)}; [ "$MAX" -gt 16 ] && MAX=16
for u in $UNITS; do
  while [ "$(jobs -rp | wc -l)" -ge "$MAX" ]; do wait -n || exit 1; done
  compile "$u" "$@" & PIDS+=($!)
done
for p in "${PIDS[@]}"; do wait "$p" || exit 1; done
# -z defs: a kernel whose host stub hipcc dropped fails the link, not the dlopen; the finished file replaces the old one in one step
hipcc --offload-arch=gfx950 -shared -fPIC -Wl,-z,defs $(for u in $UNITS; do echo "$OBJ/$u.o"; done) -o "$OUT.tmp.$$"
mv -f "$OUT.tmp.$$" "$OUT"
echo "built $(realpath "$OUT")"
