// stack_ssd.hip — launches of the blocked scalar-decay state-space recurrence on the matrix cores (kernels/stack_ssd_mfma.h); a translation unit of its own so that its
// template instances compile beside stack.hip.
#include "stack.h"

#include "kernels/stack_ssd_mfma.h"

bool ssd_mfma_shapes_ok(int heads, int groups, int N, int E, long long ld) { return N % 4 == 0 && N <= 256 && (heads * E) % 4 == 0 && ld % 4 == 0 && groups > 0; }
size_t ssd_gram_elems(int T, int S, int groups) { return ((size_t)T / tgx::SSD_BLOCK + (size_t)S + 1) * groups * tgx::SSD_BLOCK * tgx::SSD_BLOCK; }

void launch_ssd_mfma(tgx_ctx* c, const tgx::StepMeta& m, const tgx::SsdArgs& a, int S, int max_count) {
  if (!ssd_mfma_shapes_ok(a.heads, a.groups, a.N, a.E, a.ld)) { c->launch_fault = "blocked state-space recurrence: sizes it does not take"; return; }
  hipLaunchKernelGGL(tgx::ssd_gram_kernel<>, dim3((max_count + tgx::SSD_BLOCK - 1) / tgx::SSD_BLOCK, a.groups, S), dim3(256), 0, c->stream, m, a);
  const dim3 grid(S, a.heads, (a.E + 31) / 32);
  if (a.N <= 128) hipLaunchKernelGGL(tgx::ssd_block_kernel<1>, grid, dim3(256), 0, c->stream, m, a);
  else hipLaunchKernelGGL(tgx::ssd_block_kernel<2>, grid, dim3(256), 0, c->stream, m, a);
}
