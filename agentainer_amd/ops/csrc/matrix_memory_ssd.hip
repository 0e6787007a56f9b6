// Instantiations of the matrix-memory recurrence kernel: state-space
// recurrence (one decay per head, step-sized writes, skip).
#include "matrix_memory_kernel.h"

namespace mm {
void launch_ssd(const ScanArgs& a, int B, int lanes, bool bf16,
                hipStream_t stream) {
  if (bf16) launch_scan<KIND_SSD, short>(a, B, lanes, stream);
  else launch_scan<KIND_SSD, float>(a, B, lanes, stream);
}
}  // namespace mm
