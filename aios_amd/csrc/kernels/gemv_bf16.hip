// GEMV instantiations: BF16 weights.
#include "gemv_impl.h"
namespace aios {
void gemv_bf16(const GemvArgs& a, hipStream_t st) { launch_gemv_pair<QT_BF16, QT_BF16>(a, st); }
bool gemv_bf16_engine_fits(const GemvArgs& a) { return launch_gemv_lds16(a, nullptr, true); }
}  // namespace aios
