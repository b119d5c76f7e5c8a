// k_gemv instantiations for CTHIP_BF16 weights (see gemv_kernels.h).
#include "gemv_kernels.h"

namespace cthip {
extern const GemvVariant kGemvBF16[] = {
    GEMV_SHAPES_BF16(V)
};
extern const int kGemvBF16Count = (int)(sizeof(kGemvBF16) / sizeof(kGemvBF16[0]));
}  // namespace cthip
