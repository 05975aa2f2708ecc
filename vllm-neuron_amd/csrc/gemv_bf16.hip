// Token-generation weight stream, BF16 weights (templates: linear_device.h).
#include "linear_device.h"

namespace mi {
template int launch_gemv_wd<MI_W_BF16>(const LinearW&, int, int, const ProArgs&, int, const EpiArgs&, hipStream_t);
}
