// Token-generation weight stream, INT8 weights (templates: linear_device.h).
#include "linear_device.h"

namespace mi {
template int launch_gemv_wd<MI_W_INT8>(const LinearW&, int, int, const ProArgs&, int, const EpiArgs&, hipStream_t);
}
