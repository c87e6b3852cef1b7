// The boundary between two blocks of a float32 residual whose blocks read a layer norm (weight, no bias) of it and add
// their result as it is:  x <- x + y,  h = (x - mean) / sqrt(mean((x - mean)^2) + eps) * w.  One launch per token; the row
// stays in registers between the sums.  Routed experts may leave their sum to this launch: the rows of a token's (token,
// expert) pairs are added here in float32.  With token ids x is assigned a row of the embedding table instead.
#include "hm_common.h"

namespace hm {

// NP packs of VEC channels per thread: W <= 256 NP VEC
template <typename T, int VEC, int NP>
__global__ __launch_bounds__(256) void layer_norm_residual_kernel(float* __restrict__ x, const T* __restrict__ y,
                                                                  const int64_t* __restrict__ ids, const T* __restrict__ y2,
                                                                  const T* __restrict__ prod, const int32_t* __restrict__ pair_row,
                                                                  const float* __restrict__ wts, int top,
                                                                  const T* __restrict__ next_w, float eps, T* __restrict__ h_out,
                                                                  int W) {
    struct alignas(sizeof(T) * VEC) Pack { T v[VEC]; };
    struct alignas(4 * VEC) PackF { float v[VEC]; };
    __shared__ float red[16];
    const int64_t t = blockIdx.x;
    float* xr = x + (size_t)t * W;
    float v[NP][VEC], sum = 0.f;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int c = (threadIdx.x + 256 * p) * VEC;
#pragma unroll
        for (int e = 0; e < VEC; ++e) v[p][e] = 0.f;
        if (c >= W) continue;
        if (ids == nullptr) {
            const PackF a = *(const PackF*)(xr + c);
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[p][e] = a.v[e];
        }
        if (y != nullptr) {
            const Pack a = *(const Pack*)(y + (size_t)(ids ? ids[t] : t) * W + c);
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[p][e] += to_f(a.v[e]);
        }
        if (y2 != nullptr) {
            const Pack a = *(const Pack*)(y2 + (size_t)t * W + c);
#pragma unroll
            for (int e = 0; e < VEC; ++e) v[p][e] += to_f(a.v[e]);
        }
        if (prod != nullptr)
            for (int k = 0; k < top; ++k) {
                const Pack a = *(const Pack*)(prod + (size_t)pair_row[t * top + k] * W + c);
                const float w = wts ? wts[t * top + k] : 1.f;
#pragma unroll
                for (int e = 0; e < VEC; ++e) v[p][e] += w * to_f(a.v[e]);
            }
        PackF o;
#pragma unroll
        for (int e = 0; e < VEC; ++e) { o.v[e] = v[p][e]; sum += v[p][e]; }
        if (y != nullptr || y2 != nullptr || prod != nullptr) *(PackF*)(xr + c) = o;
    }
    if (h_out == nullptr) return;
    const float mean = block_sum(sum, red) / (float)W;
    float ss = 0.f;
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        if ((int)(threadIdx.x + 256 * p) * VEC >= W) continue;
#pragma unroll
        for (int e = 0; e < VEC; ++e) { v[p][e] -= mean; ss += v[p][e] * v[p][e]; }
    }
    const float r = 1.f / sqrtf(block_sum(ss, red) / (float)W + eps);
#pragma unroll
    for (int p = 0; p < NP; ++p) {
        const int c = (threadIdx.x + 256 * p) * VEC;
        if (c >= W) continue;
        const Pack w = *(const Pack*)(next_w + c);
        Pack o;
#pragma unroll
        for (int e = 0; e < VEC; ++e) o.v[e] = from_f<T>(v[p][e] * r * to_f(w.v[e]));
        *(Pack*)(h_out + (size_t)t * W + c) = o;
    }
}

}  // namespace hm

using namespace hm;

extern "C" int hm_layer_norm_residual(int dtype, float* x, const void* y, const int64_t* ids, const void* y2, const void* prod,
                                      const int32_t* pair_row, const float* wts, int top, const void* next_w, float eps,
                                      void* h_out, int64_t T, int W, void* stream) {
    if (T < 0 || W < 1 || (ids && !y) || (prod && (!pair_row || top < 1)) || (h_out && !next_w) || (T > 0 && !x)) {
        set_error("hm_layer_norm_residual: bad argument");
        return HM_EINVAL;
    }
    if (W > 32 * 1024 || (W % 4 != 0 && W > 16 * 256)) {
        set_error("hm_layer_norm_residual: width %d does not fit the row registers (multiples of 4 up to 32768, others up to 4096)", W);
        return HM_ESHAPE;
    }
    if (T == 0) return HM_OK;
    const uintptr_t bits = (uintptr_t)x | (uintptr_t)y | (uintptr_t)y2 | (uintptr_t)prod | (uintptr_t)next_w | (uintptr_t)h_out;
    const bool wide = W % 4 == 0 && bits % 16 == 0;
    if (!wide && W > 16 * 256) { set_error("hm_layer_norm_residual: unaligned rows of width %d", W); return HM_ESHAPE; }
#define HM_LN(VEC_, NP_)                                                                                                      \
    hipLaunchKernelGGL((layer_norm_residual_kernel<DT, VEC_, NP_>), dim3((unsigned)T), dim3(256), 0, as_stream(stream), x, (const DT*)y, \
                       ids, (const DT*)y2, (const DT*)prod, pair_row, wts, top, (const DT*)next_w, eps, (DT*)h_out, W)
    HM_DISPATCH(dtype, "hm_layer_norm_residual",
                if (!wide) HM_LN(1, 16);
                else if (W <= 1024) HM_LN(4, 1);
                else if (W <= 2048) HM_LN(4, 2);
                else if (W <= 4096) HM_LN(4, 4);
                else if (W <= 8192) HM_LN(4, 8);
                else HM_LN(4, 32));
#undef HM_LN
    HM_CHECK_LAUNCH("hm_layer_norm_residual");
    return HM_OK;
}
