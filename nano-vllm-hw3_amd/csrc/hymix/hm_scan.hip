// Selective scan: a recurrence whose decay, step size, input and output vectors all come from the token.  Per channel c with
// a float32 state S[N]:
//   S_t[n] = exp(dt_c A[c, n]) S_(t-1)[n] + dt_c x_c B[n],   y_c = sum_n S_t[n] C[n] + D_c x_c,   out_c = y_c silu(z_c),
// dt_c = softplus(dt_pre_c + bias_c).  Sequential over a portion's tokens, parallel over sequences, channels and states.
// The state f32 [slots, channels, N] is read at a portion's start (zero at position 0, whatever the slot holds) and left at
// its end.
#include "hm_common.h"

namespace hm {

// sum over L neighbouring lanes (L a power of two); every lane gets the total
template <int L>
__device__ __forceinline__ float group_sum(float v) {
#define HM_DPP_ADD(CTRL) v += __builtin_bit_cast(float, __builtin_amdgcn_update_dpp(0, __builtin_bit_cast(int, v), CTRL, 0xF, 0xF, true))
    if (L >= 2) HM_DPP_ADD(0xB1);              // quad_perm [1,0,3,2]
    if (L >= 4) HM_DPP_ADD(0x4E);              // quad_perm [2,3,0,1]
    if (L >= 8) HM_DPP_ADD(0x141);             // row_half_mirror
    if (L >= 16) HM_DPP_ADD(0x140);            // row_mirror
#undef HM_DPP_ADD
    if (L >= 32) v += __shfl_xor(v, 16);
    if (L >= 64) v += __shfl_xor(v, 32);
    return v;
}

__device__ __forceinline__ float softplus_f(float v) { return fmaxf(v, 0.f) + log1pf(__expf(-fabsf(v))); }

// A workgroup of 256 threads owns 256 / L channels of one sequence; a channel's states are spread over L neighbouring lanes,
// NS in each lane's registers (L * NS >= N; the lanes beyond N hold zeros that meet zero B and C).  CH tokens are staged at
// a time: every (token, channel) is fetched by one thread, which turns it into the pair (dt, dt x) in LDS; B and C of the
// tokens lie beside them.  The next chunk is requested from global memory before the current one runs.  A channel's sum over
// the states replaces its pair in LDS, and the thread that fetched the element adds the skip, applies the gate and stores.
template <typename T, int L, int NS, int CH>
__global__ __launch_bounds__(256) void selective_scan_kernel(const T* __restrict__ x, int64_t x_stride,
                                                             const float* __restrict__ dt_pre, int64_t dt_stride,
                                                             const float* __restrict__ dt_bias, const T* __restrict__ bc,
                                                             int64_t bc_stride, int b_off, int c_off, const float* __restrict__ A,
                                                             const float* __restrict__ D, const T* __restrict__ z,
                                                             int64_t z_stride, float* __restrict__ state,
                                                             const int32_t* __restrict__ qstart,
                                                             const int32_t* __restrict__ seq_pos0,
                                                             const int32_t* __restrict__ seq_slot, T* __restrict__ out,
                                                             int64_t out_stride, int C, int N) {
    constexpr int CPW = 256 / L, NP = L * NS, EL = CH * CPW, NR = (EL + 255) / 256, BC = CH * 2 * NP, NB = (BC + 255) / 256;
    __shared__ __attribute__((aligned(16))) float2 step_lds[EL];            // (dt, dt x); then the sum over the states in .x
    __shared__ __attribute__((aligned(16))) float bc_lds[BC];               // per token B[NP], C[NP]
    const int b = blockIdx.x;
    const int q0 = qstart[b], n = qstart[b + 1] - q0;
    if (n <= 0) return;
    const int tid = threadIdx.x, slice = tid % L, chl = tid / L;
    const int c0 = blockIdx.y * CPW, ch = c0 + chl, n0 = slice * NS;
    float* st = state + ((size_t)seq_slot[b] * C + ch) * N + n0;
    const bool fresh = seq_pos0[b] == 0;
    float s[NS], a2[NS];
#pragma unroll
    for (int i = 0; i < NS; ++i) {
        const bool in = ch < C && n0 + i < N;
        s[i] = in && !fresh ? st[i] : 0.f;
        a2[i] = in ? A[(size_t)ch * N + n0 + i] * 1.4426950408889634f : 0.f;
    }
    // the elements this thread fetches and finishes: token el_t of the chunk, channel el_c
    float el_bias[NR], el_D[NR];
#pragma unroll
    for (int k = 0; k < NR; ++k) {
        const int e = tid + 256 * k, c = c0 + e % CPW;
        el_bias[k] = e < EL && c < C ? dt_bias[c] : 0.f;
        el_D[k] = e < EL && c < C ? D[c] : 0.f;
    }
    T rx[NR], rz[NR], rbc[NB];
    float rdt[NR];
    auto request = [&](int tok0) {
#pragma unroll
        for (int k = 0; k < NR; ++k) {
            const int e = tid + 256 * k, tok = tok0 + e / CPW, c = c0 + e % CPW;
            const bool in = e < EL && tok < n && c < C;
            const size_t row = (size_t)(q0 + tok);
            rx[k] = in ? x[row * x_stride + c] : from_f<T>(0.f);
            rz[k] = in ? z[row * z_stride + c] : from_f<T>(0.f);
            rdt[k] = in ? dt_pre[row * dt_stride + c] : 0.f;
        }
#pragma unroll
        for (int k = 0; k < NB; ++k) {
            const int e = tid + 256 * k, tok = tok0 + e / (2 * NP), r = e % (2 * NP), i = r % NP;
            const bool in = e < BC && tok < n && i < N;
            rbc[k] = in ? bc[(size_t)(q0 + tok) * bc_stride + (r < NP ? b_off : c_off) + i] : from_f<T>(0.f);
        }
    };
    request(0);
    for (int tok0 = 0; tok0 < n; tok0 += CH) {
        float xs[NR], zs[NR];
#pragma unroll
        for (int k = 0; k < NR; ++k) {
            const int e = tid + 256 * k;
            xs[k] = to_f(rx[k]);
            zs[k] = to_f(rz[k]);
            const float dt = softplus_f(rdt[k] + el_bias[k]);
            if (e < EL) step_lds[e] = make_float2(dt, dt * xs[k]);
        }
#pragma unroll
        for (int k = 0; k < NB; ++k) {
            const int e = tid + 256 * k;
            if (e < BC) bc_lds[e] = to_f(rbc[k]);
        }
        __syncthreads();
        if (tok0 + CH < n) request(tok0 + CH);
        auto step = [&](int t) {
            const float2 d = step_lds[t * CPW + chl];
            const float* pb = bc_lds + t * 2 * NP + n0;
            float acc = 0.f;
#pragma unroll
            for (int i = 0; i < NS; ++i) {
                s[i] = __builtin_amdgcn_exp2f(d.x * a2[i]) * s[i] + d.y * pb[i];
                acc += s[i] * pb[NP + i];
            }
            acc = group_sum<L>(acc);
            if (slice == 0) step_lds[t * CPW + chl].x = acc;       // (only this group of lanes reads the pair)
        };
        const int nt = min(CH, n - tok0);
        if (CH > 1 && nt == CH) {
#pragma unroll 4
            for (int t = 0; t < CH; ++t) step(t);
        } else {
            for (int t = 0; t < nt; ++t) step(t);
        }
        __syncthreads();
#pragma unroll
        for (int k = 0; k < NR; ++k) {
            const int e = tid + 256 * k, tok = tok0 + e / CPW, c = c0 + e % CPW;
            if (e < EL && tok < n && c < C) {
                const float y = step_lds[e].x + el_D[k] * xs[k];
                out[(size_t)(q0 + tok) * out_stride + c] = from_f<T>(y * zs[k] / (1.f + __expf(-zs[k])));
            }
        }
        // (the next deposit writes elements that this thread alone has just read; B and C were last read before the barrier)
    }
#pragma unroll
    for (int i = 0; i < NS; ++i)
        if (ch < C && n0 + i < N) st[i] = s[i];
}

template <typename DT>
static void launch_scan(const void* x, int64_t x_stride, const float* dt_pre, int64_t dt_stride, const float* dt_bias, const void* bc,
                        int64_t bc_stride, int b_off, int c_off, const float* A, const float* D, const void* z, int64_t z_stride,
                        float* state, const int32_t* qstart, const int32_t* seq_pos0, const int32_t* seq_slot, void* out,
                        int64_t out_stride, int B, int C, int N, int max_q, hipStream_t s) {
#define HM_SCAN(L, NS, CH)                                                                                                   \
    hipLaunchKernelGGL((selective_scan_kernel<DT, L, NS, CH>), dim3((unsigned)B, (unsigned)((C + 256 / L - 1) / (256 / L))), dim3(256), \
                       0, s, (const DT*)x, x_stride, dt_pre, dt_stride, dt_bias, (const DT*)bc, bc_stride, b_off, c_off, A, D,  \
                       (const DT*)z, z_stride, state, qstart, seq_pos0, seq_slot, (DT*)out, out_stride, C, N)
#define HM_SCAN_T(L, NS) do { if (max_q <= 1) HM_SCAN(L, NS, 1); else HM_SCAN(L, NS, 16); } while (0)
    // states per lane: more of them share a token's fetches and sums, fewer give more lanes to a small batch
    const int64_t states = (int64_t)B * C * N;
    const int ns = N > 8 && N <= 128 && states < 8 * 48 * 1024 ? (N <= 32 && states < 4 * 48 * 1024 ? 2 : 4) : 8;
    if (ns == 2) {
        if (N <= 16) HM_SCAN_T(8, 2); else HM_SCAN_T(16, 2);
    } else if (ns == 4) {
        if (N <= 16) HM_SCAN_T(4, 4); else if (N <= 32) HM_SCAN_T(8, 4); else if (N <= 64) HM_SCAN_T(16, 4); else HM_SCAN_T(32, 4);
    } else if (N <= 8) HM_SCAN_T(1, 8);
    else if (N <= 16) HM_SCAN_T(2, 8);
    else if (N <= 32) HM_SCAN_T(4, 8);
    else if (N <= 64) HM_SCAN_T(8, 8);
    else if (N <= 128) HM_SCAN_T(16, 8);
    else if (N <= 256) HM_SCAN_T(32, 8);
    else HM_SCAN_T(64, 8);
#undef HM_SCAN_T
#undef HM_SCAN
}

}  // namespace hm

using namespace hm;

extern "C" int hm_selective_scan(int dtype, const void* x, int64_t x_stride, const float* dt_pre, int64_t dt_stride,
                                 const float* dt_bias, const void* bc, int64_t bc_stride, int b_off, int c_off, const float* A,
                                 const float* D, const void* z, int64_t z_stride, float* state, const int32_t* qstart,
                                 const int32_t* seq_pos0, const int32_t* seq_slot, void* out, int64_t out_stride, int B, int C,
                                 int N, int max_q, void* stream) {
    if (B < 0 || C < 1 || N < 1 || b_off < 0 || c_off < 0 || x_stride < C || dt_stride < C || z_stride < C || out_stride < C ||
        bc_stride < (int64_t)b_off + N || bc_stride < (int64_t)c_off + N ||
        (B > 0 && (!x || !dt_pre || !dt_bias || !bc || !A || !D || !z || !state || !qstart || !seq_pos0 || !seq_slot || !out))) {
        set_error("hm_selective_scan: bad argument");
        return HM_EINVAL;
    }
    if (N > 512 || C > 4 * 65535) { set_error("hm_selective_scan: at most 512 states per channel"); return HM_ESHAPE; }
    if (B == 0) return HM_OK;
    HM_DISPATCH(dtype, "hm_selective_scan",
                launch_scan<DT>(x, x_stride, dt_pre, dt_stride, dt_bias, bc, bc_stride, b_off, c_off, A, D, z, z_stride, state, qstart,
                                seq_pos0, seq_slot, out, out_stride, B, C, N, max_q, as_stream(stream)));
    HM_CHECK_LAUNCH("hm_selective_scan");
    return HM_OK;
}
