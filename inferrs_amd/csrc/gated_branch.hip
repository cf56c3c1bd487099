// What closes a sub-layer around a 32-bit residual stream x whose sub-layers read x as it stands and whose outputs are
// gated and normed before they enter it:
//     s = y1 (+ sum_k w_k r_k) (+ f y3)                     the sub-layer's output, every addend optional
//     s = s * sigmoid(g + b)                                (optional) a gate a feature
//     x <- x + s / sqrt(mean(s^2) + eps) * w
// and the new x once more in the products' precision (`xr`), which is what the next sub-layer's products read.  A block
// owns a row; every sum, gate and statistic is 32-bit.  y1 and y3 may each be a product still split along its k
// ([splits, n, W], 32-bit); r_k are the rows of routed experts [n, top, W] (32-bit) with weights w_k; f is one 32-bit
// factor a row.  The gate's projection lies in rows of pitch g_ld from column g_off on, its bias in 32-bit.
#include "api.h"
#include "common.h"

#define GB_MAX_TOP 16
#define GB_VEC_ITERS 4

struct BranchArgs {
    float* x;
    const void *y1, *y3;
    int y1_splits, y3_splits;
    long long split_stride;
    const float* y3_scale;
    const float *routed, *routed_w;
    int top;
    const void* gate;
    long long g_ld;
    int g_off;
    const float *gate_b, *norm_w;
    float eps;
    void* xr;
    int W;
};

template <typename T>
__device__ __forceinline__ float gb_sum_splits(const T* p, int splits, long long stride) {
    float t = ld(p);
    for (int s = 1; s < splits; ++s) t += ld(p + s * stride);
    return t;
}

template <typename TY, typename TG, typename TX>
__global__ __launch_bounds__(1024) void branch_step_kernel(const BranchArgs a) {
    extern __shared__ float gb_row[];            // [W]
    __shared__ float scratch[16];
    const int W = a.W, row = blockIdx.x;
    const long long at = (long long)row * W;
    const TY *y1 = (const TY*)a.y1, *y3 = (const TY*)a.y3;
    const TG* gate = a.gate != nullptr ? (const TG*)a.gate + (long long)row * a.g_ld + a.g_off : nullptr;
    const float f3 = y3 != nullptr && a.y3_scale != nullptr ? a.y3_scale[row] : 1.0f;
    float sq = 0.f;
    for (int c = threadIdx.x; c < W; c += blockDim.x) {
        float v = y1 != nullptr ? gb_sum_splits(y1 + at + c, a.y1_splits, a.split_stride) : 0.f;
        for (int k = 0; k < a.top; ++k) v = fmaf(a.routed_w[(long long)row * a.top + k], a.routed[((long long)row * a.top + k) * W + c], v);
        if (y3 != nullptr) v = fmaf(f3, gb_sum_splits(y3 + at + c, a.y3_splits, a.split_stride), v);
        if (gate != nullptr) v /= 1.0f + expf(-(ld(gate + c) + a.gate_b[c]));
        gb_row[c] = v;
        sq = fmaf(v, v, sq);
    }
    const float rs = 1.0f / sqrtf(block_sum(sq, scratch) / (float)W + a.eps);
    for (int c = threadIdx.x; c < W; c += blockDim.x) {          // (a thread reads back the features it wrote)
        const float v = fmaf(gb_row[c] * rs, a.norm_w[c], a.x[at + c]);
        a.x[at + c] = v;
        if (a.xr != nullptr) st((TX*)a.xr + at + c, v);
    }
}

// The same for widths in steps of 8 up to 8 * GB_VEC_ITERS * 1024: a thread owns eight neighbouring features a round (16-
// and 32-byte accesses) and keeps them in registers; every load of a row is asked for before its sum of squares is known.
__device__ __forceinline__ void gb_load8(const float* p, float (&v)[8]) {
    const float4 a = *reinterpret_cast<const float4*>(p), b = *reinterpret_cast<const float4*>(p + 4);
    v[0] = a.x; v[1] = a.y; v[2] = a.z; v[3] = a.w; v[4] = b.x; v[5] = b.y; v[6] = b.z; v[7] = b.w;
}
__device__ __forceinline__ void gb_load8(const bf16_t* p, float (&v)[8]) {
    const uint4 a = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {a.x, a.y, a.z, a.w};
#pragma unroll
    for (int i = 0; i < 4; ++i) {
        v[2 * i] = __uint_as_float(w[i] << 16);
        v[2 * i + 1] = __uint_as_float(w[i] & 0xffff0000u);
    }
}
__device__ __forceinline__ void gb_store8(float* p, const float (&v)[8]) {
    *reinterpret_cast<float4*>(p) = make_float4(v[0], v[1], v[2], v[3]);
    *reinterpret_cast<float4*>(p + 4) = make_float4(v[4], v[5], v[6], v[7]);
}
__device__ __forceinline__ void gb_store8(bf16_t* p, const float (&v)[8]) {
    *reinterpret_cast<uint4*>(p) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]),
                                              pack_bf16x2(v[6], v[7]));
}
template <typename T>
__device__ __forceinline__ void gb_load8_splits(const T* p, int splits, long long stride, float (&t)[8]) {
    gb_load8(p, t);
    for (int s = 1; s < splits; ++s) {
        float u[8];
        gb_load8(p + s * stride, u);
#pragma unroll
        for (int i = 0; i < 8; ++i) t[i] += u[i];
    }
}

template <typename TY, typename TG, typename TX, int ITERS>
__global__ __launch_bounds__(1024) void branch_step_vec_kernel(const BranchArgs a) {
    __shared__ float scratch[16];
    const int W = a.W, row = blockIdx.x;
    const long long at = (long long)row * W;
    const TY *y1 = (const TY*)a.y1, *y3 = (const TY*)a.y3;
    const TG* gate = a.gate != nullptr ? (const TG*)a.gate + (long long)row * a.g_ld + a.g_off : nullptr;
    const float f3 = y3 != nullptr && a.y3_scale != nullptr ? a.y3_scale[row] : 1.0f;
    float v[ITERS][8], xv[ITERS][8], wv[ITERS][8];
    float sq = 0.f;
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
        const int c = (it * blockDim.x + threadIdx.x) * 8;
        if (c >= W) continue;
        float t[8], gt[8], gb[8];
        gb_load8(a.x + at + c, xv[it]);
        gb_load8(a.norm_w + c, wv[it]);
        if (gate != nullptr) {
            gb_load8(gate + c, gt);
            gb_load8(a.gate_b + c, gb);
        }
        if (y1 != nullptr) {
            gb_load8_splits(y1 + at + c, a.y1_splits, a.split_stride, v[it]);
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) v[it][i] = 0.f;
        }
#pragma unroll 4
        for (int k = 0; k < a.top; ++k) {
            const float wk = a.routed_w[(long long)row * a.top + k];
            gb_load8(a.routed + ((long long)row * a.top + k) * W + c, t);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[it][i] = fmaf(wk, t[i], v[it][i]);
        }
        if (y3 != nullptr) {
            gb_load8_splits(y3 + at + c, a.y3_splits, a.split_stride, t);
#pragma unroll
            for (int i = 0; i < 8; ++i) v[it][i] = fmaf(f3, t[i], v[it][i]);
        }
        if (gate != nullptr) {
#pragma unroll
            for (int i = 0; i < 8; ++i) v[it][i] /= 1.0f + expf(-(gt[i] + gb[i]));
        }
#pragma unroll
        for (int i = 0; i < 8; ++i) sq = fmaf(v[it][i], v[it][i], sq);
    }
    const float rs = 1.0f / sqrtf(block_sum(sq, scratch) / (float)W + a.eps);
#pragma unroll
    for (int it = 0; it < ITERS; ++it) {
        const int c = (it * blockDim.x + threadIdx.x) * 8;
        if (c >= W) continue;
#pragma unroll
        for (int i = 0; i < 8; ++i) v[it][i] = fmaf(v[it][i] * rs, wv[it][i], xv[it][i]);
        gb_store8(a.x + at + c, v[it]);
        if (a.xr != nullptr) gb_store8((TX*)a.xr + at + c, v[it]);
    }
}

// y_dtype: precision of y1 and y3; g_dtype: of the gate's rows; x_dtype: of xr.  0 float32, 1 bfloat16.
extern "C" int ia_branch_step(float* x, const void* y1, const void* y3, int y1_splits, int y3_splits, const float* y3_scale,
                              const float* routed, const float* routed_w, int top, const void* gate, long long g_ld, int g_off,
                              const float* gate_b, const float* norm_w, float eps, void* xr, int n, int W, int y_dtype,
                              int g_dtype, int x_dtype, hipStream_t stream) {
    IA_CHECK(n >= 0 && W > 0 && x != nullptr && norm_w != nullptr, "branch_step: n=%d width=%d, the stream and the norm's weight", n, W);
    IA_CHECK((size_t)W * sizeof(float) <= 60 * 1024, "branch_step: width %d does not fit shared memory", W);
    IA_CHECK(y1 != nullptr || routed != nullptr || y3 != nullptr, "branch_step: nothing to add");
    IA_CHECK(routed == nullptr ? top == 0 : (top >= 1 && top <= GB_MAX_TOP && routed_w != nullptr),
             "branch_step: 1 to %d routed rows a row with their weights (top=%d)", GB_MAX_TOP, top);
    IA_CHECK(gate == nullptr || (gate_b != nullptr && g_off >= 0 && g_off + W <= g_ld), "branch_step: a gate of %d features at %d of rows of %lld",
             W, g_off, g_ld);
    IA_CHECK(y1_splits >= 1 && y3_splits >= 1 && ((y1_splits == 1 && y3_splits == 1) || y_dtype == IA_F32),
             "branch_step: outputs in %d and %d splits are 32-bit", y1_splits, y3_splits);
    IA_CHECK((y_dtype == IA_F32 || y_dtype == IA_BF16) && (g_dtype == IA_F32 || g_dtype == IA_BF16) &&
             (x_dtype == IA_F32 || x_dtype == IA_BF16), "branch_step: unknown dtype");
    if (n == 0) return 0;
    BranchArgs a;
    a.x = x; a.y1 = y1; a.y3 = y3; a.y1_splits = y1_splits; a.y3_splits = y3_splits; a.split_stride = (long long)n * W;
    a.y3_scale = y3_scale; a.routed = routed; a.routed_w = routed_w; a.top = top; a.gate = gate; a.g_ld = g_ld; a.g_off = g_off;
    a.gate_b = gate_b; a.norm_w = norm_w; a.eps = eps; a.xr = xr; a.W = W;
    const uintptr_t ptrs = (uintptr_t)x | (uintptr_t)y1 | (uintptr_t)y3 | (uintptr_t)routed | (uintptr_t)gate | (uintptr_t)gate_b |
                           (uintptr_t)norm_w | (uintptr_t)xr;
#define GB_TYPES_X(CALL, TX)                                                    \
    do {                                                                        \
        if (y_dtype == IA_F32 && g_dtype == IA_F32) { CALL(float, float, TX); } \
        else if (y_dtype == IA_F32) { CALL(float, bf16_t, TX); }                \
        else if (g_dtype == IA_F32) { CALL(bf16_t, float, TX); }                \
        else { CALL(bf16_t, bf16_t, TX); }                                      \
    } while (0)
#define GB_TYPES(CALL)                                                          \
    do {                                                                        \
        if (x_dtype == IA_F32) GB_TYPES_X(CALL, float);                         \
        else GB_TYPES_X(CALL, bf16_t);                                          \
    } while (0)
    const int g_per = g_dtype == IA_F32 ? 4 : 8;
    if (W % 8 == 0 && (gate == nullptr || (g_ld % g_per == 0 && g_off % g_per == 0)) && (ptrs & 15) == 0 && W <= 8 * GB_VEC_ITERS * 1024) {
        // a piece of eight a thread up to 512 threads, then more rounds
        const int pieces = W / 8;
#define GB_VEC1(TY, TG, TX) branch_step_vec_kernel<TY, TG, TX, 1><<<n, (pieces + 63) / 64 * 64, 0, stream>>>(a)
#define GB_VEC2(TY, TG, TX) branch_step_vec_kernel<TY, TG, TX, 2><<<n, (pieces + 127) / 128 * 64, 0, stream>>>(a)
#define GB_VEC4(TY, TG, TX) branch_step_vec_kernel<TY, TG, TX, 4><<<n, (pieces + 255) / 256 * 64, 0, stream>>>(a)
        if (pieces <= 512) GB_TYPES(GB_VEC1);
        else if (pieces <= 1024) GB_TYPES(GB_VEC2);
        else GB_TYPES(GB_VEC4);
#undef GB_VEC1
#undef GB_VEC2
#undef GB_VEC4
        IA_LAUNCH_CHECK("branch_step");
        return 0;
    }
    const int threads = W >= 4096 ? 1024 : W >= 1024 ? 512 : W >= 512 ? 256 : 128;
    const size_t shm = (size_t)W * sizeof(float);
#define GB_PLAIN(TY, TG, TX) branch_step_kernel<TY, TG, TX><<<n, threads, shm, stream>>>(a)
    GB_TYPES(GB_PLAIN);
#undef GB_PLAIN
#undef GB_TYPES
#undef GB_TYPES_X
    IA_LAUNCH_CHECK("branch_step");
    return 0;
}
