// Per-head RMS norm of queries and keys, rotary position encoding, and the write of the new
// keys and values into their cache pages, in one pass over the projection output.
//
// Order as in the reference: norm per head over head_dim with one shared weight vector
// (inferrs-models/src/models/qwen3.rs:128-129, attention_utils.rs:52-58), then rotation
// (qwen3.rs:132-135) with out[i] = x[i]c - x[j]s, out[j] = x[i]s + x[j]c
// (inferrs-kernels/candle-kernels/src/reduce.cu:292-312 for j = i + rot/2, :275-289 for the
// interleaved pairing), then the cache append (qwen3.rs:145-161).  Values are copied as they are.
// Norm, angles and rotation stay in 32-bit registers; one rounding happens at the store.
#include "common.h"
#include "api.h"

#define QK_MAX_HEAD_DIM 512
#define QK_WAVES 4

// One wave per (token, head).  Heads 0..nq are queries, nq..nq+nkv keys, the rest values.
template <typename T>
__global__ __launch_bounds__(QK_WAVES * IA_WAVE) void qk_rope_kv_kernel(
    T* __restrict__ q_out,              // [n, nq, d]
    T* __restrict__ k_cache,            // [pages, nkv, page_size, d] or null
    T* __restrict__ v_cache,            // [pages, nkv, d, page_size] or null
    const T* __restrict__ qkv,          // [n, (nq + 2 nkv) d]
    const float* __restrict__ q_norm_w, // [d] or null
    const float* __restrict__ k_norm_w, // [d] or null
    const float* __restrict__ cos_t,    // [n, rot/2] or null
    const float* __restrict__ sin_t,
    const int* __restrict__ slots,      // [n] page * page_size + offset, or null (no write)
    int n, int nq, int nkv, int d, int rot, int interleaved, int page_size, float eps, int add_one) {
    __shared__ float buf[QK_WAVES][QK_MAX_HEAD_DIM];
    const int lane = threadIdx.x & (IA_WAVE - 1);
    const int wave = threadIdx.x / IA_WAVE;
    const int heads = slots ? nq + 2 * nkv : nq;
    const long long unit = (long long)blockIdx.x * QK_WAVES + wave;
    const bool active = unit < (long long)n * heads;
    const int tok = active ? (int)(unit / heads) : 0;
    const int hh = active ? (int)(unit % heads) : 0;
    const int kind = hh < nq ? 0 : (hh < nq + nkv ? 1 : 2);
    const T* src = qkv + ((size_t)tok * (nq + 2 * nkv) + hh) * d;
    float* row = buf[wave];

    float ss = 0.f;
    if (active) {
        for (int j = lane; j < d; j += IA_WAVE) {
            const float v = ld(src + j);
            row[j] = v;
            ss += v * v;
        }
    }
    const float* nw = kind == 0 ? q_norm_w : (kind == 1 ? k_norm_w : nullptr);
    if (nw != nullptr) {
        ss = wave_sum(ss);
        const float scale = 1.0f / sqrtf(ss / (float)d + eps);
        if (active)
            for (int j = lane; j < d; j += IA_WAVE) row[j] = scale * row[j] * (add_one ? 1.0f + nw[j] : nw[j]);
    }
    __syncthreads();
    if (!active) return;

    T* dst;
    if (kind == 0) {
        dst = q_out + ((size_t)tok * nq + hh) * d;
    } else {
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        if (kind == 2) {
            // values are kept transposed inside a page: [dim][slot]
            T* vt = v_cache + ((size_t)page * nkv + (hh - nq - nkv)) * d * page_size + off;
            for (int j = lane; j < d; j += IA_WAVE) st(vt + (size_t)j * page_size, row[j]);
            return;
        }
        dst = k_cache + (((size_t)page * nkv + (hh - nq)) * page_size + off) * d;
    }
    if (cos_t == nullptr) {
        for (int j = lane; j < d; j += IA_WAVE) st(dst + j, row[j]);
        return;
    }
    const int half = rot / 2;
    for (int i = lane; i < half; i += IA_WAVE) {
        const float c = cos_t[(size_t)tok * half + i], s = sin_t[(size_t)tok * half + i];
        const int ia = interleaved ? 2 * i : i;
        const int ib = interleaved ? 2 * i + 1 : i + half;
        const float a = row[ia], b = row[ib];
        st(dst + ia, a * c - b * s);
        st(dst + ib, a * s + b * c);
    }
    for (int j = rot + lane; j < d; j += IA_WAVE) st(dst + j, row[j]);
}

// A value mixed with another layer's value of the same token.
__device__ __forceinline__ float mixed_value(float v, float with, float mix) { return fmaf(mix, with, (1.0f - mix) * v); }

// The same work on rows of any layout: the projections' output holds a token's query heads from `q_off`, its key heads
// from `k_off` and its value heads (each `dv` wide, which need not be the keys' width) from `v_off`, `ld` elements a
// row; whatever else the row holds (a gate, say) is left alone.  `k_off` < 0 or no slots: the layer writes no cache
// (it reads another layer's), and only the queries are formed.  `v_with` (rows `vw_ld` apart, value heads side by side):
// a value becomes (1 - v_mix) v + v_mix v_with on its way to the cache.  One wave per (token, head).
template <typename T>
__global__ __launch_bounds__(QK_WAVES * IA_WAVE) void qk_rope_kv_strided_kernel(
    T* __restrict__ q_out,              // [n, nq, d]
    T* __restrict__ k_cache,            // [pages, nkv, page_size, d] or null
    T* __restrict__ v_cache,            // [pages, nkv, dv, page_size] or null
    const T* __restrict__ proj,         // [n, ld]
    const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, const int* __restrict__ slots,
    int n, int ld_, int q_off, int k_off, int v_off, int nq, int nkv, int d, int dv, int rot, int interleaved,
    int page_size, float eps, int add_one, const T* __restrict__ v_with, long long vw_ld, float v_mix) {
    __shared__ float buf[QK_WAVES][QK_MAX_HEAD_DIM];
    const int lane = threadIdx.x & (IA_WAVE - 1);
    const int wave = threadIdx.x / IA_WAVE;
    const int heads = slots ? nq + 2 * nkv : nq;
    const long long unit = (long long)blockIdx.x * QK_WAVES + wave;
    const bool active = unit < (long long)n * heads;
    const int tok = active ? (int)(unit / heads) : 0;
    const int hh = active ? (int)(unit % heads) : 0;
    const int kind = hh < nq ? 0 : (hh < nq + nkv ? 1 : 2);
    const int width = kind == 2 ? dv : d;
    const T* src = proj + (size_t)tok * ld_ +
                   (kind == 0 ? q_off + hh * d : kind == 1 ? k_off + (hh - nq) * d : v_off + (hh - nq - nkv) * dv);
    float* row = buf[wave];

    float ss = 0.f;
    if (active) {
        for (int j = lane; j < width; j += IA_WAVE) {
            float v = ld(src + j);
            if (kind == 2 && v_with != nullptr) v = mixed_value(v, ld(v_with + (size_t)tok * vw_ld + (hh - nq - nkv) * dv + j), v_mix);
            row[j] = v;
            ss += v * v;
        }
    }
    const float* nw = kind == 0 ? q_norm_w : (kind == 1 ? k_norm_w : nullptr);
    if (nw != nullptr) {
        ss = wave_sum(ss);
        const float scale = 1.0f / sqrtf(ss / (float)d + eps);
        if (active)
            for (int j = lane; j < d; j += IA_WAVE) row[j] = scale * row[j] * (add_one ? 1.0f + nw[j] : nw[j]);
    }
    __syncthreads();
    if (!active) return;

    T* dst;
    if (kind == 0) {
        dst = q_out + ((size_t)tok * nq + hh) * d;
    } else {
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        if (kind == 2) {
            // values are kept transposed inside a page: [dim][slot]
            T* vt = v_cache + ((size_t)page * nkv + (hh - nq - nkv)) * dv * page_size + off;
            for (int j = lane; j < dv; j += IA_WAVE) st(vt + (size_t)j * page_size, row[j]);
            return;
        }
        dst = k_cache + (((size_t)page * nkv + (hh - nq)) * page_size + off) * d;
    }
    if (cos_t == nullptr) {
        for (int j = lane; j < d; j += IA_WAVE) st(dst + j, row[j]);
        return;
    }
    const int half = rot / 2;
    for (int i = lane; i < half; i += IA_WAVE) {
        const float c = cos_t[(size_t)tok * half + i], s = sin_t[(size_t)tok * half + i];
        const int ia = interleaved ? 2 * i : i;
        const int ib = interleaved ? 2 * i + 1 : i + half;
        const float a = row[ia], b = row[ib];
        st(dst + ia, a * c - b * s);
        st(dst + ib, a * s + b * c);
    }
    for (int j = rot + lane; j < d; j += IA_WAVE) st(dst + j, row[j]);
}

// The same with 16-byte accesses, for bfloat16 rows whose head sizes, pitch and offsets are multiples of 8: a thread owns
// eight neighbouring features of one (token, head); the threads of a head meet in shared memory for the sum of squares
// (added up in the order of the features) and for their rotation partners.  The blocks from `qk_blocks` on take the
// values, eight features of a (token, key/value head) a thread, which go to their page slot by slot.
#define QKS_THREADS 256
__global__ __launch_bounds__(QKS_THREADS) void qk_rope_kv_strided_bf16_vec_kernel(
    bf16_t* __restrict__ q_out, bf16_t* __restrict__ k_cache, bf16_t* __restrict__ v_cache, const bf16_t* __restrict__ proj,
    const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w, const float* __restrict__ cos_t,
    const float* __restrict__ sin_t, const int* __restrict__ slots, int n, int ld_, int q_off, int k_off, int v_off, int nq,
    int nkv, int d, int dv, int rot, int interleaved, int page_size, float eps, int add_one, int qk_blocks,
    const bf16_t* __restrict__ v_with, long long vw_ld, float v_mix) {
    __shared__ float rows[QKS_THREADS * 8];          // normalised features, unit after unit
    __shared__ float partial[QKS_THREADS];
    if ((int)blockIdx.x >= qk_blocks) {
        const int tpu = dv / 8, upb = QKS_THREADS / tpu;
        const int u = threadIdx.x / tpu, t = threadIdx.x - u * tpu;
        const long long unit = (long long)((int)blockIdx.x - qk_blocks) * upb + u;
        if (u >= upb || unit >= (long long)n * nkv) return;
        const int tok = (int)(unit / nkv), hh = (int)(unit % nkv);
        uint4 v = *(const uint4*)(proj + (size_t)tok * ld_ + v_off + hh * dv + t * 8);
        if (v_with != nullptr) {
            const uint4 f = *(const uint4*)(v_with + (size_t)tok * vw_ld + hh * dv + t * 8);
            auto both = [&](uint32_t a, uint32_t b) {
                return pack_bf16x2(mixed_value(__uint_as_float(a << 16), __uint_as_float(b << 16), v_mix),
                                   mixed_value(__uint_as_float(a & 0xffff0000u), __uint_as_float(b & 0xffff0000u), v_mix));
            };
            v = make_uint4(both(v.x, f.x), both(v.y, f.y), both(v.z, f.z), both(v.w, f.w));
        }
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        bf16_t* dst = v_cache + (((size_t)page * nkv + hh) * dv + t * 8) * page_size + off;
        const uint32_t w[4] = {v.x, v.y, v.z, v.w};
#pragma unroll
        for (int j = 0; j < 8; ++j) dst[(size_t)j * page_size].bits = (uint16_t)(j & 1 ? w[j >> 1] >> 16 : w[j >> 1] & 0xffffu);
        return;
    }
    const int tpu = d / 8, upb = QKS_THREADS / tpu;
    const int u = threadIdx.x / tpu, t = threadIdx.x - u * tpu;
    const int heads = slots ? nq + nkv : nq;
    const long long unit = (long long)blockIdx.x * upb + u;
    const bool active = u < upb && unit < (long long)n * heads;
    const int tok = active ? (int)(unit / heads) : 0;
    const int hh = active ? (int)(unit % heads) : 0;
    const bool is_q = hh < nq;
    const float* nw = is_q ? q_norm_w : k_norm_w;
    float v[8];
    float ss = 0.f;
    if (active) {
        const uint4 raw = *(const uint4*)(proj + (size_t)tok * ld_ + (is_q ? q_off + hh * d : k_off + (hh - nq) * d) + t * 8);
        const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            v[2 * j] = __uint_as_float(w[j] << 16);
            v[2 * j + 1] = __uint_as_float(w[j] & 0xffff0000u);
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) ss = fmaf(v[j], v[j], ss);
    } else {
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = 0.f;
    }
    if (q_norm_w != nullptr || k_norm_w != nullptr) {                    // (the same for all threads: they meet at the barrier)
        partial[threadIdx.x] = ss;
        __syncthreads();
        float total = 0.f;
        if (active)
            for (int j = 0; j < tpu; ++j) total += partial[u * tpu + j];
        const float scale = 1.0f / sqrtf(total / (float)d + eps);
        if (active && nw != nullptr) {
            const float4 g0 = *(const float4*)(nw + t * 8), g1 = *(const float4*)(nw + t * 8 + 4);
            const float g[8] = {g0.x, g0.y, g0.z, g0.w, g1.x, g1.y, g1.z, g1.w};
#pragma unroll
            for (int j = 0; j < 8; ++j) v[j] = scale * v[j] * (add_one ? 1.0f + g[j] : g[j]);
        }
    }
    const bool rotates = cos_t != nullptr && t * 8 < rot;               // (the same for all threads up to the barrier below)
    if (cos_t != nullptr) {
#pragma unroll
        for (int j = 0; j < 8; ++j) rows[threadIdx.x * 8 + j] = v[j];
        __syncthreads();
    }
    if (!active) return;
    float o[8];
    const int half = rot / 2;
    const float* mine = rows + (size_t)u * tpu * 8;
#pragma unroll
    for (int j = 0; j < 8; ++j) {
        const int e = t * 8 + j;
        o[j] = v[j];
        if (rotates && e < rot) {
            const bool first = interleaved ? (e & 1) == 0 : e < half;
            const int i = interleaved ? e >> 1 : (first ? e : e - half);
            const int other = interleaved ? e ^ 1 : (first ? e + half : e - half);
            const float c = cos_t[(size_t)tok * half + i], sn = sin_t[(size_t)tok * half + i];
            const float partner = mine[other];
            o[j] = first ? v[j] * c - partner * sn : partner * sn + v[j] * c;
        }
    }
    bf16_t* dst;
    if (is_q) {
        dst = q_out + ((size_t)tok * nq + hh) * d + t * 8;
    } else {
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        dst = k_cache + (((size_t)page * nkv + (hh - nq)) * page_size + off) * d + t * 8;
    }
    *(uint4*)dst = make_uint4(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]), pack_bf16x2(o[4], o[5]), pack_bf16x2(o[6], o[7]));
}

extern "C" int ia_qk_rope_kv_strided(void* q_out, void* k_cache, void* v_cache, const void* proj, const float* q_norm_w,
                                     const float* k_norm_w, const float* cos_t, const float* sin_t, const int* slots, int n,
                                     int ld_, int q_off, int k_off, int v_off, int nq, int nkv, int d, int dv, int rot,
                                     int interleaved, int page_size, float eps, int add_one, const void* v_with,
                                     long long vw_ld, float v_mix, int dtype, hipStream_t stream) {
    IA_CHECK(v_with == nullptr || vw_ld >= (long long)nkv * dv, "qk_rope_kv_strided: values to mix with, rows %lld apart, of %d x %d", vw_ld, nkv, dv);
    IA_CHECK(n >= 0 && nq > 0 && nkv > 0, "qk_rope_kv_strided: bad sizes n=%d nq=%d nkv=%d", n, nq, nkv);
    IA_CHECK(d > 0 && d <= QK_MAX_HEAD_DIM && dv > 0 && dv <= QK_MAX_HEAD_DIM,
             "qk_rope_kv_strided: head sizes %d / %d are outside 1..%d", d, dv, QK_MAX_HEAD_DIM);
    IA_CHECK(rot >= 0 && rot <= d && rot % 2 == 0, "qk_rope_kv_strided: rot_dim %d must be even and <= head_dim %d", rot, d);
    IA_CHECK((cos_t == nullptr) == (sin_t == nullptr), "qk_rope_kv_strided: cos and sin tables must come together");
    IA_CHECK(cos_t == nullptr || rot > 0, "qk_rope_kv_strided: a rotary table needs rot_dim > 0");
    IA_CHECK(q_off >= 0 && q_off + nq * d <= ld_, "qk_rope_kv_strided: the queries at %d do not fit rows of %d", q_off, ld_);
    if (k_off < 0) slots = nullptr;
    IA_CHECK(slots == nullptr || (k_cache && v_cache && page_size > 0 && v_off >= 0 && k_off + nkv * d <= ld_ && v_off + nkv * dv <= ld_),
             "qk_rope_kv_strided: keys at %d and values at %d need a cache and room in rows of %d", k_off, v_off, ld_);
    if (n == 0) return 0;
    const long long units = (long long)n * (slots ? nq + 2 * nkv : nq);
    const unsigned grid = (unsigned)((units + QK_WAVES - 1) / QK_WAVES);
    const uintptr_t ptrs = (uintptr_t)q_out | (uintptr_t)proj | (uintptr_t)(slots ? k_cache : nullptr) | (uintptr_t)q_norm_w |
                           (uintptr_t)k_norm_w | (uintptr_t)v_with;
    if (dtype == IA_BF16 && d % 8 == 0 && dv % 8 == 0 && d / 8 <= QKS_THREADS && dv / 8 <= QKS_THREADS && ld_ % 8 == 0 &&
        q_off % 8 == 0 && (slots == nullptr || (k_off % 8 == 0 && v_off % 8 == 0)) && (v_with == nullptr || vw_ld % 8 == 0) && (ptrs & 15) == 0) {
        const long long qk_units = (long long)n * (slots ? nq + nkv : nq);
        const int upb = QKS_THREADS / (d / 8), upb_v = QKS_THREADS / (dv / 8);
        const long long qk_blocks = (qk_units + upb - 1) / upb;
        const long long v_blocks = slots ? ((long long)n * nkv + upb_v - 1) / upb_v : 0;
        IA_CHECK(qk_blocks + v_blocks < (1ll << 31), "qk_rope_kv_strided: %d tokens are too many for one launch", n);
        qk_rope_kv_strided_bf16_vec_kernel<<<(unsigned)(qk_blocks + v_blocks), QKS_THREADS, 0, stream>>>(
            (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, (const bf16_t*)proj, q_norm_w, k_norm_w, cos_t, sin_t, slots, n,
            ld_, q_off, k_off, v_off, nq, nkv, d, dv, rot, interleaved, page_size, eps, add_one, (int)qk_blocks, (const bf16_t*)v_with, vw_ld,
            v_mix);
        IA_LAUNCH_CHECK("qk_rope_kv_strided");
        return 0;
    }
    if (dtype == IA_F32)
        qk_rope_kv_strided_kernel<float><<<grid, QK_WAVES * IA_WAVE, 0, stream>>>(
            (float*)q_out, (float*)k_cache, (float*)v_cache, (const float*)proj, q_norm_w, k_norm_w, cos_t, sin_t, slots, n,
            ld_, q_off, k_off, v_off, nq, nkv, d, dv, rot, interleaved, page_size, eps, add_one, (const float*)v_with, vw_ld, v_mix);
    else if (dtype == IA_BF16)
        qk_rope_kv_strided_kernel<bf16_t><<<grid, QK_WAVES * IA_WAVE, 0, stream>>>(
            (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, (const bf16_t*)proj, q_norm_w, k_norm_w, cos_t, sin_t, slots,
            n, ld_, q_off, k_off, v_off, nq, nkv, d, dv, rot, interleaved, page_size, eps, add_one, (const bf16_t*)v_with, vw_ld, v_mix);
    else
        IA_CHECK(false, "qk_rope_kv_strided: unknown dtype %d", dtype);
    IA_LAUNCH_CHECK("qk_rope_kv_strided");
    return 0;
}

#define QKV_THREADS 256
#define QKV_GROUP 8

// The values of eight neighbouring tokens, for as many heads as the block's threads cover (see below).
__device__ __forceinline__ void values_in_groups(uint16_t* tile /* [head of the block][token of the group][d] */,
                                                 bf16_t* __restrict__ v_cache, const bf16_t* __restrict__ qkv,
                                                 const int* __restrict__ slots, int vb, int n, int nq, int nkv,
                                                 int d, int page_size) {
    const int tpu = d / 8;
    const int units_per_block = QKV_THREADS / tpu;
    const int u = threadIdx.x / tpu, t = threadIdx.x - u * tpu;
    const int hpb = units_per_block / QKV_GROUP;      // heads a block
    const int head_groups = (nkv + hpb - 1) / hpb;
    const int tok0 = vb / head_groups * QKV_GROUP, head0 = vb % head_groups * hpb;
    if (u < hpb * QKV_GROUP) {
        const int hl = u / QKV_GROUP, ti = u - hl * QKV_GROUP;
        if (tok0 + ti < n && head0 + hl < nkv)
            *(uint4*)(tile + (size_t)u * d + t * 8) =
                *(const uint4*)(qkv + ((size_t)(tok0 + ti) * (nq + 2 * nkv) + nq + nkv + head0 + hl) * d + t * 8);
    }
    int slot[QKV_GROUP];
    bool together = tok0 + QKV_GROUP <= n;
#pragma unroll
    for (int i = 0; i < QKV_GROUP; ++i) {
        slot[i] = tok0 + i < n ? slots[tok0 + i] : -1;
        together = together && slot[i] == slot[0] + i;
    }
    together = together && slot[0] % QKV_GROUP == 0 && page_size % QKV_GROUP == 0;
    __syncthreads();
    for (int p = threadIdx.x; p < hpb * d; p += QKV_THREADS) {
        const int hl = p / d, j = p - hl * d;
        if (head0 + hl >= nkv) continue;
        const uint16_t* col = tile + (size_t)hl * QKV_GROUP * d + j;
        bf16_t* feature = v_cache + ((size_t)(head0 + hl) * d + j) * page_size;   // + page * nkv * d * page_size
        if (together) {
            const int page = slot[0] / page_size, off = slot[0] - page * page_size;
            uint32_t w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) w[i] = (uint32_t)col[(2 * i) * d] | ((uint32_t)col[(2 * i + 1) * d] << 16);
            *(uint4*)(feature + (size_t)page * nkv * d * page_size + off) = make_uint4(w[0], w[1], w[2], w[3]);
        } else {
#pragma unroll
            for (int i = 0; i < QKV_GROUP; ++i) {
                if (slot[i] < 0) continue;
                const int page = slot[i] / page_size, off = slot[i] - page * page_size;
                feature[(size_t)page * nkv * d * page_size + off].bits = col[i * d];
            }
        }
    }
}

// The same work with 16-byte accesses, for bfloat16 and head sizes that are a multiple of 8:
// a thread owns eight neighbouring features of one (token, head); the threads of a head meet in
// shared memory for the sum of squares and for their rotation partners.
//
// Values lie transposed inside a page ([dim][slot]): written token by token, every feature is a
// store of two bytes of its own.  With `v_from` >= 0 the blocks from that index on write the values
// instead, eight tokens at a time: a block turns the rows of eight neighbouring tokens (of as many
// heads as its threads cover) round in shared memory, and where the eight tokens' slots are
// neighbours in one page, starting at a multiple of eight, a thread stores a feature's eight
// slots as 16 bytes.  Other groups (a page's edge inside, a sequence's end, the last tokens of the
// batch) are stored slot by slot.  The other blocks then leave the values alone.
__global__ __launch_bounds__(QKV_THREADS) void qk_rope_kv_bf16_vec_kernel(
    bf16_t* __restrict__ q_out, bf16_t* __restrict__ k_cache, bf16_t* __restrict__ v_cache,
    const bf16_t* __restrict__ qkv, const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, const int* __restrict__ slots,
    int n, int nq, int nkv, int d, int rot, int interleaved, int page_size, float eps, int add_one, int v_from) {
    __shared__ float rows[QKV_THREADS * 8];          // normalised features, unit after unit
    __shared__ float partial[QKV_THREADS];
    const int tpu = d / 8;                            // threads a (token, head) unit
    const int units_per_block = QKV_THREADS / tpu;
    const int u = threadIdx.x / tpu, t = threadIdx.x - u * tpu;
    if (v_from >= 0 && (int)blockIdx.x >= v_from) {
        values_in_groups((uint16_t*)rows, v_cache, qkv, slots, (int)blockIdx.x - v_from, n, nq, nkv, d, page_size);
        return;
    }
    const int heads = slots ? (v_from >= 0 ? nq + nkv : nq + 2 * nkv) : nq;
    const long long unit = (long long)blockIdx.x * units_per_block + u;
    const bool active = u < units_per_block && unit < (long long)n * heads;
    const int tok = active ? (int)(unit / heads) : 0;
    const int hh = active ? (int)(unit % heads) : 0;
    const int kind = hh < nq ? 0 : (hh < nq + nkv ? 1 : 2);
    // Everything that does not depend on the features is asked for before the first barrier, in
    // 16-byte pieces: norm weights, and the angles when a thread's eight features lie on one
    // side of the rotation's halves (else they are read one by one further down).
    const float* nw = kind == 0 ? q_norm_w : (kind == 1 ? k_norm_w : nullptr);
    const int half = rot / 2;
    const bool vec_angles = interleaved ? rot % 8 == 0 : half % 8 == 0;
    const bool rotates = active && cos_t != nullptr && kind != 2 && t * 8 < rot;
    float gw[8], cs[8], sn[8];
    if (active && nw != nullptr) {
        const float4 g0 = *(const float4*)(nw + t * 8), g1 = *(const float4*)(nw + t * 8 + 4);
        gw[0] = g0.x; gw[1] = g0.y; gw[2] = g0.z; gw[3] = g0.w; gw[4] = g1.x; gw[5] = g1.y; gw[6] = g1.z; gw[7] = g1.w;
    }
    if (rotates && vec_angles) {
        if (interleaved) {
            const size_t at = (size_t)tok * half + t * 4;
            const float4 c0 = *(const float4*)(cos_t + at), s0 = *(const float4*)(sin_t + at);
            cs[0] = cs[1] = c0.x; cs[2] = cs[3] = c0.y; cs[4] = cs[5] = c0.z; cs[6] = cs[7] = c0.w;
            sn[0] = sn[1] = s0.x; sn[2] = sn[3] = s0.y; sn[4] = sn[5] = s0.z; sn[6] = sn[7] = s0.w;
        } else {
            const int e0 = t * 8;
            const size_t at = (size_t)tok * half + (e0 < half ? e0 : e0 - half);
            const float4 c0 = *(const float4*)(cos_t + at), c1 = *(const float4*)(cos_t + at + 4);
            const float4 s0 = *(const float4*)(sin_t + at), s1 = *(const float4*)(sin_t + at + 4);
            cs[0] = c0.x; cs[1] = c0.y; cs[2] = c0.z; cs[3] = c0.w; cs[4] = c1.x; cs[5] = c1.y; cs[6] = c1.z; cs[7] = c1.w;
            sn[0] = s0.x; sn[1] = s0.y; sn[2] = s0.z; sn[3] = s0.w; sn[4] = s1.x; sn[5] = s1.y; sn[6] = s1.z; sn[7] = s1.w;
        }
    }
    float v[8];
    float ss = 0.f;
    if (active) {
        const uint4 raw = *(const uint4*)(qkv + ((size_t)tok * (nq + 2 * nkv) + hh) * d + t * 8);
        const uint32_t w[4] = {raw.x, raw.y, raw.z, raw.w};
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            v[2 * j] = __uint_as_float(w[j] << 16);
            v[2 * j + 1] = __uint_as_float(w[j] & 0xffff0000u);
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) ss += v[j] * v[j];
    }
    partial[threadIdx.x] = ss;
    __syncthreads();
    if (active && nw != nullptr) {
        float total = 0.f;
        for (int i = 0; i < tpu; ++i) total += partial[u * tpu + i];      // the same order in every thread
        const float scale = 1.0f / sqrtf(total / (float)d + eps);
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = scale * v[j] * (add_one ? 1.0f + gw[j] : gw[j]);
    }
    if (active) {
#pragma unroll
        for (int j = 0; j < 8; ++j) rows[threadIdx.x * 8 + j] = v[j];
    }
    __syncthreads();
    if (!active) return;
    if (kind == 2) {
        // values are kept transposed inside a page: [dim][slot]
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        bf16_t* vt = v_cache + ((size_t)page * nkv + (hh - nq - nkv)) * d * page_size + off;
#pragma unroll
        for (int j = 0; j < 8; ++j) st(vt + (size_t)(t * 8 + j) * page_size, v[j]);
        return;
    }
    if (cos_t != nullptr) {
        const float* row = rows + (size_t)u * tpu * 8;
        float o[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int e = t * 8 + j;
            o[j] = v[j];
            if (e < rot) {
                const int i = interleaved ? e >> 1 : (e < half ? e : e - half);
                const bool first = interleaved ? (e & 1) == 0 : e < half;
                const int partner = interleaved ? e ^ 1 : (first ? e + half : e - half);
                const float c = vec_angles ? cs[j] : cos_t[(size_t)tok * half + i];
                const float s = vec_angles ? sn[j] : sin_t[(size_t)tok * half + i];
                o[j] = first ? v[j] * c - row[partner] * s : row[partner] * s + v[j] * c;
            }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = o[j];
    }
    bf16_t* dst;
    if (kind == 0) {
        dst = q_out + ((size_t)tok * nq + hh) * d;
    } else {
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        dst = k_cache + (((size_t)page * nkv + (hh - nq)) * page_size + off) * d;
    }
    *(uint4*)(dst + t * 8) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]),
                                        pack_bf16x2(v[6], v[7]));
}

// Steps with prompt portions, where the head size is a power of two and the whole head rotates in
// halves: the threads of a head (d / 8 of them, neighbours in one wave) walk up to QKV_HEADS heads
// of one token.  The token's angles and the norm weights are read once for all of them, the heads'
// rows are all asked for before the first is used, and the sum of squares and the rotation partners
// go from lane to lane without shared memory.  The sum runs in the order of the kernel above, so
// that both give the same bits.
#define QKV_HEADS 8
template <int TPU>
__global__ __launch_bounds__(QKV_THREADS) void qk_rope_kv_bf16_rows_kernel(
    bf16_t* __restrict__ q_out, bf16_t* __restrict__ k_cache, bf16_t* __restrict__ v_cache,
    const bf16_t* __restrict__ qkv, const float* __restrict__ q_norm_w, const float* __restrict__ k_norm_w,
    const float* __restrict__ cos_t, const float* __restrict__ sin_t, const int* __restrict__ slots,
    int n, int nq, int nkv, int page_size, float eps, int add_one, int v_from) {
    constexpr int D = TPU * 8, HALF = D / 2;
    __shared__ uint16_t tile[QKV_THREADS * 8];
    if ((int)blockIdx.x >= v_from) {
        values_in_groups(tile, v_cache, qkv, slots, (int)blockIdx.x - v_from, n, nq, nkv, D, page_size);
        return;
    }
    const int rg = threadIdx.x / TPU, t = threadIdx.x % TPU;
    const int chunks = (nq + nkv + QKV_HEADS - 1) / QKV_HEADS;
    const long long item = (long long)blockIdx.x * (QKV_THREADS / TPU) + rg;
    if (item >= (long long)n * chunks) return;
    const int tok = (int)(item / chunks), h0 = (int)(item % chunks) * QKV_HEADS;
    const int hn = nq + nkv - h0 < QKV_HEADS ? nq + nkv - h0 : QKV_HEADS;
    const int e0 = t * 8;
    const bool first = e0 < HALF;
    const bf16_t* src = qkv + ((size_t)tok * (nq + 2 * nkv) + h0) * D + e0;
    uint4 raw[QKV_HEADS];
#pragma unroll
    for (int i = 0; i < QKV_HEADS; ++i)
        if (i < hn) raw[i] = *(const uint4*)(src + (size_t)i * D);
    const size_t at = (size_t)tok * HALF + (first ? e0 : e0 - HALF);
    const float4 c0 = *(const float4*)(cos_t + at), c1 = *(const float4*)(cos_t + at + 4);
    const float4 s0 = *(const float4*)(sin_t + at), s1 = *(const float4*)(sin_t + at + 4);
    const float cs[8] = {c0.x, c0.y, c0.z, c0.w, c1.x, c1.y, c1.z, c1.w};
    const float sn[8] = {s0.x, s0.y, s0.z, s0.w, s1.x, s1.y, s1.z, s1.w};
    float gq[8], gk[8];
    if (q_norm_w != nullptr && h0 < nq) {
        const float4 g0 = *(const float4*)(q_norm_w + e0), g1 = *(const float4*)(q_norm_w + e0 + 4);
        gq[0] = g0.x; gq[1] = g0.y; gq[2] = g0.z; gq[3] = g0.w; gq[4] = g1.x; gq[5] = g1.y; gq[6] = g1.z; gq[7] = g1.w;
    }
    if (k_norm_w != nullptr && h0 + hn > nq) {
        const float4 g0 = *(const float4*)(k_norm_w + e0), g1 = *(const float4*)(k_norm_w + e0 + 4);
        gk[0] = g0.x; gk[1] = g0.y; gk[2] = g0.z; gk[3] = g0.w; gk[4] = g1.x; gk[5] = g1.y; gk[6] = g1.z; gk[7] = g1.w;
    }
    bf16_t* k_row = nullptr;
    if (h0 + hn > nq) {
        const int slot = slots[tok];
        const int page = slot / page_size, off = slot - page * page_size;
        k_row = k_cache + ((size_t)page * nkv * page_size + off) * D + e0;      // + head * page_size * D
    }
#pragma unroll
    for (int i = 0; i < QKV_HEADS; ++i) {
        if (i >= hn) break;
        const int hh = h0 + i;
        const bool is_q = hh < nq;
        const uint32_t w[4] = {raw[i].x, raw[i].y, raw[i].z, raw[i].w};
        float v[8];
#pragma unroll
        for (int j = 0; j < 4; ++j) {
            v[2 * j] = __uint_as_float(w[j] << 16);
            v[2 * j + 1] = __uint_as_float(w[j] & 0xffff0000u);
        }
        if ((is_q ? q_norm_w : k_norm_w) != nullptr) {
            float ss = 0.f;
#pragma unroll
            for (int j = 0; j < 8; ++j) ss += v[j] * v[j];
            float total = 0.f;
#pragma unroll
            for (int j = 0; j < TPU; ++j) total += __shfl(ss, j, TPU);
            const float scale = 1.0f / sqrtf(total / (float)D + eps);
#pragma unroll
            for (int j = 0; j < 8; ++j) {
                const float g = is_q ? gq[j] : gk[j];
                v[j] = scale * v[j] * (add_one ? 1.0f + g : g);
            }
        }
        float o[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const float partner = __shfl_xor(v[j], TPU / 2, TPU);
            o[j] = first ? v[j] * cs[j] - partner * sn[j] : partner * sn[j] + v[j] * cs[j];
        }
        bf16_t* dst = is_q ? q_out + ((size_t)tok * nq + hh) * D + e0 : k_row + (size_t)(hh - nq) * page_size * D;
        *(uint4*)dst = make_uint4(pack_bf16x2(o[0], o[1]), pack_bf16x2(o[2], o[3]), pack_bf16x2(o[4], o[5]),
                                  pack_bf16x2(o[6], o[7]));
    }
}

template <int TPU>
static void launch_rows(bf16_t* q_out, bf16_t* k_cache, bf16_t* v_cache, const bf16_t* qkv, const float* q_norm_w,
                        const float* k_norm_w, const float* cos_t, const float* sin_t, const int* slots, int n,
                        int nq, int nkv, int page_size, float eps, int add_one, long long v_blocks,
                        hipStream_t stream) {
    const long long chunks = (nq + nkv + QKV_HEADS - 1) / QKV_HEADS;
    const long long qk_blocks = ((long long)n * chunks + QKV_THREADS / TPU - 1) / (QKV_THREADS / TPU);
    qk_rope_kv_bf16_rows_kernel<TPU><<<(unsigned)(qk_blocks + v_blocks), QKV_THREADS, 0, stream>>>(
        q_out, k_cache, v_cache, qkv, q_norm_w, k_norm_w, cos_t, sin_t, slots, n, nq, nkv, page_size, eps, add_one,
        (int)qk_blocks);
}

static int g_group_values = 1, g_rows = 1;
// Measurement switches: group_values 0 writes the values token by token in every step; rows 0 keeps
// steps with prompt portions on the kernel that gives a thread one head.
extern "C" void ia_qk_rope_kv_tune(int group_values, int rows) { g_group_values = group_values; g_rows = rows; }

extern "C" int ia_qk_rope_kv(void* q_out, void* k_cache, void* v_cache, const void* qkv,
                             const float* q_norm_w, const float* k_norm_w, const float* cos_t,
                             const float* sin_t, const int* slots, int n, int nq, int nkv, int d,
                             int rot, int interleaved, int page_size, float eps, int add_one,
                             int dtype, hipStream_t stream) {
    IA_CHECK(n >= 0 && nq > 0 && nkv > 0, "qk_rope_kv: bad sizes n=%d nq=%d nkv=%d", n, nq, nkv);
    IA_CHECK(d > 0 && d <= QK_MAX_HEAD_DIM, "qk_rope_kv: head_dim %d is outside 1..%d", d, QK_MAX_HEAD_DIM);
    IA_CHECK(rot >= 0 && rot <= d && rot % 2 == 0, "qk_rope_kv: rot_dim %d must be even and <= head_dim %d", rot, d);
    IA_CHECK((cos_t == nullptr) == (sin_t == nullptr), "qk_rope_kv: cos and sin tables must come together");
    IA_CHECK(cos_t == nullptr || rot > 0, "qk_rope_kv: a rotary table needs rot_dim > 0");
    IA_CHECK(slots == nullptr || (k_cache && v_cache && page_size > 0), "qk_rope_kv: slots given without a cache");
    if (n == 0) return 0;
    const long long units = (long long)n * (slots ? nq + 2 * nkv : nq);
    const unsigned grid = (unsigned)((units + QK_WAVES - 1) / QK_WAVES);
    const uintptr_t ptrs = (uintptr_t)q_out | (uintptr_t)qkv | (uintptr_t)(slots ? k_cache : nullptr) |
                           (uintptr_t)q_norm_w | (uintptr_t)k_norm_w | (uintptr_t)cos_t | (uintptr_t)sin_t;
    if (dtype == IA_BF16 && d % 8 == 0 && d / 8 <= QKV_THREADS && (ptrs & 15) == 0) {
        const int units_per_block = QKV_THREADS / (d / 8);
        // values in groups of eight tokens: where a block's threads cover eight rows, pages hold whole
        // groups, and the step has prompt portions in it (single decoded tokens have no neighbours)
        const bool grouped = g_group_values && slots != nullptr && units_per_block >= QKV_GROUP &&
                             page_size % QKV_GROUP == 0 && n >= 2 * QKV_GROUP && ((uintptr_t)v_cache & 15) == 0;
        long long qk_units = units, v_blocks = 0;
        if (grouped) {
            const int hpb = units_per_block / QKV_GROUP;
            qk_units = (long long)n * (nq + nkv);
            v_blocks = (long long)((n + QKV_GROUP - 1) / QKV_GROUP) * ((nkv + hpb - 1) / hpb);
        }
        const long long qk_blocks = (qk_units + units_per_block - 1) / units_per_block;
        IA_CHECK(qk_blocks + v_blocks < (1ll << 31), "qk_rope_kv: %d tokens are too many for one launch", n);
        const int tpu = d / 8;
        if (grouped && g_rows && cos_t != nullptr && rot == d && !interleaved && tpu >= 2 && tpu <= 64 &&
            (tpu & (tpu - 1)) == 0) {
#define ROWS_CASE(T) case T: launch_rows<T>((bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, (const bf16_t*)qkv, \
                     q_norm_w, k_norm_w, cos_t, sin_t, slots, n, nq, nkv, page_size, eps, add_one, v_blocks, stream); break;
            switch (tpu) { ROWS_CASE(2) ROWS_CASE(4) ROWS_CASE(8) ROWS_CASE(16) ROWS_CASE(32) ROWS_CASE(64) }
#undef ROWS_CASE
            IA_LAUNCH_CHECK("qk_rope_kv");
            return 0;
        }
        qk_rope_kv_bf16_vec_kernel<<<(unsigned)(qk_blocks + v_blocks), QKV_THREADS, 0, stream>>>(
            (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, (const bf16_t*)qkv, q_norm_w, k_norm_w,
            cos_t, sin_t, slots, n, nq, nkv, d, rot, interleaved, page_size, eps, add_one,
            grouped ? (int)qk_blocks : -1);
        IA_LAUNCH_CHECK("qk_rope_kv");
        return 0;
    }
    if (dtype == IA_F32)
        qk_rope_kv_kernel<float><<<grid, QK_WAVES * IA_WAVE, 0, stream>>>(
            (float*)q_out, (float*)k_cache, (float*)v_cache, (const float*)qkv, q_norm_w, k_norm_w,
            cos_t, sin_t, slots, n, nq, nkv, d, rot, interleaved, page_size, eps, add_one);
    else if (dtype == IA_BF16)
        qk_rope_kv_kernel<bf16_t><<<grid, QK_WAVES * IA_WAVE, 0, stream>>>(
            (bf16_t*)q_out, (bf16_t*)k_cache, (bf16_t*)v_cache, (const bf16_t*)qkv, q_norm_w, k_norm_w,
            cos_t, sin_t, slots, n, nq, nkv, d, rot, interleaved, page_size, eps, add_one);
    else
        IA_CHECK(false, "qk_rope_kv: unknown dtype %d", dtype);
    IA_LAUNCH_CHECK("qk_rope_kv");
    return 0;
}
