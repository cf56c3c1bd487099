// The two ends of an attention whose heads have several maps (queries and keys of their own) over shared values:
// what stands between the projections and the attention kernels, and the combination of two maps behind them.
//
// conv_qkv: the projections' rows [q | k | v | ...] (q: heads x maps x d, k: kv heads x maps x d, v: kv heads x dv) pass a
// short causal convolution a channel (zeros before a sequence's start; a request's last inputs lie in its row of a 32-bit
// state array, [taps - 1][channels], oldest first), then q and k an RMS norm a map of a head (one weight for all) and a
// turn by position of the first `rot` features of each map; keys and values go to their pages, a key head's maps side by
// side (maps * d wide).  The queries leave as [n, heads * maps, maps * d]: query (head, map) is as wide as a key head and
// zero outside its own map, so that its product with the key head's row is the map's score and the attention kernels,
// which know nothing of maps, read every key and every value once for all maps.  Everything between load and store is
// 32-bit.
#include "api.h"
#include "common.h"

#define MA_MAX_WIDTH 512
#define MA_WAVES 4
#define MA_THREADS 256

struct ConvQkvArgs {
    void *q_out, *k_cache, *v_cache;
    const void *proj, *taps;                 // taps [k][C], C channels: q, k and v in the rows' order
    long long ld;
    float* state;
    long long row_floats, tail_off;
    const float *q_norm_w, *k_norm_w, *cos_t, *sin_t;
    const int *slots, *token_seq, *cu_tokens, *state_slots;
    int n, H, G, maps, d, dv, k, rot, interleaved, page;
    float eps;
    int inline_tail;                         // every request of the step brings one token: the kernel moves its tail on itself
    int qk_blocks;
};

// One wave per (token, unit): units are the maps of the query heads, those of the key heads, then the value heads.
template <typename T>
__global__ __launch_bounds__(MA_WAVES * IA_WAVE) void conv_qkv_kernel(const ConvQkvArgs a) {
    __shared__ float buf[MA_WAVES][MA_MAX_WIDTH];
    const int lane = threadIdx.x & (IA_WAVE - 1), wave = threadIdx.x / IA_WAVE;
    const int nq = a.H * a.maps, nk = a.G * a.maps, units = nq + nk + a.G;
    const int C = nq * a.d + nk * a.d + a.G * a.dv;
    const long long unit = (long long)blockIdx.x * MA_WAVES + wave;
    const bool active = unit < (long long)a.n * units;
    const int tok = active ? (int)(unit / units) : 0;
    const int hh = active ? (int)(unit % units) : 0;
    const int kind = hh < nq ? 0 : (hh < nq + nk ? 1 : 2);
    const int width = kind == 2 ? a.dv : a.d;
    const int c0 = kind == 2 ? (nq + nk) * a.d + (hh - nq - nk) * a.dv : hh * a.d;
    float* row = buf[wave];
    float ss = 0.f;
    if (active) {
        const int seq = a.token_seq[tok], first = a.cu_tokens[seq];
        float* tail = a.state != nullptr ? a.state + (long long)a.state_slots[seq] * a.row_floats + a.tail_off : nullptr;
        const T *x = (const T*)a.proj, *taps = (const T*)a.taps;
        for (int j = lane; j < width; j += IA_WAVE) {
            const int c = c0 + j;
            float acc = 0.f;
            for (int q = 0; q < a.k; ++q) {
                const int src = tok - (a.k - 1 - q);
                const float v = src >= first ? ld(x + (long long)src * a.ld + c) : tail[(long long)(a.k - 1 + src - first) * C + c];
                acc = fmaf(ld(taps + (long long)q * C + c), v, acc);
            }
            if (a.inline_tail) {
                for (int m = 0; m + 1 < a.k - 1; ++m) tail[(long long)m * C + c] = tail[(long long)(m + 1) * C + c];
                if (a.k > 1) tail[(long long)(a.k - 2) * C + c] = ld(x + (long long)tok * a.ld + c);
            }
            row[j] = acc;
            ss += acc * acc;
        }
    }
    if (kind != 2) {
        ss = wave_sum(ss);
        const float scale = 1.0f / sqrtf(ss / (float)a.d + a.eps);
        const float* nw = kind == 0 ? a.q_norm_w : a.k_norm_w;
        if (active)
            for (int j = lane; j < a.d; j += IA_WAVE) row[j] = scale * row[j] * nw[j];
    }
    __syncthreads();
    if (!active) return;
    T* dst;
    if (kind == 0) {
        const int m = hh % a.maps;
        T* q_row = (T*)a.q_out + ((size_t)tok * nq + hh) * a.maps * a.d;
        for (int j = lane; j < a.maps * a.d; j += IA_WAVE)
            if (j / a.d != m) st(q_row + j, 0.f);
        dst = q_row + m * a.d;
    } else {
        const int slot = a.slots[tok];
        const int page = slot / a.page, off = slot - page * a.page;
        if (kind == 2) {                          // values are kept transposed inside a page: [dim][slot]
            T* vt = (T*)a.v_cache + ((size_t)page * a.G + (hh - nq - nk)) * a.dv * a.page + off;
            for (int j = lane; j < a.dv; j += IA_WAVE) st(vt + (size_t)j * a.page, row[j]);
            return;
        }
        const int g = (hh - nq) / a.maps, m = (hh - nq) % a.maps;
        dst = (T*)a.k_cache + ((((size_t)page * a.G + g) * a.page + off) * a.maps + m) * a.d;
    }
    const int rot = a.cos_t != nullptr ? a.rot : 0, half = rot / 2;
    for (int i = lane; i < half; i += IA_WAVE) {
        const float c = a.cos_t[(size_t)tok * half + i], s = a.sin_t[(size_t)tok * half + i];
        const int ia = a.interleaved ? 2 * i : i, ib = a.interleaved ? 2 * i + 1 : i + half;
        const float u = row[ia], v = row[ib];
        st(dst + ia, u * c - v * s);
        st(dst + ib, u * s + v * c);
    }
    for (int j = rot + lane; j < a.d; j += IA_WAVE) st(dst + j, row[j]);
}

// The same with 16-byte accesses for bfloat16 and sizes in steps of 8: a thread owns eight neighbouring channels of one
// token.  In the blocks up to qk_blocks the threads of a map meet in shared memory for its sum of squares (added up in
// the order of the features) and for their partners in the turn.  The blocks from there on take the values of eight
// neighbouring tokens, turned round in shared memory: where the tokens' slots are neighbours in one page, starting at a
// multiple of eight, a thread stores a feature's eight slots as 16 bytes.
__device__ __forceinline__ void ma_unpack8(const bf16_t* p, float (&v)[8]) {
    const uint4 q = *reinterpret_cast<const uint4*>(p);
    const uint32_t w[4] = {q.x, q.y, q.z, q.w};
#pragma unroll
    for (int e = 0; e < 4; ++e) {
        v[2 * e] = __uint_as_float(w[e] << 16);
        v[2 * e + 1] = __uint_as_float(w[e] & 0xffff0000u);
    }
}

__device__ __forceinline__ void ma_conv8(const ConvQkvArgs& a, int C, int tok, int c, float (&acc)[8]) {
    const int seq = a.token_seq[tok], first = a.cu_tokens[seq];
    const bf16_t *x = (const bf16_t*)a.proj + c, *taps = (const bf16_t*)a.taps + c;
    float* tail = a.state != nullptr ? a.state + (long long)a.state_slots[seq] * a.row_floats + a.tail_off + c : nullptr;
#pragma unroll
    for (int e = 0; e < 8; ++e) acc[e] = 0.f;
    float v[8], tp[8];
#pragma unroll 4
    for (int q = 0; q < a.k; ++q) {
        const int src = tok - (a.k - 1 - q);
        ma_unpack8(taps + (long long)q * C, tp);
        if (src >= first) {
            ma_unpack8(x + (long long)src * a.ld, v);
        } else {
            const int m = a.k - 1 + src - first;
            const float4 lo = *(const float4*)(tail + (long long)m * C), hi = *(const float4*)(tail + (long long)m * C + 4);
            v[0] = lo.x; v[1] = lo.y; v[2] = lo.z; v[3] = lo.w; v[4] = hi.x; v[5] = hi.y; v[6] = hi.z; v[7] = hi.w;
            if (a.inline_tail && m > 0) {                     // (one token a request: entry m is this thread's alone)
                *(float4*)(tail + (long long)(m - 1) * C) = lo;
                *(float4*)(tail + (long long)(m - 1) * C + 4) = hi;
            }
        }
#pragma unroll
        for (int e = 0; e < 8; ++e) acc[e] = fmaf(tp[e], v[e], acc[e]);
    }
    if (a.inline_tail && a.k > 1) {                           // (the last round's v is the token's own row)
        *(float4*)(tail + (long long)(a.k - 2) * C) = make_float4(v[0], v[1], v[2], v[3]);
        *(float4*)(tail + (long long)(a.k - 2) * C + 4) = make_float4(v[4], v[5], v[6], v[7]);
    }
}

__global__ __launch_bounds__(MA_THREADS) void conv_qkv_vec_kernel(const ConvQkvArgs a) {
    __shared__ float rows[MA_THREADS * 8];
    __shared__ float partial[MA_THREADS];
    const int nq = a.H * a.maps, nk = a.G * a.maps, d = a.d;
    const int Cv = a.G * a.dv, C = (nq + nk) * d + Cv;
    if ((int)blockIdx.x >= a.qk_blocks) {
        uint16_t* tile = (uint16_t*)rows;                     // [8 tokens][256 channels]
        const int vb = (int)blockIdx.x - a.qk_blocks, cbs = (Cv + 255) / 256;
        const int tok0 = vb / cbs * 8, cb0 = vb % cbs * 256;
        const int ti = threadIdx.x >> 5, cc = (threadIdx.x & 31) * 8;
        if (tok0 + ti < a.n && cb0 + cc < Cv) {
            float v[8];
            ma_conv8(a, C, tok0 + ti, (nq + nk) * d + cb0 + cc, v);
            *(uint4*)(tile + ti * 256 + cc) = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]),
                                                         pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
        }
        int slot[8];
        bool together = tok0 + 8 <= a.n;
#pragma unroll
        for (int i = 0; i < 8; ++i) {
            slot[i] = tok0 + i < a.n ? a.slots[tok0 + i] : -1;
            together = together && slot[i] == slot[0] + i;
        }
        together = together && slot[0] % 8 == 0 && a.page % 8 == 0;
        __syncthreads();
        const int c = cb0 + threadIdx.x;
        if (c >= Cv) return;
        const int g = c / a.dv, j = c - g * a.dv;
        bf16_t* feature = (bf16_t*)a.v_cache + ((size_t)g * a.dv + j) * a.page;          // + page * G * dv * page size
        const uint16_t* col = tile + threadIdx.x;
        if (together) {
            const int page = slot[0] / a.page, off = slot[0] - page * a.page;
            uint32_t w[4];
#pragma unroll
            for (int i = 0; i < 4; ++i) w[i] = (uint32_t)col[2 * i * 256] | ((uint32_t)col[(2 * i + 1) * 256] << 16);
            *(uint4*)(feature + (size_t)page * Cv * a.page + off) = make_uint4(w[0], w[1], w[2], w[3]);
        } else {
#pragma unroll
            for (int i = 0; i < 8; ++i) {
                if (slot[i] < 0) continue;
                const int page = slot[i] / a.page, off = slot[i] - page * a.page;
                feature[(size_t)page * Cv * a.page + off].bits = col[i * 256];
            }
        }
        return;
    }
    const int tpu = d / 8, upb = MA_THREADS / tpu;
    const int u = threadIdx.x / tpu, t = threadIdx.x - u * tpu;
    const int units = nq + nk;
    const long long unit = (long long)blockIdx.x * upb + u;
    const bool active = u < upb && unit < (long long)a.n * units;
    const int tok = active ? (int)(unit / units) : 0;
    const int hh = active ? (int)(unit % units) : 0;
    const bool is_q = hh < nq;
    float v[8];
    float ss = 0.f;
    if (active) {
        ma_conv8(a, C, tok, hh * d + t * 8, v);
#pragma unroll
        for (int j = 0; j < 8; ++j) ss = fmaf(v[j], v[j], ss);
    }
    partial[threadIdx.x] = ss;
    __syncthreads();
    if (active) {
        float total = 0.f;
        for (int j = 0; j < tpu; ++j) total += partial[u * tpu + j];
        const float scale = 1.0f / sqrtf(total / (float)d + a.eps);
        const float* nw = is_q ? a.q_norm_w : a.k_norm_w;
        const float4 g0 = *(const float4*)(nw + t * 8), g1 = *(const float4*)(nw + t * 8 + 4);
        const float g[8] = {g0.x, g0.y, g0.z, g0.w, g1.x, g1.y, g1.z, g1.w};
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = scale * v[j] * g[j];
    }
    const int half = a.rot / 2;
    if (a.cos_t != nullptr && !a.interleaved) {               // (partners lie with other threads; all threads pass the barrier)
        if (active) {
#pragma unroll
            for (int j = 0; j < 8; ++j) rows[threadIdx.x * 8 + j] = v[j];
        }
        __syncthreads();
    }
    if (!active) return;
    if (a.cos_t != nullptr) {
        float o[8];
#pragma unroll
        for (int j = 0; j < 8; ++j) {
            const int e = t * 8 + j;
            o[j] = v[j];
            if (e < a.rot) {
                const bool first = a.interleaved ? (e & 1) == 0 : e < half;
                const int i = a.interleaved ? e >> 1 : (first ? e : e - half);
                const float c = a.cos_t[(size_t)tok * half + i], s = a.sin_t[(size_t)tok * half + i];
                const float partner = a.interleaved ? v[j ^ 1] : rows[(size_t)u * tpu * 8 + (first ? e + half : e - half)];
                o[j] = first ? v[j] * c - partner * s : partner * s + v[j] * c;
            }
        }
#pragma unroll
        for (int j = 0; j < 8; ++j) v[j] = o[j];
    }
    const uint4 w = make_uint4(pack_bf16x2(v[0], v[1]), pack_bf16x2(v[2], v[3]), pack_bf16x2(v[4], v[5]), pack_bf16x2(v[6], v[7]));
    if (is_q) {
        const int m = hh % a.maps;
        bf16_t* q_row = (bf16_t*)a.q_out + ((size_t)tok * nq + hh) * a.maps * d + t * 8;
        for (int o = 0; o < a.maps; ++o) *(uint4*)(q_row + o * d) = o == m ? w : make_uint4(0, 0, 0, 0);
    } else {
        const int slot = a.slots[tok];
        const int page = slot / a.page, off = slot - page * a.page;
        const int g = (hh - nq) / a.maps, m = (hh - nq) % a.maps;
        *(uint4*)((bf16_t*)a.k_cache + ((((size_t)page * a.G + g) * a.page + off) * a.maps + m) * d + t * 8) = w;
    }
}

// Behind the convolution of a step whose requests bring more than a token: a request's tail takes its last k - 1 inputs.
template <typename T>
__global__ void conv_qkv_tail_kernel(const ConvQkvArgs a, int C) {
    const int c = blockIdx.x * blockDim.x + threadIdx.x;
    if (c >= C) return;
    const int seq = blockIdx.y;
    const int first = a.cu_tokens[seq], last = a.cu_tokens[seq + 1], q = last - first;
    float* tail = a.state + (long long)a.state_slots[seq] * a.row_floats + a.tail_off + c;
    for (int m = 0; m < a.k - 1; ++m) {
        const int src = last - (a.k - 1) + m;
        const float v = src >= first ? ld((const T*)a.proj + (long long)src * a.ld + c) : tail[(long long)(m + q) * C];
        tail[(long long)m * C] = v;                                      // (m + q < k - 1 here; read before it is written)
    }
}

extern "C" int ia_conv_qkv(void* q_out, void* k_cache, void* v_cache, const void* proj, long long ld, const void* taps, int k,
                           float* state, long long row_floats, long long tail_off, const float* q_norm_w, const float* k_norm_w,
                           float eps, const float* cos_t, const float* sin_t, int rot, int interleaved, const int* slots,
                           const int* token_seq, const int* cu_tokens, const int* state_slots, int n, int n_seqs, int H, int G,
                           int maps, int d, int dv, int page_size, int max_q_len, int dtype, hipStream_t stream) {
    IA_CHECK(n >= 0 && n_seqs >= 0 && H > 0 && G > 0 && maps >= 1 && k >= 1 && max_q_len >= 1,
             "conv_qkv: bad sizes n=%d heads=%d kv heads=%d maps=%d taps=%d", n, H, G, maps, k);
    IA_CHECK(d > 0 && d <= MA_MAX_WIDTH && dv > 0 && dv <= MA_MAX_WIDTH, "conv_qkv: head sizes %d / %d are outside 1..%d", d, dv, MA_MAX_WIDTH);
    IA_CHECK(rot >= 0 && rot <= d && rot % 2 == 0 && (cos_t == nullptr) == (sin_t == nullptr) && (cos_t == nullptr || rot > 0),
             "conv_qkv: a turn of %d features must be even and within %d, with both tables", rot, d);
    const int C = (H + G) * maps * d + G * dv;
    IA_CHECK(C <= ld, "conv_qkv: %d channels do not fit rows of %lld", C, ld);
    IA_CHECK(k == 1 || (state != nullptr && tail_off >= 0 && tail_off + (long long)(k - 1) * C <= row_floats),
             "conv_qkv: the tail of %d x %d does not fit the state row", k - 1, C);
    IA_CHECK(q_out && k_cache && v_cache && slots && page_size > 0 && q_norm_w && k_norm_w, "conv_qkv: outputs, pages and norm weights are needed");
    if (n == 0 || n_seqs == 0) return 0;
    ConvQkvArgs a;
    a.q_out = q_out; a.k_cache = k_cache; a.v_cache = v_cache; a.proj = proj; a.taps = taps; a.ld = ld;
    a.state = k > 1 ? state : nullptr; a.row_floats = row_floats; a.tail_off = tail_off;
    a.q_norm_w = q_norm_w; a.k_norm_w = k_norm_w; a.cos_t = cos_t; a.sin_t = sin_t;
    a.slots = slots; a.token_seq = token_seq; a.cu_tokens = cu_tokens; a.state_slots = state_slots;
    a.n = n; a.H = H; a.G = G; a.maps = maps; a.d = d; a.dv = dv; a.k = k; a.rot = rot; a.interleaved = interleaved; a.page = page_size;
    a.eps = eps; a.inline_tail = k > 1 && max_q_len == 1 ? 1 : 0; a.qk_blocks = 0;
    const uintptr_t ptrs = (uintptr_t)q_out | (uintptr_t)k_cache | (uintptr_t)v_cache | (uintptr_t)proj | (uintptr_t)taps |
                           (uintptr_t)a.state | (uintptr_t)q_norm_w | (uintptr_t)k_norm_w;
    if (dtype == IA_BF16 && d % 8 == 0 && dv % 8 == 0 && ld % 8 == 0 && (ptrs & 15) == 0 && row_floats % 4 == 0 && tail_off % 4 == 0) {
        const int upb = MA_THREADS / (d / 8);
        const long long qk_blocks = ((long long)n * (H + G) * maps + upb - 1) / upb;
        const long long v_blocks = (long long)((n + 7) / 8) * ((G * dv + 255) / 256);
        IA_CHECK(qk_blocks + v_blocks < (1ll << 31), "conv_qkv: %d tokens are too many for one launch", n);
        a.qk_blocks = (int)qk_blocks;
        conv_qkv_vec_kernel<<<(unsigned)(qk_blocks + v_blocks), MA_THREADS, 0, stream>>>(a);
    } else {
        const long long units = (long long)n * ((H + G) * maps + G);
        const unsigned grid = (unsigned)((units + MA_WAVES - 1) / MA_WAVES);
        if (dtype == IA_F32) conv_qkv_kernel<float><<<grid, MA_WAVES * IA_WAVE, 0, stream>>>(a);
        else if (dtype == IA_BF16) conv_qkv_kernel<bf16_t><<<grid, MA_WAVES * IA_WAVE, 0, stream>>>(a);
        else IA_CHECK(false, "conv_qkv: unknown dtype %d", dtype);
    }
    IA_LAUNCH_CHECK("conv_qkv");
    if (k > 1 && !a.inline_tail) {
        const dim3 grid((unsigned)((C + 255) / 256), (unsigned)n_seqs);
        if (dtype == IA_F32) conv_qkv_tail_kernel<float><<<grid, 256, 0, stream>>>(a, C);
        else conv_qkv_tail_kernel<bf16_t><<<grid, 256, 0, stream>>>(a, C);
        IA_LAUNCH_CHECK("conv_qkv (tail)");
    }
    return 0;
}

// ---- the second map taken off the first -----------------------------------------------------------------------------
//     o = a1 - lambda a2,   out = o / sqrt(mean(o^2) + eps) * scale            (a head's dv features; 32-bit, rounded once)
// a [n, H, 2, dv].  One wave a (token, head).
template <typename T>
__global__ __launch_bounds__(256) void differ_norm_kernel(T* __restrict__ out, const T* __restrict__ a, float lambda, float eps,
                                                          float scale, int dv, long long units) {
    const long long unit = (long long)blockIdx.x * 4 + threadIdx.x / IA_WAVE;
    if (unit >= units) return;
    const int lane = threadIdx.x & (IA_WAVE - 1);
    const T *a1 = a + unit * 2 * dv, *a2 = a1 + dv;
    float sq = 0.f;
    for (int c = lane; c < dv; c += IA_WAVE) {
        const float o = fmaf(-lambda, ld(a2 + c), ld(a1 + c));
        sq = fmaf(o, o, sq);
    }
    const float rs = scale / sqrtf(wave_sum(sq) / (float)dv + eps);
    for (int c = lane; c < dv; c += IA_WAVE) st(out + unit * dv + c, fmaf(-lambda, ld(a2 + c), ld(a1 + c)) * rs);
}

// The same for bfloat16 and heads in steps of 8: `lanes` (a power of two) neighbouring lanes a (token, head), eight
// features a lane.
__global__ __launch_bounds__(256) void differ_norm_vec_kernel(bf16_t* __restrict__ out, const bf16_t* __restrict__ a, float lambda,
                                                              float eps, float scale, int dv, int lanes, long long units) {
    const int per_block = 256 / lanes;
    const long long unit = (long long)blockIdx.x * per_block + threadIdx.x / lanes;
    const int c = threadIdx.x % lanes * 8;
    const bool mine = unit < units && c < dv;
    float o[8] = {0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f, 0.f};
    if (mine) {
        float u[8], v[8];
        ma_unpack8(a + unit * 2 * dv + c, u);
        ma_unpack8(a + unit * 2 * dv + dv + c, v);
#pragma unroll
        for (int i = 0; i < 8; ++i) o[i] = fmaf(-lambda, v[i], u[i]);
    }
    float sq = 0.f;
#pragma unroll
    for (int i = 0; i < 8; ++i) sq = fmaf(o[i], o[i], sq);
    for (int s = lanes / 2; s > 0; s >>= 1) sq += __shfl_xor(sq, s, IA_WAVE);
    if (!mine) return;
    const float rs = scale / sqrtf(sq / (float)dv + eps);
    *(uint4*)(out + unit * dv + c) = make_uint4(pack_bf16x2(o[0] * rs, o[1] * rs), pack_bf16x2(o[2] * rs, o[3] * rs),
                                                pack_bf16x2(o[4] * rs, o[5] * rs), pack_bf16x2(o[6] * rs, o[7] * rs));
}

extern "C" int ia_differ_norm(void* out, const void* a, float lambda, float eps, float scale, int n, int H, int dv, int dtype,
                              hipStream_t stream) {
    IA_CHECK(n >= 0 && H > 0 && dv > 0, "differ_norm: n=%d heads=%d of %d", n, H, dv);
    if (n == 0) return 0;
    const long long units = (long long)n * H;
    IA_CHECK(units < (1ll << 31), "differ_norm: %d tokens x %d heads exceed the grid", n, H);
    if (dtype == IA_BF16 && dv % 8 == 0 && dv <= 512 && (((uintptr_t)out | (uintptr_t)a) & 15) == 0) {
        int lanes = 1;
        while (lanes * 8 < dv) lanes *= 2;
        const int per_block = 256 / lanes;
        differ_norm_vec_kernel<<<(unsigned)((units + per_block - 1) / per_block), 256, 0, stream>>>(
            (bf16_t*)out, (const bf16_t*)a, lambda, eps, scale, dv, lanes, units);
    } else if (dtype == IA_F32) {
        differ_norm_kernel<float><<<(unsigned)((units + 3) / 4), 256, 0, stream>>>((float*)out, (const float*)a, lambda, eps, scale, dv, units);
    } else if (dtype == IA_BF16) {
        differ_norm_kernel<bf16_t><<<(unsigned)((units + 3) / 4), 256, 0, stream>>>((bf16_t*)out, (const bf16_t*)a, lambda, eps, scale, dv, units);
    } else {
        IA_CHECK(false, "differ_norm: unknown dtype %d", dtype);
    }
    IA_LAUNCH_CHECK("differ_norm");
    return 0;
}
