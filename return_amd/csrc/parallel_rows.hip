// Row kernels of a layer whose sublayers run side by side, of attentions with biases, blended values, norms over whole
// projections and gates on their output, and of feed-forwards whose halves meet in a kernel of their own.
//
//   add_rmsnorm_pair   h += a + b (the 32-bit stream; a and b, in the storage type, may each be null), then two RMS
//                      norms of the same row with weights of their own: x1 = h / sqrt(mean(h^2) + eps1) * w1,
//                      x2 = h / sqrt(mean(h^2) + eps2) * w2. One workgroup per row, one pass over the row: its
//                      elements stay in registers between the sum of squares and the two results.
//   qkv_blend_prepare  one wave per (token, head) over the projection row [q heads | k heads | v heads], all heads
//                      of D elements (rows ld_qkv elements apart): a 32-bit bias per column is added (null: none); a
//                      q or k head is divided by the root mean square of its first Dn elements and weighed (w_q, w_k
//                      [D], null: no norm; elements from Dn on are zeros); the first R elements of a q or k head turn by
//                      the token's position, element j with j + R/2; q goes to q_out [T, Hq, D], k to its row of the
//                      key pool. v: mode 1 writes the first Dv elements of the biased v into `first` (32-bit,
//                      [T, Hkv, Dv]: a head's true width, which layers of other row widths share) and v into the
//                      value pool; mode 2 stores (1 - lambda) v + lambda first[t]; mode 0 stores v.
//   qkv_rows_prepare   one workgroup per token over the same row [q heads | k heads | v heads]: the whole query part is
//                      divided by the root mean square of its nq elements and weighed (w_q [Hq D]), the whole key part
//                      by that of its nk elements (w_k [Hkv D]; elements beyond a head's true width are zeros and do
//                      not count), the first R elements of every q and k head turn as above, q goes to q_out, k and v
//                      to their cache rows.
//   gate_rows          o[t][i] *= sigmoid(g[t][i]); both rows apart by their own distances
//   gated_rows         out[t][i] from gu[t][i] and gu[t][I + i] (32-bit or storage type, rows ld_gu elements apart): kind 0
//                      silu(g) u; kind 1 g sigmoid(slope g) (u + 1) with g = min(gate, limit), u = clamp(up, -limit, limit).
#include "common.h"
#include <algorithm>

#define PR_THREADS 256
#define PR_KEEP 16

template <typename T>
__global__ __launch_bounds__(PR_THREADS) void add_rmsnorm_pair_kernel(
    float* __restrict__ h, const T* __restrict__ a, const T* __restrict__ b, const float* __restrict__ w1, float eps1,
    T* __restrict__ x1, const float* __restrict__ w2, float eps2, T* __restrict__ x2, int H) {
    __shared__ float scratch[16];
    const size_t r = blockIdx.x;
    float* hr = h + r * H;
    const bool fits = H <= PR_THREADS * PR_KEEP;
    float ss = 0.f;
    if (fits) {
        // every read of the row is asked for before the first sum
        float v[PR_KEEP], av[PR_KEEP], bv[PR_KEEP], w1v[PR_KEEP], w2v[PR_KEEP];
#pragma unroll
        for (int i = 0; i < PR_KEEP; ++i) {
            const int c = threadIdx.x + i * PR_THREADS;
            const bool in = c < H;
            v[i] = in ? hr[c] : 0.f;
            av[i] = (in && a != nullptr) ? to_f(a[r * H + c]) : 0.f;
            bv[i] = (in && b != nullptr) ? to_f(b[r * H + c]) : 0.f;
            w1v[i] = in ? w1[c] : 0.f;
            w2v[i] = in ? w2[c] : 0.f;
        }
#pragma unroll
        for (int i = 0; i < PR_KEEP; ++i) {
            v[i] = (v[i] + av[i]) + bv[i];
            ss = fmaf(v[i], v[i], ss);
        }
        const float ms = block_sum(ss, scratch) / (float)H;
        const float r1 = 1.0f / sqrtf(ms + eps1), r2 = 1.0f / sqrtf(ms + eps2);
#pragma unroll
        for (int i = 0; i < PR_KEEP; ++i) {
            const int c = threadIdx.x + i * PR_THREADS;
            if (c < H) {
                if (a != nullptr || b != nullptr) hr[c] = v[i];
                x1[r * H + c] = from_f<T>(v[i] * r1 * w1v[i]);
                x2[r * H + c] = from_f<T>(v[i] * r2 * w2v[i]);
            }
        }
        return;
    }
    for (int c = threadIdx.x; c < H; c += PR_THREADS) {
        float v = hr[c];
        if (a != nullptr) v += to_f(a[r * H + c]);
        if (b != nullptr) v += to_f(b[r * H + c]);
        if (a != nullptr || b != nullptr) hr[c] = v;
        ss = fmaf(v, v, ss);
    }
    const float ms = block_sum(ss, scratch) / (float)H;
    const float r1 = 1.0f / sqrtf(ms + eps1), r2 = 1.0f / sqrtf(ms + eps2);
    for (int c = threadIdx.x; c < H; c += PR_THREADS) {
        const float v = hr[c];                               // (the thread's own store, or the stream as it was)
        x1[r * H + c] = from_f<T>(v * r1 * w1[c]);
        x2[r * H + c] = from_f<T>(v * r2 * w2[c]);
    }
}

// The same for rows of H = 4 n elements up to 4,096: a thread takes four neighbours at a time (16-byte reads of the
// stream and the weights, 8- or 16-byte reads of the deltas), all asked for before the first sum.
__device__ __forceinline__ float4 pr_load4(const float* p) { return *reinterpret_cast<const float4*>(p); }
__device__ __forceinline__ float4 pr_load4(const bf16* p) {
    const uint2 t = *reinterpret_cast<const uint2*>(p);
    return make_float4(__uint_as_float(t.x << 16), __uint_as_float(t.x & 0xffff0000u), __uint_as_float(t.y << 16),
                       __uint_as_float(t.y & 0xffff0000u));
}
__device__ __forceinline__ void pr_store4(float* p, float4 v) { *reinterpret_cast<float4*>(p) = v; }
__device__ __forceinline__ void pr_store4(bf16* p, float4 v) {
    uint2 t;
    t.x = (uint32_t)f2bf_bits(v.x) | ((uint32_t)f2bf_bits(v.y) << 16);
    t.y = (uint32_t)f2bf_bits(v.z) | ((uint32_t)f2bf_bits(v.w) << 16);
    *reinterpret_cast<uint2*>(p) = t;
}

#define PR_VEC 4          // groups of four a thread: rows up to 4 * 4 * 256
template <typename T>
__global__ __launch_bounds__(PR_THREADS) void add_rmsnorm_pair_vec_kernel(
    float* __restrict__ h, const T* __restrict__ a, const T* __restrict__ b, const float* __restrict__ w1, float eps1,
    T* __restrict__ x1, const float* __restrict__ w2, float eps2, T* __restrict__ x2, int H) {
    __shared__ float scratch[16];
    const size_t r = blockIdx.x;
    float* hr = h + r * H;
    const float4 zero = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 v[PR_VEC], av[PR_VEC], bv[PR_VEC], w1v[PR_VEC], w2v[PR_VEC];
#pragma unroll
    for (int i = 0; i < PR_VEC; ++i) {
        const int c = 4 * (threadIdx.x + i * PR_THREADS);
        const bool in = c < H;
        v[i] = in ? pr_load4(hr + c) : zero;
        av[i] = (in && a != nullptr) ? pr_load4(a + r * H + c) : zero;
        bv[i] = (in && b != nullptr) ? pr_load4(b + r * H + c) : zero;
        w1v[i] = in ? pr_load4(w1 + c) : zero;
        w2v[i] = in ? pr_load4(w2 + c) : zero;
    }
    float ss = 0.f;
#pragma unroll
    for (int i = 0; i < PR_VEC; ++i) {
        v[i].x = (v[i].x + av[i].x) + bv[i].x;
        v[i].y = (v[i].y + av[i].y) + bv[i].y;
        v[i].z = (v[i].z + av[i].z) + bv[i].z;
        v[i].w = (v[i].w + av[i].w) + bv[i].w;
        ss = fmaf(v[i].x, v[i].x, ss);
        ss = fmaf(v[i].y, v[i].y, ss);
        ss = fmaf(v[i].z, v[i].z, ss);
        ss = fmaf(v[i].w, v[i].w, ss);
    }
    const float ms = block_sum(ss, scratch) / (float)H;
    const float r1 = 1.0f / sqrtf(ms + eps1), r2 = 1.0f / sqrtf(ms + eps2);
#pragma unroll
    for (int i = 0; i < PR_VEC; ++i) {
        const int c = 4 * (threadIdx.x + i * PR_THREADS);
        if (c < H) {
            if (a != nullptr || b != nullptr) pr_store4(hr + c, v[i]);
            pr_store4(x1 + r * H + c, make_float4(v[i].x * r1 * w1v[i].x, v[i].y * r1 * w1v[i].y, v[i].z * r1 * w1v[i].z,
                                                  v[i].w * r1 * w1v[i].w));
            pr_store4(x2 + r * H + c, make_float4(v[i].x * r2 * w2v[i].x, v[i].y * r2 * w2v[i].y, v[i].z * r2 * w2v[i].z,
                                                  v[i].w * r2 * w2v[i].w));
        }
    }
}

extern "C" int ra_add_rmsnorm_pair(float* h, const void* a, const void* b, const float* w1, float eps1, void* x1,
                                   const float* w2, float eps2, void* x2, int rows, int H, int dtype, void* stream) {
    if (rows <= 0) return RA_OK;
    if (H < 1 || h == nullptr || w1 == nullptr || w2 == nullptr || x1 == nullptr || x2 == nullptr) return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    if (dtype != RA_DTYPE_F32 && dtype != RA_DTYPE_BF16) return RA_ERR_ARG;
    const auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    if (H % 4 == 0 && H <= 4 * PR_VEC * PR_THREADS && aligned(h) && aligned(a) && aligned(b) && aligned(w1) && aligned(w2) &&
        aligned(x1) && aligned(x2) && (dtype == RA_DTYPE_F32 || H % 8 == 0)) {
        if (dtype == RA_DTYPE_F32)
            hipLaunchKernelGGL(add_rmsnorm_pair_vec_kernel<float>, dim3(rows), dim3(PR_THREADS), 0, st, h, (const float*)a,
                               (const float*)b, w1, eps1, (float*)x1, w2, eps2, (float*)x2, H);
        else
            hipLaunchKernelGGL(add_rmsnorm_pair_vec_kernel<bf16>, dim3(rows), dim3(PR_THREADS), 0, st, h, (const bf16*)a,
                               (const bf16*)b, w1, eps1, (bf16*)x1, w2, eps2, (bf16*)x2, H);
        return ra_launch_status();
    }
    if (dtype == RA_DTYPE_F32)
        hipLaunchKernelGGL(add_rmsnorm_pair_kernel<float>, dim3(rows), dim3(PR_THREADS), 0, st, h, (const float*)a,
                           (const float*)b, w1, eps1, (float*)x1, w2, eps2, (float*)x2, H);
    else if (dtype == RA_DTYPE_BF16)
        hipLaunchKernelGGL(add_rmsnorm_pair_kernel<bf16>, dim3(rows), dim3(PR_THREADS), 0, st, h, (const bf16*)a,
                           (const bf16*)b, w1, eps1, (bf16*)x1, w2, eps2, (bf16*)x2, H);
    else
        return RA_ERR_ARG;
    return ra_launch_status();
}

// ------------------------------------------------------------------ q/k/v preparation with biases and blended values
template <typename T>
__global__ void qkv_blend_prepare_kernel(const T* __restrict__ qkv, long long ld_qkv, int Hq, int Hkv, int D,
                                         const float* __restrict__ bias, const float* __restrict__ w_q,
                                         const float* __restrict__ w_k, int Dn, float eps,
                                         const int* __restrict__ positions, const float* __restrict__ cos_t,
                                         const float* __restrict__ sin_t, int R, T* __restrict__ q_out,
                                         T* __restrict__ k_pool, T* __restrict__ v_pool, const int* __restrict__ slots,
                                         int P, long long pool_rows, float* __restrict__ first, int Dv, int mode,
                                         float lambda, long long n_rows) {
    const long long row = (long long)blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
    if (row >= n_rows) return;
    const int lane = threadIdx.x & 63;
    const int heads = Hq + 2 * Hkv;
    const int t = (int)(row / heads);
    const int head = (int)(row % heads);
    const T* src = qkv + (size_t)t * ld_qkv + (size_t)head * D;
    const float* b = bias != nullptr ? bias + (size_t)head * D : nullptr;
    auto value = [&](int c) { return b != nullptr ? to_f(src[c]) + b[c] : to_f(src[c]); };
    if (head >= Hq + Hkv) {
        // a value head: bias, the first layer's values out or blended in, the cache row
        const int kvh = head - Hq - Hkv;
        float* fr = first != nullptr ? first + ((size_t)t * Hkv + kvh) * Dv : nullptr;
        T* dst = nullptr;
        if (v_pool != nullptr) {
            const long long s = slots[t];
            if (s >= 0 && s < pool_rows) dst = v_pool + ra_cache_offset(s, kvh, Hkv, P, D);
        }
        for (int c = lane; c < D; c += 64) {
            float v = value(c);
            if (mode == 1 && c < Dv) fr[c] = v;
            else if (mode == 2) v = (1.0f - lambda) * v + (c < Dv ? lambda * fr[c] : 0.f);
            if (dst != nullptr) dst[c] = from_f<T>(v);
        }
        return;
    }
    T* dst;
    if (head < Hq) {
        dst = q_out + ((size_t)t * Hq + head) * D;
    } else {
        if (k_pool == nullptr) return;
        const long long s = slots[t];
        if (s < 0 || s >= pool_rows) return;
        dst = k_pool + ra_cache_offset(s, head - Hq, Hkv, P, D);
    }
    const int half = R >> 1;
    const int pos = positions[t];
    const float* wn = head < Hq ? w_q : w_k;
    float rstd = 1.f;
    if (wn != nullptr) {
        float ss = 0.f;
        for (int c = lane; c < Dn; c += 64) ss = fmaf(value(c), value(c), ss);
        rstd = 1.0f / sqrtf(wave_sum(ss) / (float)Dn + eps);
    }
    auto normed = [&](int c) { return wn != nullptr ? value(c) * rstd * wn[c] : value(c); };
    for (int j = lane; j < half; j += 64) {
        const float x1 = normed(j), x2 = normed(j + half);
        const float cs = cos_t[(size_t)pos * half + j], sn = sin_t[(size_t)pos * half + j];
        dst[j] = from_f<T>(x1 * cs - x2 * sn);
        dst[j + half] = from_f<T>(x2 * cs + x1 * sn);
    }
    for (int c = R + lane; c < D; c += 64) dst[c] = from_f<T>(normed(c));
}

// The same without biases and blending, for heads of D = 64, 128, 256 or 512 elements that turn wholly or not at all:
// D / 8 neighbouring lanes share a head, each with four neighbours of its first half and the four they turn with, so a
// wave takes 512 / D heads of a token, reads and writes 8 or 16 bytes a lane, and sums the squares by lane moves.
template <typename T, int LPH>
__global__ __launch_bounds__(256) void qkv_heads_prepare_kernel(const T* __restrict__ qkv, long long ld_qkv, int Hq, int Hkv,
                                                                const float* __restrict__ w_q, const float* __restrict__ w_k,
                                                                int Dn, float eps, const int* __restrict__ positions,
                                                                const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                                                T* __restrict__ q_out, T* __restrict__ k_pool,
                                                                T* __restrict__ v_pool, const int* __restrict__ slots, int P,
                                                                long long pool_rows, long long n_rows) {
    constexpr int D = 8 * LPH, HALF = 4 * LPH;
    const long long row = ((long long)blockIdx.x * 256 + threadIdx.x) / LPH;
    const int l = threadIdx.x % LPH;
    const int heads = Hq + 2 * Hkv;
    const bool live = row < n_rows;                          // (every lane stays for the sums)
    const int t = live ? (int)(row / heads) : 0, head = live ? (int)(row % heads) : 0;
    const T* src = qkv + (size_t)t * ld_qkv + (size_t)head * D;
    float4 a = pr_load4(src + 4 * l), b = pr_load4(src + HALF + 4 * l);
    const bool value = head >= Hq + Hkv;
    T* dst = nullptr;
    if (live) {
        if (head < Hq) {
            dst = q_out + ((size_t)t * Hq + head) * D;
        } else if (k_pool != nullptr) {
            const long long s = slots[t];
            if (s >= 0 && s < pool_rows)
                dst = (value ? v_pool : k_pool) + ra_cache_offset(s, value ? head - Hq - Hkv : head - Hq, Hkv, P, D);
        }
    }
    const float* wn = head < Hq ? w_q : w_k;
    const bool turn = cos_t != nullptr;
    const float4 one = make_float4(1.f, 1.f, 1.f, 1.f), zero = make_float4(0.f, 0.f, 0.f, 0.f);
    float4 wa = one, wb = one, cs = one, sn = zero;
    if (wn != nullptr) {
        wa = pr_load4(wn + 4 * l);
        wb = pr_load4(wn + HALF + 4 * l);
    }
    if (turn) {
        const size_t at = (size_t)positions[t] * HALF + 4 * l;
        cs = pr_load4(cos_t + at);
        sn = pr_load4(sin_t + at);
    }
    float ss = fmaf(a.x, a.x, fmaf(a.y, a.y, fmaf(a.z, a.z, a.w * a.w)));
    ss += fmaf(b.x, b.x, fmaf(b.y, b.y, fmaf(b.z, b.z, b.w * b.w)));
#pragma unroll
    for (int o = 1; o < LPH; o <<= 1) ss += __shfl_xor(ss, o, 64);
    if (dst == nullptr) return;
    if (!value) {
        const float rstd = wn != nullptr ? 1.0f / sqrtf(ss / (float)Dn + eps) : 1.f;
        a = make_float4(a.x * rstd * wa.x, a.y * rstd * wa.y, a.z * rstd * wa.z, a.w * rstd * wa.w);
        b = make_float4(b.x * rstd * wb.x, b.y * rstd * wb.y, b.z * rstd * wb.z, b.w * rstd * wb.w);
        if (turn) {
            const float4 u = a, v = b;
            a = make_float4(u.x * cs.x - v.x * sn.x, u.y * cs.y - v.y * sn.y, u.z * cs.z - v.z * sn.z, u.w * cs.w - v.w * sn.w);
            b = make_float4(v.x * cs.x + u.x * sn.x, v.y * cs.y + u.y * sn.y, v.z * cs.z + u.z * sn.z, v.w * cs.w + u.w * sn.w);
        }
    }
    pr_store4(dst + 4 * l, a);
    pr_store4(dst + HALF + 4 * l, b);
}

extern "C" int ra_qkv_blend_prepare(const void* qkv, long long ld_qkv, int T_tokens, int Hq, int Hkv, int D,
                                    const float* bias, const float* w_q, const float* w_k, int Dn, float eps,
                                    const int* positions, const float* cos_t, const float* sin_t, int R, void* q_out,
                                    void* k_pool, void* v_pool, const int* slots, int P, long long pool_rows,
                                    float* first, int Dv, int mode, float lambda, int dtype, void* stream) {
    if (T_tokens <= 0) return RA_OK;
    if ((k_pool == nullptr) != (v_pool == nullptr) || (k_pool != nullptr && (P <= 0 || slots == nullptr))) return RA_ERR_ARG;
    if (D < 1 || Hq < 1 || Hkv < 1 || R < 0 || R > D || (R & 1) || q_out == nullptr ||
        ld_qkv < (long long)(Hq + 2 * Hkv) * D || (w_q == nullptr) != (w_k == nullptr) || Dn < 1 || Dn > D ||
        (R > 0 && (cos_t == nullptr || sin_t == nullptr)) || mode < 0 || mode > 2 ||
        (mode != 0 && (first == nullptr || Dv < 1 || Dv > D)))
        return RA_ERR_ARG;
    const long long n_rows = (long long)T_tokens * (Hq + 2 * Hkv);
    dim3 block(256), grid((unsigned)((n_rows + 3) / 4));
    hipStream_t st = (hipStream_t)stream;
    const auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    if (bias == nullptr && mode == 0 && (R == 0 || R == D) && (D == 64 || D == 128 || D == 256 || D == 512) && ld_qkv % 4 == 0 &&
        aligned(qkv) && aligned(q_out) && aligned(k_pool) && aligned(v_pool) && aligned(w_q) && aligned(w_k) &&
        aligned(cos_t) && aligned(sin_t) && (dtype == RA_DTYPE_F32 || dtype == RA_DTYPE_BF16)) {
        dim3 hgrid((unsigned)((n_rows * (D / 8) + 255) / 256));
#define QKV_HEADS(T_, LPH_)                                                                                            \
    hipLaunchKernelGGL((qkv_heads_prepare_kernel<T_, LPH_>), hgrid, block, 0, st, (const T_*)qkv, ld_qkv, Hq, Hkv, w_q, w_k, \
                       Dn, eps, positions, R ? cos_t : nullptr, R ? sin_t : nullptr, (T_*)q_out, (T_*)k_pool,         \
                       (T_*)v_pool, slots, P, pool_rows, n_rows)
#define QKV_HEADS_D(T_)                                                                                                \
    do {                                                                                                               \
        if (D == 64) QKV_HEADS(T_, 8); else if (D == 128) QKV_HEADS(T_, 16);                                           \
        else if (D == 256) QKV_HEADS(T_, 32); else QKV_HEADS(T_, 64);                                                  \
    } while (0)
        if (dtype == RA_DTYPE_F32) QKV_HEADS_D(float); else QKV_HEADS_D(bf16);
#undef QKV_HEADS_D
#undef QKV_HEADS
        return ra_launch_status();
    }
    if (dtype == RA_DTYPE_F32)
        hipLaunchKernelGGL(qkv_blend_prepare_kernel<float>, grid, block, 0, st, (const float*)qkv, ld_qkv, Hq, Hkv, D, bias, w_q, w_k, Dn, eps,
                           positions, cos_t, sin_t, R, (float*)q_out, (float*)k_pool, (float*)v_pool, slots, P, pool_rows,
                           first, Dv, mode, lambda, n_rows);
    else if (dtype == RA_DTYPE_BF16)
        hipLaunchKernelGGL(qkv_blend_prepare_kernel<bf16>, grid, block, 0, st, (const bf16*)qkv, ld_qkv, Hq, Hkv, D, bias, w_q, w_k, Dn, eps,
                           positions, cos_t, sin_t, R, (bf16*)q_out, (bf16*)k_pool, (bf16*)v_pool, slots, P, pool_rows,
                           first, Dv, mode, lambda, n_rows);
    else
        return RA_ERR_ARG;
    return ra_launch_status();
}

// ------------------------------------------------------------------ q/k/v preparation with norms over whole projections
// V elements at a time: of a q or k head R/2/V units of (V, and the V they turn with) and (D - R)/V units that pass, of a
// v head D/V units. 0 <= unit < total of all heads; the row is read twice (the second time from the caches).
template <typename T, int V> struct PrVec;
template <typename T> struct PrVec<T, 1> {
    static __device__ __forceinline__ void load(const T* p, float (&v)[1]) { v[0] = to_f(*p); }
    static __device__ __forceinline__ void store(T* p, const float (&v)[1]) { *p = from_f<T>(v[0]); }
};
template <typename T> struct PrVec<T, 4> {
    static __device__ __forceinline__ void load(const T* p, float (&v)[4]) {
        const float4 t = pr_load4(p);
        v[0] = t.x; v[1] = t.y; v[2] = t.z; v[3] = t.w;
    }
    static __device__ __forceinline__ void store(T* p, const float (&v)[4]) { pr_store4(p, make_float4(v[0], v[1], v[2], v[3])); }
};

template <typename T, int V>
__global__ __launch_bounds__(1024) void qkv_rows_prepare_kernel(const T* __restrict__ qkv, long long ld_qkv, int Hq, int Hkv,
                                                               int D, const float* __restrict__ w_q,
                                                               const float* __restrict__ w_k, int nq, int nk, float eps,
                                                               const int* __restrict__ positions,
                                                               const float* __restrict__ cos_t, const float* __restrict__ sin_t,
                                                               int R, T* __restrict__ q_out, T* __restrict__ k_pool,
                                                               T* __restrict__ v_pool, const int* __restrict__ slots, int P,
                                                               long long pool_rows) {
    __shared__ float scratch[16];
    const int t = blockIdx.x, tid = threadIdx.x, nt = blockDim.x;
    const T* src = qkv + (size_t)t * ld_qkv;
    const int wq = Hq * D, wk = Hkv * D;
    float sq = 0.f, sk = 0.f;
    for (int c = tid * V; c < wq + wk; c += nt * V) {
        float v[V], s = 0.f;
        PrVec<T, V>::load(src + c, v);
#pragma unroll
        for (int e = 0; e < V; ++e) s = fmaf(v[e], v[e], s);
        if (c < wq) sq += s; else sk += s;                   // (V divides D, so a group lies in one part)
    }
    const float rq = 1.0f / sqrtf(block_sum(sq, scratch) / (float)nq + eps);
    const float rk = 1.0f / sqrtf(block_sum(sk, scratch) / (float)nk + eps);
    long long slot = -1;
    if (k_pool != nullptr) {
        slot = slots[t];
        if (slot >= pool_rows) slot = -1;
    }
    const int half = R >> 1, pairs = half / V, passing = (D - R) / V, per = pairs + passing, per_v = D / V;
    const int n_qk = (slot >= 0 ? Hq + Hkv : Hq) * per, n_all = n_qk + (slot >= 0 ? Hkv * per_v : 0);
    const int pos = positions[t];
    for (int unit = tid; unit < n_all; unit += nt) {
        if (unit >= n_qk) {
            const int kvh = (unit - n_qk) / per_v, c = (unit - n_qk - kvh * per_v) * V;
            float v[V];
            PrVec<T, V>::load(src + wq + wk + (size_t)kvh * D + c, v);
            PrVec<T, V>::store(v_pool + ra_cache_offset(slot, kvh, Hkv, P, D) + c, v);
            continue;
        }
        const int head = unit / per, u = unit - head * per;
        const bool is_q = head < Hq;
        const float rstd = is_q ? rq : rk;
        const float* wn = is_q ? w_q + (size_t)head * D : w_k + (size_t)(head - Hq) * D;
        const T* hs = src + (size_t)head * D;
        T* dst = is_q ? q_out + ((size_t)t * Hq + head) * D : k_pool + ra_cache_offset(slot, head - Hq, Hkv, P, D);
        float a[V], wa[V];
        if (u < pairs) {
            const int j = u * V;
            float b[V], wb[V], cs[V], sn[V], oa[V], ob[V];
            PrVec<T, V>::load(hs + j, a);
            PrVec<T, V>::load(hs + half + j, b);
            PrVec<float, V>::load(wn + j, wa);
            PrVec<float, V>::load(wn + half + j, wb);
            PrVec<float, V>::load(cos_t + (size_t)pos * half + j, cs);
            PrVec<float, V>::load(sin_t + (size_t)pos * half + j, sn);
#pragma unroll
            for (int e = 0; e < V; ++e) {
                const float x1 = a[e] * rstd * wa[e], x2 = b[e] * rstd * wb[e];
                oa[e] = x1 * cs[e] - x2 * sn[e];
                ob[e] = x2 * cs[e] + x1 * sn[e];
            }
            PrVec<T, V>::store(dst + j, oa);
            PrVec<T, V>::store(dst + half + j, ob);
        } else {
            const int c = R + (u - pairs) * V;
            PrVec<T, V>::load(hs + c, a);
            PrVec<float, V>::load(wn + c, wa);
#pragma unroll
            for (int e = 0; e < V; ++e) a[e] = a[e] * rstd * wa[e];
            PrVec<T, V>::store(dst + c, a);
        }
    }
}

extern "C" int ra_qkv_rows_prepare(const void* qkv, long long ld_qkv, int T_tokens, int Hq, int Hkv, int D, const float* w_q,
                                   const float* w_k, int nq, int nk, float eps, const int* positions, const float* cos_t,
                                   const float* sin_t, int R, void* q_out, void* k_pool, void* v_pool, const int* slots,
                                   int P, long long pool_rows, int dtype, void* stream) {
    if (T_tokens <= 0) return RA_OK;
    if ((k_pool == nullptr) != (v_pool == nullptr) || (k_pool != nullptr && (P <= 0 || slots == nullptr))) return RA_ERR_ARG;
    if (D < 1 || Hq < 1 || Hkv < 1 || R < 0 || R > D || (R & 1) || q_out == nullptr || w_q == nullptr || w_k == nullptr ||
        positions == nullptr || ld_qkv < (long long)(Hq + 2 * Hkv) * D || nq < 1 || nq > Hq * D || nk < 1 || nk > Hkv * D ||
        (R > 0 && (cos_t == nullptr || sin_t == nullptr)) || (dtype != RA_DTYPE_F32 && dtype != RA_DTYPE_BF16))
        return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    const auto aligned = [](const void* p) { return ((uintptr_t)p & 15) == 0; };
    const bool vec = D % 4 == 0 && R % 8 == 0 && ld_qkv % 4 == 0 && aligned(qkv) && aligned(q_out) && aligned(k_pool) &&
                     aligned(v_pool) && aligned(w_q) && aligned(w_k) && aligned(cos_t) && aligned(sin_t);
    const int threads = T_tokens <= 256 ? 1024 : 256;        // few tokens: one round of reads a thread
#define QKV_ROWS(T_, V_)                                                                                                 \
    hipLaunchKernelGGL((qkv_rows_prepare_kernel<T_, V_>), dim3(T_tokens), dim3(threads), 0, st, (const T_*)qkv, ld_qkv, Hq, \
                       Hkv, D, w_q, w_k, nq, nk, eps, positions, cos_t, sin_t, R, (T_*)q_out, (T_*)k_pool, (T_*)v_pool, \
                       slots, P, pool_rows)
    if (dtype == RA_DTYPE_F32) { if (vec) QKV_ROWS(float, 4); else QKV_ROWS(float, 1); }
    else { if (vec) QKV_ROWS(bf16, 4); else QKV_ROWS(bf16, 1); }
#undef QKV_ROWS
    return ra_launch_status();
}

// ------------------------------------------------------------------ a gate on every element of a row
template <typename T, int V>
__global__ void gate_rows_kernel(T* __restrict__ o, long long ld_o, const T* __restrict__ g, long long ld_g, int N,
                                 long long total) {
    const int per = N / V;
    for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (long long)gridDim.x * blockDim.x) {
        const long long t = i / per;
        const int c = (int)(i - t * per) * V;
        float a[V], b[V];
        PrVec<T, V>::load(o + t * ld_o + c, a);
        PrVec<T, V>::load(g + t * ld_g + c, b);
#pragma unroll
        for (int e = 0; e < V; ++e) a[e] = a[e] / (1.0f + expf(-b[e]));
        PrVec<T, V>::store(o + t * ld_o + c, a);
    }
}

extern "C" int ra_gate_rows(void* o, long long ld_o, const void* g, long long ld_g, int T_tokens, int N, int dtype,
                            void* stream) {
    if (T_tokens <= 0) return RA_OK;
    if (N < 1 || ld_o < N || ld_g < N || o == nullptr || g == nullptr || (dtype != RA_DTYPE_F32 && dtype != RA_DTYPE_BF16))
        return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    const bool vec = N % 4 == 0 && ld_o % 4 == 0 && ld_g % 4 == 0 && ((uintptr_t)o & 15) == 0 && ((uintptr_t)g & 15) == 0;
    const long long total = (long long)T_tokens * (N / (vec ? 4 : 1));
    const unsigned blocks = (unsigned)std::min<long long>((total + 255) / 256, 65535LL * 16);
#define GATE_ROWS(T_, V_)                                                                                       \
    hipLaunchKernelGGL((gate_rows_kernel<T_, V_>), dim3(blocks), dim3(256), 0, st, (T_*)o, ld_o, (const T_*)g, ld_g, N, total)
    if (dtype == RA_DTYPE_F32) { if (vec) GATE_ROWS(float, 4); else GATE_ROWS(float, 1); }
    else { if (vec) GATE_ROWS(bf16, 4); else GATE_ROWS(bf16, 1); }
#undef GATE_ROWS
    return ra_launch_status();
}

// ------------------------------------------------------------------ the two halves of a feed-forward
template <typename S, typename T, int V>
__global__ void gated_rows_kernel(const S* __restrict__ gu, long long ld_gu, T* __restrict__ out, int I, int kind, float limit,
                                  float slope, long long total) {
    const int per = I / V;
    for (long long i = (long long)blockIdx.x * blockDim.x + threadIdx.x; i < total; i += (long long)gridDim.x * blockDim.x) {
        const long long t = i / per;
        const int c = (int)(i - t * per) * V;
        float a[V], b[V];
        PrVec<S, V>::load(gu + t * ld_gu + c, a);
        PrVec<S, V>::load(gu + t * ld_gu + I + c, b);
#pragma unroll
        for (int e = 0; e < V; ++e) {
            if (kind == 1) {
                const float g = fminf(a[e], limit), u = fminf(fmaxf(b[e], -limit), limit);
                a[e] = g / (1.0f + expf(-slope * g)) * (u + 1.0f);
            } else {
                a[e] = a[e] / (1.0f + expf(-a[e])) * b[e];
            }
        }
        PrVec<T, V>::store(out + t * I + c, a);
    }
}

extern "C" int ra_gated_rows(const void* gu, int gu_dtype, long long ld_gu, void* out, int T_tokens, int I, int kind,
                             float limit, float slope, int dtype, void* stream) {
    if (T_tokens <= 0) return RA_OK;
    if (I < 1 || ld_gu < 2LL * I || kind < 0 || kind > 1 || (kind == 1 && !(limit > 0.f)) || gu == nullptr || out == nullptr ||
        (gu_dtype != RA_DTYPE_F32 && gu_dtype != dtype))
        return RA_ERR_ARG;
    hipStream_t st = (hipStream_t)stream;
    const bool vec = I % 4 == 0 && ld_gu % 4 == 0 && ((uintptr_t)gu & 15) == 0 && ((uintptr_t)out & 15) == 0;
    const long long total = (long long)T_tokens * (I / (vec ? 4 : 1));
    const unsigned blocks = (unsigned)std::min<long long>((total + 255) / 256, 65535LL * 16);
#define GATED_ROWS(S_, T_)                                                                                           \
    do {                                                                                                             \
        if (vec) hipLaunchKernelGGL((gated_rows_kernel<S_, T_, 4>), dim3(blocks), dim3(256), 0, st, (const S_*)gu, ld_gu, \
                                    (T_*)out, I, kind, limit, slope, total);                                         \
        else hipLaunchKernelGGL((gated_rows_kernel<S_, T_, 1>), dim3(blocks), dim3(256), 0, st, (const S_*)gu, ld_gu, \
                                (T_*)out, I, kind, limit, slope, total);                                             \
    } while (0)
    if (dtype == RA_DTYPE_F32) GATED_ROWS(float, float);
    else if (dtype == RA_DTYPE_BF16 && gu_dtype == RA_DTYPE_BF16) GATED_ROWS(bf16, bf16);
    else if (dtype == RA_DTYPE_BF16) GATED_ROWS(float, bf16);
    else return RA_ERR_ARG;
#undef GATED_ROWS
    return ra_launch_status();
}
