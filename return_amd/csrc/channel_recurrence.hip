// A gated linear recurrence per channel over the rows of a step, for requests that arrive in pieces:
//
//   r = sigmoid(R_b u_b + rb),  i = sigmoid(I_b u_b + ib)      (a matrix per block b of `bw` neighbouring channels)
//   log a = rate * r,  a = exp(log a)                          (rate < 0, one number per channel)
//   S_t = a S_(t-1) + sqrt(1 - a^2) i u;   out_t = S_t gelu_tanh(y_t + yb) * out_scale
// u is what the short filter in front left, in the storage type; the gates' products are summed in 32-bit and
// everything from their logits to the read-out stays there. sqrt(1 - a^2) is formed as sqrt(-expm1(2 log a)), which
// keeps its digits where a is close to one. S [slots, width] is 32-bit and lives between steps.
//
// Kernels:
//   lru_gates_mfma_kernel (bfloat16, bw a multiple of 8): a wave takes 16 output channels of one block and 16 RT rows;
//     both gates' products run on the matrix cores (16x16x32; A = rows of the weight, B = rows of u, both read straight
//     from memory: a block's weights are a few dozen KB and stay in the caches), and the epilogue forms a and the input
//     x = sqrt(1 - a^2) i u. In a step of single tokens (STEP) it also advances the state and writes the result, so
//     that the whole recurrence of such a step is this kernel.
//   lru_gates_kernel: the same gates by 32-bit FMA, any block width, both storage types.
//   lru_carry_kernel, lru_scan_kernel: a request's rows in chunks of CH. The recurrence is linear, so a chunk's effect on
//     the state is S -> P S + E with P the product of its decays and E what it leaves from a zero state: the first kernel
//     forms (P, E) of every chunk but the last, the second folds the chunks before its own, walks its rows and writes the
//     results; the last chunk's threads write the new state. The first kernel leaves a copy of the old state for the
//     second (in the place of the first chunk's P), so that no thread reads what another one writes. One chunk: the
//     second kernel alone.
#include "common.h"

typedef __bf16 bf16x8_t __attribute__((ext_vector_type(8)));
typedef float float4_t __attribute__((ext_vector_type(4)));

__device__ __forceinline__ float lru_sigmoid(float v) { return 1.f / (1.f + expf(-v)); }
__device__ __forceinline__ float lru_gelu(float z) {
    return 0.5f * z * (1.f + tanhf(0.79788456080286535588f * (z + 0.044715f * z * z * z)));
}
// the gates' logits and u of one channel -> decay and input
__device__ __forceinline__ void lru_decay_input(float lr, float li, float rate, float u, float& a, float& x) {
    const float log_a = rate * lru_sigmoid(lr);
    a = expf(log_a);
    x = sqrtf(fmaxf(-expm1f(2.f * log_a), 0.f)) * lru_sigmoid(li) * u;
}

struct LruStep {                 // what a step of single tokens needs beyond the gates
    float* S;                    // [slots, width]
    const int* slot_ids;
    const bf16* y;               // rows ld_y apart
    long long ld_y;
    const float* y_bias;
    float out_scale;
    bf16* out;                   // rows ld_out apart, width_out columns of which those from width on become zeros
    long long ld_out;
    int width_out;
};

// (one wave a workgroup while the waves are few, four otherwise)
template <int RT, bool STEP>
__global__ __launch_bounds__(256) void lru_gates_mfma_kernel(
    const bf16* __restrict__ u, const bf16* __restrict__ w, const float* __restrict__ bias, const float* __restrict__ rate,
    float* __restrict__ a_out, float* __restrict__ x_out, int T_tokens, int width, int bw, int n_tiles, LruStep sx) {
    const int tile = blockIdx.x * (blockDim.x >> 6) + (threadIdx.x >> 6);
    if (tile >= n_tiles) return;                         // (no barrier in this kernel)
    const int lane = threadIdx.x & 63, n = lane & 15, g = lane >> 4;
    const int per_block = (bw + 15) / 16;
    const int b = tile / per_block, c0 = (tile - b * per_block) * 16;
    const int t0 = blockIdx.y * 16 * RT;
    const bf16x8_t z8 = {0, 0, 0, 0, 0, 0, 0, 0};
    const bool row_ok = c0 + n < bw;
    const bf16* wr = w + ((size_t)(b * 2) * bw + (row_ok ? c0 + n : 0)) * bw;
    const bf16* wi = wr + (size_t)bw * bw;
    const bf16* ur[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) ur[rt] = u + (size_t)min(t0 + rt * 16 + n, T_tokens - 1) * width + (size_t)b * bw;
    // lane (n, g) of the results: row n of each group of 16, channels 4g .. 4g + 3 of the tile. What the epilogue reads
    // is asked for here, so that it arrives with the operands.
    const bool ch_ok = c0 + 4 * g < bw;
    const int ch = b * bw + (ch_ok ? c0 + 4 * g : 0);
    const float4_t rb = *reinterpret_cast<const float4_t*>(bias + ch);
    const float4_t ib = *reinterpret_cast<const float4_t*>(bias + width + ch);
    const float4_t ra = *reinterpret_cast<const float4_t*>(rate + ch);
    [[maybe_unused]] float4_t yb, st[RT];
    [[maybe_unused]] uint2 yw[RT];
    [[maybe_unused]] float* Sp[RT];
    uint2 uw[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int t = min(t0 + rt * 16 + n, T_tokens - 1);
        uw[rt] = *reinterpret_cast<const uint2*>(u + (size_t)t * width + ch);
        if constexpr (STEP) {
            yw[rt] = *reinterpret_cast<const uint2*>(sx.y + (size_t)t * sx.ld_y + ch);
            Sp[rt] = sx.S + (size_t)sx.slot_ids[t] * width + ch;
            st[rt] = *reinterpret_cast<const float4_t*>(Sp[rt]);
        }
    }
    if constexpr (STEP) yb = *reinterpret_cast<const float4_t*>(sx.y_bias + ch);
    float4_t accr[RT], acci[RT];
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) accr[rt] = acci[rt] = float4_t{0.f, 0.f, 0.f, 0.f};
#pragma unroll 4
    for (int k0 = 0; k0 < bw; k0 += 32) {
        const int k = k0 + 8 * g;
        const bool in = k < bw;
        const int ks = in ? k : 0;
        bf16x8_t ar = *reinterpret_cast<const bf16x8_t*>(wr + ks);
        bf16x8_t ai = *reinterpret_cast<const bf16x8_t*>(wi + ks);
        ar = (in && row_ok) ? ar : z8;
        ai = (in && row_ok) ? ai : z8;
#pragma unroll
        for (int rt = 0; rt < RT; ++rt) {
            bf16x8_t bu = *reinterpret_cast<const bf16x8_t*>(ur[rt] + ks);
            bu = in ? bu : z8;
            accr[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ar, bu, accr[rt], 0, 0, 0);
            acci[rt] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(ai, bu, acci[rt], 0, 0, 0);
        }
    }
    MFMA_SETTLE();
    if constexpr (STEP) {
        // the last wave's lanes also clear the columns beyond the recurrence's
        if (tile == n_tiles - 1 && g == 0) {
#pragma unroll
            for (int rt = 0; rt < RT; ++rt) {
                const int t = t0 + rt * 16 + n;
                if (t < T_tokens)
                    for (int c = width; c < sx.width_out; ++c) sx.out[(size_t)t * sx.ld_out + c] = from_f<bf16>(0.f);
            }
        }
    }
    if (!ch_ok) return;
#pragma unroll
    for (int rt = 0; rt < RT; ++rt) {
        const int t = t0 + rt * 16 + n;
        if (t >= T_tokens) continue;
        const float uf[4] = {__uint_as_float(uw[rt].x << 16), __uint_as_float(uw[rt].x & 0xffff0000u),
                             __uint_as_float(uw[rt].y << 16), __uint_as_float(uw[rt].y & 0xffff0000u)};
        float4_t a4, x4;
#pragma unroll
        for (int e = 0; e < 4; ++e) {
            float a, x;
            lru_decay_input(accr[rt][e] + rb[e], acci[rt][e] + ib[e], ra[e], uf[e], a, x);
            a4[e] = a;
            x4[e] = x;
        }
        if constexpr (STEP) {
            const float yf[4] = {__uint_as_float(yw[rt].x << 16), __uint_as_float(yw[rt].x & 0xffff0000u),
                                 __uint_as_float(yw[rt].y << 16), __uint_as_float(yw[rt].y & 0xffff0000u)};
            float4_t s4 = st[rt];
            float o[4];
#pragma unroll
            for (int e = 0; e < 4; ++e) {
                s4[e] = fmaf(a4[e], s4[e], x4[e]);
                o[e] = s4[e] * lru_gelu(yf[e] + yb[e]) * sx.out_scale;
            }
            *reinterpret_cast<float4_t*>(Sp[rt]) = s4;
            uint2 ow;
            ow.x = (uint32_t)f2bf_bits(o[0]) | ((uint32_t)f2bf_bits(o[1]) << 16);
            ow.y = (uint32_t)f2bf_bits(o[2]) | ((uint32_t)f2bf_bits(o[3]) << 16);
            *reinterpret_cast<uint2*>(sx.out + (size_t)t * sx.ld_out + ch) = ow;
        } else {
            *reinterpret_cast<float4_t*>(a_out + (size_t)t * width + ch) = a4;
            *reinterpret_cast<float4_t*>(x_out + (size_t)t * width + ch) = x4;
        }
    }
}

// Grid (64-channel tiles of every block, groups of LRU_ROWS rows): a thread owns one output channel; the rows' u go
// through LDS a piece of the block at a time.
#define LRU_ROWS 8
#define LRU_PIECE 256
template <typename T>
__global__ __launch_bounds__(64) void lru_gates_kernel(const T* __restrict__ u, const T* __restrict__ w,
                                                       const float* __restrict__ bias, const float* __restrict__ rate,
                                                       float* __restrict__ a_out, float* __restrict__ x_out, int T_tokens,
                                                       int width, int bw) {
    __shared__ float u_s[LRU_ROWS][LRU_PIECE];
    const int per_block = (bw + 63) / 64;
    const int b = blockIdx.x / per_block, c = (blockIdx.x - b * per_block) * 64 + threadIdx.x;
    const int t0 = blockIdx.y * LRU_ROWS;
    const bool ok = c < bw;
    const T* wr = w + ((size_t)(b * 2) * bw + (ok ? c : 0)) * bw;
    const T* wi = wr + (size_t)bw * bw;
    float lr[LRU_ROWS], li[LRU_ROWS];
#pragma unroll
    for (int m = 0; m < LRU_ROWS; ++m) lr[m] = li[m] = 0.f;
    for (int k0 = 0; k0 < bw; k0 += LRU_PIECE) {
        const int nk = min(LRU_PIECE, bw - k0);
        __syncthreads();
        for (int m = 0; m < LRU_ROWS; ++m)
            for (int k = threadIdx.x; k < nk; k += 64)
                u_s[m][k] = t0 + m < T_tokens ? to_f(u[(size_t)(t0 + m) * width + (size_t)b * bw + k0 + k]) : 0.f;
        __syncthreads();
        for (int k = 0; k < nk; ++k) {
            const float r = to_f(wr[k0 + k]), i = to_f(wi[k0 + k]);
#pragma unroll
            for (int m = 0; m < LRU_ROWS; ++m) {
                lr[m] = fmaf(r, u_s[m][k], lr[m]);
                li[m] = fmaf(i, u_s[m][k], li[m]);
            }
        }
    }
    if (!ok) return;
    const int ch = b * bw + c;
    for (int m = 0; m < LRU_ROWS; ++m) {
        const int t = t0 + m;
        if (t >= T_tokens) break;
        float a, x;
        lru_decay_input(lr[m] + bias[ch], li[m] + bias[width + ch], rate[ch], to_f(u[(size_t)t * width + ch]), a, x);
        a_out[(size_t)t * width + ch] = a;
        x_out[(size_t)t * width + ch] = x;
    }
}

// Place of chunk j of request s (rows base ..) among the chunks' summaries: distinct for all chunks of a step, below
// T / CH + number of requests + 1.
__device__ __forceinline__ size_t lru_place(int base, int s, int CH, int j) { return (size_t)(base / CH) + s + j; }

#define LRU_AHEAD 8              // rows whose reads are on their way together
__global__ __launch_bounds__(256) void lru_carry_kernel(const float* __restrict__ a, const float* __restrict__ x,
                                                        const float* __restrict__ S, const int* __restrict__ cu_q,
                                                        const int* __restrict__ slot_ids, float* __restrict__ P,
                                                        float* __restrict__ E, int width, int CH) {
    const int s = blockIdx.y, base = cu_q[s], q_len = cu_q[s + 1] - base;
    const int j = blockIdx.x, first = j * CH;
    const int c = blockIdx.z * 256 + threadIdx.x;
    if (first >= q_len || c >= width) return;
    const size_t at = lru_place(base, s, CH, j) * width + c;
    float p = 1.f, e = 0.f;
    if (j == 0) p = e = S[(size_t)slot_ids[s] * width + c];
    const int last = min(first + CH, q_len);
    if (last < q_len) {                                  // (nothing follows the last chunk)
        for (int t = first; t < last; t += LRU_AHEAD) {
            float av[LRU_AHEAD], xv[LRU_AHEAD];
#pragma unroll
            for (int m = 0; m < LRU_AHEAD; ++m) {
                const size_t r = (size_t)(base + min(t + m, last - 1)) * width + c;
                av[m] = a[r];
                xv[m] = x[r];
            }
#pragma unroll
            for (int m = 0; m < LRU_AHEAD; ++m)
                if (t + m < last) {
                    e = fmaf(av[m], e, xv[m]);
                    if (j > 0) p *= av[m];
                }
        }
    }
    P[at] = p;                                           // (of the first chunk: the old state)
    E[at] = e;
}

template <typename T>
__global__ __launch_bounds__(256) void lru_scan_kernel(const float* __restrict__ a, const float* __restrict__ x,
                                                       float* __restrict__ S, const int* __restrict__ cu_q,
                                                       const int* __restrict__ slot_ids, const float* __restrict__ P,
                                                       const float* __restrict__ E, const T* __restrict__ y, long long ld_y,
                                                       const float* __restrict__ y_bias, float out_scale,
                                                       T* __restrict__ out, long long ld_out, int width_out, int width,
                                                       int CH) {
    const int s = blockIdx.y, base = cu_q[s], q_len = cu_q[s + 1] - base;
    const int j = blockIdx.x, first = j * CH;
    const int c = blockIdx.z * 256 + threadIdx.x;
    if (first >= q_len || c >= width_out) return;
    const int last = min(first + CH, q_len);
    if (c >= width) {                                    // columns beyond the recurrence's
        for (int t = first; t < last; ++t) out[(size_t)(base + t) * ld_out + c] = from_f<T>(0.f);
        return;
    }
    float* Sp = S + (size_t)slot_ids[s] * width + c;
    float st;
    if (P == nullptr) {                                  // one chunk: nobody else touches this state
        st = *Sp;
    } else {
        const size_t at = lru_place(base, s, CH, 0) * width + c;
        st = j == 0 ? P[at] : E[at];
        for (int i = 1; i < j; i += LRU_AHEAD) {
            float pv[LRU_AHEAD], ev[LRU_AHEAD];
#pragma unroll
            for (int m = 0; m < LRU_AHEAD; ++m) {
                const size_t q = at + (size_t)min(i + m, j - 1) * width;
                pv[m] = P[q];
                ev[m] = E[q];
            }
#pragma unroll
            for (int m = 0; m < LRU_AHEAD; ++m)
                if (i + m < j) st = fmaf(pv[m], st, ev[m]);
        }
    }
    const float yb = y_bias[c];
    for (int t = first; t < last; t += LRU_AHEAD) {
        float av[LRU_AHEAD], xv[LRU_AHEAD], yv[LRU_AHEAD];
#pragma unroll
        for (int m = 0; m < LRU_AHEAD; ++m) {
            const int row = base + min(t + m, last - 1);
            av[m] = a[(size_t)row * width + c];
            xv[m] = x[(size_t)row * width + c];
            yv[m] = to_f(y[(size_t)row * ld_y + c]);
        }
#pragma unroll
        for (int m = 0; m < LRU_AHEAD; ++m)
            if (t + m < last) {
                st = fmaf(av[m], st, xv[m]);
                out[(size_t)(base + t + m) * ld_out + c] = from_f<T>(st * lru_gelu(yv[m] + yb) * out_scale);
            }
    }
    if (last == q_len) *Sp = st;
}

// Rows of a chunk: 32, more where a request of that many rows would make more than 64 chunks.
extern "C" int ra_channel_recurrence_chunk(int max_q_len) {
    int ch = 32;
    while ((long long)ch * 64 < max_q_len) ch *= 2;
    return ch;
}
// Whether the gates run on the matrix cores (and a step of single tokens is one kernel that needs no scratch).
extern "C" int ra_channel_recurrence_mfma(int width, int bw, int dtype) {
    return dtype == RA_DTYPE_BF16 && bw % 8 == 0 && width % 8 == 0 ? 1 : 0;
}

// u [T, width] storage type, contiguous; w [blocks][2][bw][bw] (gate r, gate i; rows are outputs); bias fp32 [2][width];
// rate fp32 [width]; y rows of ld_y; y_bias fp32 [width]; S fp32 [slots, width]; out rows of ld_out elements, width_out
// columns of which those from width on become zeros. scratch fp32: 2 T width for the decays and inputs, then, when the
// step has a request of more than one chunk, 2 (T / CH + n_seqs + 1) width for the chunks' summaries; null where every
// request brings one row and ra_channel_recurrence_mfma says so.
extern "C" int ra_channel_recurrence(const void* u, const void* w, const float* bias, const float* rate, const void* y,
                                     long long ld_y, const float* y_bias, float* S, const int* cu_q, const int* slot_ids,
                                     float* scratch, float out_scale, void* out, long long ld_out, int width_out,
                                     int n_seqs, int T_tokens, int max_q_len, int width, int blocks, int dtype,
                                     void* stream) {
    if (n_seqs <= 0 || T_tokens <= 0) return RA_OK;
    if (width < 1 || blocks < 1 || width % blocks || width_out < width || ld_y < width || ld_out < width_out ||
        n_seqs > 65535 || max_q_len < 1 || (width_out + 255) / 256 > 65535)
        return RA_ERR_ARG;
    if (dtype != RA_DTYPE_F32 && dtype != RA_DTYPE_BF16) return RA_ERR_ARG;
    const int bw = width / blocks;
    hipStream_t st = (hipStream_t)stream;
    bool mfma = ra_channel_recurrence_mfma(width, bw, dtype) != 0 && ((uintptr_t)u & 15) == 0 && ((uintptr_t)w & 15) == 0;
    const bool single = max_q_len == 1 && T_tokens == n_seqs;
    const bool step = mfma && single && ld_y % 4 == 0 && ld_out % 4 == 0 && ((uintptr_t)y & 7) == 0 && ((uintptr_t)out & 7) == 0;
    LruStep sx = {S, slot_ids, (const bf16*)y, ld_y, y_bias, out_scale, (bf16*)out, ld_out, width_out};
    float* a = scratch;
    float* x = scratch != nullptr ? scratch + (size_t)T_tokens * width : nullptr;
    if (!step && scratch == nullptr) return RA_ERR_ARG;
    if (mfma) {
        const int n_tiles = blocks * ((bw + 15) / 16);
        // as many rows a wave as still leave enough waves for the chip
        int rt = 1;
        while (rt < 4 && (long long)n_tiles * ((T_tokens + 32 * rt - 1) / (32 * rt)) >= 2048 && T_tokens > 16 * rt) rt *= 2;
        const int row_tiles = (T_tokens + 16 * rt - 1) / (16 * rt);
        if (row_tiles > 65535) return RA_ERR_ARG;
        const int waves = (long long)n_tiles * row_tiles <= 1024 ? 1 : 4;
        dim3 grid((n_tiles + waves - 1) / waves, row_tiles), block(64 * waves);
#define LRU_GO(RT_, STEP_)                                                                                            \
    hipLaunchKernelGGL((lru_gates_mfma_kernel<RT_, STEP_>), grid, block, 0, st, (const bf16*)u, (const bf16*)w, bias, rate, \
                       a, x, T_tokens, width, bw, n_tiles, sx)
        if (step) {
            if (rt == 1) LRU_GO(1, true); else if (rt == 2) LRU_GO(2, true); else LRU_GO(4, true);
            return ra_launch_status();
        }
        if (rt == 1) LRU_GO(1, false); else if (rt == 2) LRU_GO(2, false); else LRU_GO(4, false);
#undef LRU_GO
    } else {
        dim3 grid(blocks * ((bw + 63) / 64), (T_tokens + LRU_ROWS - 1) / LRU_ROWS);
        if (grid.y > 65535) return RA_ERR_ARG;
        if (dtype == RA_DTYPE_F32)
            hipLaunchKernelGGL(lru_gates_kernel<float>, grid, dim3(64), 0, st, (const float*)u, (const float*)w, bias, rate, a,
                               x, T_tokens, width, bw);
        else
            hipLaunchKernelGGL(lru_gates_kernel<bf16>, grid, dim3(64), 0, st, (const bf16*)u, (const bf16*)w, bias, rate, a, x,
                               T_tokens, width, bw);
    }
    if (hipGetLastError() != hipSuccess) return RA_ERR_LAUNCH;
    const int CH = ra_channel_recurrence_chunk(max_q_len);
    const int chunks = (max_q_len + CH - 1) / CH;
    float* P = nullptr;
    float* E = nullptr;
    dim3 grid(chunks, n_seqs, (width_out + 255) / 256), block(256);
    if (chunks > 1) {
        P = x + (size_t)T_tokens * width;
        E = P + ((size_t)T_tokens / CH + n_seqs + 1) * width;
        hipLaunchKernelGGL(lru_carry_kernel, grid, block, 0, st, a, x, S, cu_q, slot_ids, P, E, width, CH);
        if (hipGetLastError() != hipSuccess) return RA_ERR_LAUNCH;
    }
    if (dtype == RA_DTYPE_F32)
        hipLaunchKernelGGL(lru_scan_kernel<float>, grid, block, 0, st, a, x, S, cu_q, slot_ids, P, E, (const float*)y, ld_y,
                           y_bias, out_scale, (float*)out, ld_out, width_out, width, CH);
    else
        hipLaunchKernelGGL(lru_scan_kernel<bf16>, grid, block, 0, st, a, x, S, cu_q, slot_ids, P, E, (const bf16*)y, ld_y,
                           y_bias, out_scale, (bf16*)out, ld_out, width_out, width, CH);
    return ra_launch_status();
}
