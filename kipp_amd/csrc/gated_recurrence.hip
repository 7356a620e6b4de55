// The real-gated linear recurrent unit behind a short causal filter (Griffin's recurrent block): a vector state a request,
// carried from token to token in float32 in the request's slot.
//
//     u = filter(x + x_bias) + filter_bias      a causal filter a channel over the last `taps` inputs
//     r = sigmoid(R_b u_b + r_bias), i = sigmoid(I_b u_b + i_bias)      in each of `blocks` equal parts b of the channels
//     a = exp(-r decay),  decay = factor * softplus(lam)
//     S_t = a S_(t-1) + sqrt(1 - a^2) i u;     out = S gelu_tanh(y + y_bias)
//
// `filter` makes u and `keep` moves the slot's last inputs on; `gates` multiplies every part of u by its two square
// matrices and leaves (a, sqrt(1 - a^2) i u) a number; `scan` walks the tokens; `step` is all of it for single tokens in one
// launch.  Everything is float32: on the matrix cores u goes in as three bfloat16 numbers whose sum is u (8 bits of it each),
// so that a product of u and a bfloat16 matrix is the float32 one, summed in float32.
//
// Slot: S [width], then a ring of the last `taps` inputs [taps][width] (with their bias): the input of position p lies at
// p % taps.  A token reads positions p - taps + 1 .. p - 1 and a single token writes only its own, so that no workgroup of
// `step` overwrites what another still reads.
#include "common.h"
#include <math.h>

#define THREADS 256
#define MAX_TAPS 16

typedef __attribute__((ext_vector_type(8))) __bf16 bf16x8;
typedef __attribute__((ext_vector_type(4))) float f32x4;
typedef __attribute__((ext_vector_type(4))) uint32_t u32x4;
union Frag {
    u32x4 u;
    bf16x8 v;
    bf16_t e[8];
};

__device__ __forceinline__ float sigmoid_f(float z) { return 1.0f / (1.0f + expf(-z)); }
// 0.5 z (1 + tanh(w)) = z / (1 + e^(-2 w))
__device__ __forceinline__ float gelu_tanh_f(float z) {
    const float w = 0.79788456080286535588f * (z + 0.044715f * z * z * z);
    return z / (1.0f + expf(-2.0f * w));
}

// (a, sqrt(1 - a^2) i u) from the two gates' sums (biases added).
__device__ __forceinline__ float2 recurrence_terms(float zr, float zi, float decay, float u) {
    const float log_a = -decay * sigmoid_f(zr);
    return make_float2(expf(log_a), sqrtf(-expm1f(2.0f * log_a)) * (sigmoid_f(zi) * u));
}

struct Filter {
    const float* proj;          // [tokens][stride], the filter's inputs from column x_at on
    int stride, x_at;
    const float* x_bias;        // [width]
    const float* w;             // [taps][width], the last tap is the current token's
    const float* b;             // [width]
    int taps, width;
};

// u of token row t at position p, channel c; `first` is the row of its entry's first token, `ring` the slot's kept inputs.
__device__ __forceinline__ float filter_at(const Filter& f, int t, int first, int p, const float* __restrict__ ring, int c) {
    float y = f.b[c];
    const float xb = f.x_bias[c];
    for (int j = 0; j < f.taps; ++j) {
        const int back = f.taps - 1 - j;
        float in = 0.0f;
        if (t - back >= first) in = f.proj[(size_t)(t - back) * f.stride + f.x_at + c] + xb;
        else if (p - back >= 0) in = ring[(size_t)((p - back) % f.taps) * f.width + c];
        y = fmaf(f.w[(size_t)j * f.width + c], in, y);
    }
    return y;
}

__global__ void __launch_bounds__(THREADS)
filter_kernel(Filter f, const float* __restrict__ state, size_t state_stride, const int32_t* __restrict__ positions,
              const int32_t* __restrict__ seq_of_token, const int32_t* __restrict__ q_start, const int32_t* __restrict__ slots,
              float* __restrict__ u) {
    const int t = blockIdx.x, c = blockIdx.y * THREADS + threadIdx.x;
    if (c >= f.width) return;
    const int entry = seq_of_token[t];
    const float* ring = state + (size_t)slots[entry] * state_stride + f.width;
    u[(size_t)t * f.width + c] = filter_at(f, t, q_start[entry], positions[t], ring, c);
}

// The slot's ring after a portion: its last `taps` inputs (as many as the portion has) at their positions' places.
__global__ void __launch_bounds__(THREADS)
keep_kernel(Filter f, float* __restrict__ state, size_t state_stride, const int32_t* __restrict__ positions,
            const int32_t* __restrict__ q_start, const int32_t* __restrict__ q_len, const int32_t* __restrict__ slots) {
    const int entry = blockIdx.y, c = blockIdx.x * THREADS + threadIdx.x;
    if (c >= f.width) return;
    const int first = q_start[entry], n = q_len[entry];
    float* ring = state + (size_t)slots[entry] * state_stride + f.width;
    const float xb = f.x_bias[c];
    for (int i = max(0, n - f.taps); i < n; ++i)
        ring[(size_t)(positions[first + i] % f.taps) * f.width + c] = f.proj[(size_t)(first + i) * f.stride + f.x_at + c] + xb;
}

// ---- the gates, plain: any size, float32 or bfloat16 matrices [blocks][size in][2 size out] (r's columns, then i's).  A
// thread takes one column of both gates for four tokens; every sum runs over the part's numbers in order.
#define PLAIN_TOKENS 16
#define PLAIN_COLS 64
#define PLAIN_KC 128

template <typename TW>
__global__ void __launch_bounds__(THREADS)
gates_kernel(const float* __restrict__ u, const TW* __restrict__ w, const float* __restrict__ r_bias, const float* __restrict__ i_bias,
             const float* __restrict__ decay, float2* __restrict__ terms, int tokens, int width, int size) {
    __shared__ float u_s[PLAIN_TOKENS][PLAIN_KC];
    const int t0 = blockIdx.x * PLAIN_TOKENS, block = blockIdx.y;
    const int col = blockIdx.z * PLAIN_COLS + (threadIdx.x & (PLAIN_COLS - 1)), tg = threadIdx.x / PLAIN_COLS * 4;
    const TW* w_b = w + (size_t)block * size * 2 * size;
    float zr[4] = {0.0f, 0.0f, 0.0f, 0.0f}, zi[4] = {0.0f, 0.0f, 0.0f, 0.0f};
    for (int k0 = 0; k0 < size; k0 += PLAIN_KC) {
        const int kc = min(PLAIN_KC, size - k0);
        __syncthreads();
        for (int i = threadIdx.x; i < PLAIN_TOKENS * PLAIN_KC; i += THREADS) {
            const int r = i / PLAIN_KC, e = i - r * PLAIN_KC;
            u_s[r][e] = t0 + r < tokens && e < kc ? u[(size_t)(t0 + r) * width + block * size + k0 + e] : 0.0f;
        }
        __syncthreads();
        if (col < size)
            for (int e = 0; e < kc; ++e) {
                const float wr = load_f(w_b, (size_t)(k0 + e) * 2 * size + col), wi = load_f(w_b, (size_t)(k0 + e) * 2 * size + size + col);
#pragma unroll
                for (int j = 0; j < 4; ++j) {
                    zr[j] = fmaf(wr, u_s[tg + j][e], zr[j]);
                    zi[j] = fmaf(wi, u_s[tg + j][e], zi[j]);
                }
            }
    }
    if (col >= size) return;
    const int c = block * size + col;
#pragma unroll
    for (int j = 0; j < 4; ++j) {
        const int t = t0 + tg + j;
        if (t < tokens) terms[(size_t)t * width + c] = recurrence_terms(zr[j] + r_bias[c], zi[j] + i_bias[c], decay[c], u[(size_t)t * width + c]);
    }
}

// u as three bfloat16 numbers: the nearest, the nearest to what is left, and once more.
__device__ __forceinline__ void split3(float v, bf16_t& hi, bf16_t& mid, bf16_t& lo) {
    hi = f32_to_bf16(v);
    v -= bf16_to_f32(hi);
    mid = f32_to_bf16(v);
    v -= bf16_to_f32(mid);
    lo = f32_to_bf16(v);
}

// ---- the gates on the matrix cores: bfloat16 matrices [blocks][2][size out][size in], size a multiple of 8.  A workgroup
// takes 64 tokens and 64 columns of a part, a wave 32 of either with both gates; steps of 32 numbers of the part come
// through LDS, the next one on its way from memory while this one is multiplied.  A 16 x 16 x 32 product takes, from lane l,
// 8 numbers of row l % 16 at k = 8 (l / 16) .. + 7 of either operand, and leaves C[4 (l / 16) + v][l % 16] in its register v.
#define GT 64
#define GC 64
#define GK 32
#define GPITCH 40       // bfloat16 numbers from a row to the next in LDS

__global__ void __launch_bounds__(THREADS)
gates_mfma_kernel(const float* __restrict__ u, const bf16_t* __restrict__ w, const float* __restrict__ r_bias,
                  const float* __restrict__ i_bias, const float* __restrict__ decay, float2* __restrict__ terms, int tokens, int width,
                  int size) {
    __shared__ __attribute__((aligned(16))) bf16_t a_s[3][GT * GPITCH];
    __shared__ __attribute__((aligned(16))) bf16_t b_s[2][GC * GPITCH];
    const int t0 = blockIdx.x * GT, block = blockIdx.y, c0 = blockIdx.z * GC;
    const int tid = threadIdx.x, wave = tid / KIPP_WAVE, lane = tid & (KIPP_WAVE - 1), l16 = lane & 15, h = lane >> 4;
    const int wt = (wave & 1) * 32, wc = (wave >> 1) * 32;      // the wave's tokens and columns
    const int ld_row = tid >> 2, ld_k = (tid & 3) * 8;          // from memory: 4 threads take a row's step
    const float* a_src = u + (size_t)min(t0 + ld_row, tokens - 1) * width + block * size + ld_k;
    const bf16_t* b_src = w + ((size_t)block * 2 * size + min(c0 + ld_row, size - 1)) * size + ld_k;
    const size_t b_next = (size_t)size * size;                  // from r's matrix to i's
    float4 a_r[2];
    u32x4 b_r[2];
    auto fetch = [&](int k0) {
        const bool there = k0 + ld_k < size;                    // the size is a multiple of 8: all of a thread's 8 numbers or none
        a_r[0] = a_r[1] = make_float4(0.0f, 0.0f, 0.0f, 0.0f);
        b_r[0] = b_r[1] = (u32x4){0u, 0u, 0u, 0u};
        if (there) {
            a_r[0] = *(const float4*)(a_src + k0);
            a_r[1] = *(const float4*)(a_src + k0 + 4);
            b_r[0] = *(const u32x4*)(b_src + k0);
            b_r[1] = *(const u32x4*)(b_src + b_next + k0);
        }
    };
    f32x4 acc[2][2][2];         // [token fragment][gate][column fragment]
#pragma unroll
    for (int i = 0; i < 8; ++i) acc[i >> 2][(i >> 1) & 1][i & 1] = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    fetch(0);
    for (int k0 = 0; k0 < size; k0 += GK) {
        __syncthreads();        // the step before has been multiplied
        {
            const float v[8] = {a_r[0].x, a_r[0].y, a_r[0].z, a_r[0].w, a_r[1].x, a_r[1].y, a_r[1].z, a_r[1].w};
            Frag s[3];
#pragma unroll
            for (int e = 0; e < 8; ++e) split3(v[e], s[0].e[e], s[1].e[e], s[2].e[e]);
#pragma unroll
            for (int p = 0; p < 3; ++p) *(u32x4*)(a_s[p] + ld_row * GPITCH + ld_k) = s[p].u;
#pragma unroll
            for (int g = 0; g < 2; ++g) *(u32x4*)(b_s[g] + ld_row * GPITCH + ld_k) = b_r[g];
        }
        __syncthreads();
        if (k0 + GK < size) fetch(k0 + GK);
        Frag b[2][2];
#pragma unroll
        for (int g = 0; g < 2; ++g)
#pragma unroll
            for (int j = 0; j < 2; ++j) b[g][j].u = *(const u32x4*)(b_s[g] + (wc + 16 * j + l16) * GPITCH + 8 * h);
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int p = 2; p >= 0; --p) {      // the smallest part first
                Frag a;
                a.u = *(const u32x4*)(a_s[p] + (wt + 16 * i + l16) * GPITCH + 8 * h);
#pragma unroll
                for (int g = 0; g < 2; ++g)
#pragma unroll
                    for (int j = 0; j < 2; ++j) acc[i][g][j] = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b[g][j].v, acc[i][g][j], 0, 0, 0);
            }
    }
#pragma unroll
    for (int j = 0; j < 2; ++j) {
        const int col = c0 + wc + 16 * j + l16;
        if (col >= size) continue;
        const int c = block * size + col;
        const float rb = r_bias[c], ib = i_bias[c], dc = decay[c];
#pragma unroll
        for (int i = 0; i < 2; ++i)
#pragma unroll
            for (int v = 0; v < 4; ++v) {
                const int t = t0 + wt + 16 * i + 4 * h + v;
                if (t < tokens) {
                    const size_t at = (size_t)t * width + c;
                    terms[at] = recurrence_terms(acc[i][0][j][v] + rb, acc[i][1][j][v] + ib, dc, u[at]);
                }
            }
    }
}

// ---- the walk: a workgroup takes (entry, 16 channels); 64 tokens of terms come through LDS at a time, 16 lanes walk them in
// order while the next 64 are on their way into registers, then every thread multiplies by the other branch and writes.
#define SCAN_CH 16
#define SCAN_T 64
#define SCAN_N (SCAN_T * SCAN_CH / THREADS)

template <typename TO>
__global__ void __launch_bounds__(THREADS)
scan_kernel(const float2* __restrict__ terms, const float* __restrict__ proj, int stride, int y_at, const float* __restrict__ y_bias,
            float* __restrict__ state, size_t state_stride, const int32_t* __restrict__ q_start, const int32_t* __restrict__ q_len,
            const int32_t* __restrict__ slots, TO* __restrict__ out, int width) {
    __shared__ float2 in_s[SCAN_T * SCAN_CH];
    __shared__ float s_s[SCAN_T * SCAN_CH];
    const int entry = blockIdx.y;
    const int ch = threadIdx.x & (SCAN_CH - 1), tt = threadIdx.x / SCAN_CH;
    const int c = min(blockIdx.x * SCAN_CH + ch, width - 1);
    const bool live = blockIdx.x * SCAN_CH + ch < width;
    const int first = q_start[entry], n = q_len[entry];
    float* s_at = state + (size_t)slots[entry] * state_stride + c;
    const bool walks = threadIdx.x < SCAN_CH;
    float S = walks ? *s_at : 0.0f;
    const float yb = y_bias[c];
    float2 in_r[SCAN_N];
    float y_r[SCAN_N], y_now[SCAN_N];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int j = 0; j < SCAN_N; ++j) {
            const int t = t0 + tt + j * (THREADS / SCAN_CH);
            if (t < n) {
                in_r[j] = terms[(size_t)(first + t) * width + c];
                y_r[j] = proj[(size_t)(first + t) * stride + y_at + c];
            }
        }
    };
    fetch(0);
    for (int t0 = 0; t0 < n; t0 += SCAN_T) {
        const int m = min(SCAN_T, n - t0);
        // (what the walkers read last round lies behind the barrier in front of the write-out)
#pragma unroll
        for (int j = 0; j < SCAN_N; ++j) {
            in_s[threadIdx.x + j * THREADS] = in_r[j];
            y_now[j] = y_r[j];
        }
        __syncthreads();
        fetch(t0 + SCAN_T);
        if (walks) {
            int t = 0;
            for (; t + 8 <= m; t += 8) {
                float2 v[8];
#pragma unroll
                for (int e = 0; e < 8; ++e) v[e] = in_s[(t + e) * SCAN_CH + ch];
#pragma unroll
                for (int e = 0; e < 8; ++e) {
                    S = fmaf(v[e].x, S, v[e].y);
                    s_s[(t + e) * SCAN_CH + ch] = S;
                }
            }
            for (; t < m; ++t) {
                const float2 v = in_s[t * SCAN_CH + ch];
                S = fmaf(v.x, S, v.y);
                s_s[t * SCAN_CH + ch] = S;
            }
        }
        __syncthreads();
#pragma unroll
        for (int j = 0; j < SCAN_N; ++j) {
            const int t = t0 + tt + j * (THREADS / SCAN_CH);
            if (t < n && live) store_f(out, (size_t)(first + t) * width + c, s_s[threadIdx.x + j * THREADS] * gelu_tanh_f(y_now[j] + yb));
        }
    }
    if (walks && live) *s_at = S;
}

// ---- single tokens in one launch: a workgroup takes 16 columns of a part for 16 tokens.  It filters the part's inputs
// into LDS as three bfloat16 planes (256 numbers of the part at a time), its four waves multiply them by the 16 rows of the
// two matrices (a wave a gate and every second step of 32), and every thread ends one (token, column): terms, state, ring, output.
#define STEP_ROWS 16
#define STEP_COLS 16
#define STEP_KC 256
#define STEP_PITCH (STEP_KC + 8)

template <typename TO>
__global__ void __launch_bounds__(THREADS)
step_kernel(Filter f, int y_at, const float* __restrict__ y_bias, const bf16_t* __restrict__ w, const float* __restrict__ r_bias,
            const float* __restrict__ i_bias, const float* __restrict__ decay, float* __restrict__ state, size_t state_stride,
            const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_of_token, const int32_t* __restrict__ slots,
            TO* __restrict__ out, int tokens, int size, int col_tiles) {
    __shared__ __attribute__((aligned(16))) bf16_t a_s[3][STEP_ROWS * STEP_PITCH];
    __shared__ float red[4][STEP_ROWS * STEP_COLS];
    const int block = blockIdx.x / col_tiles, c0 = (blockIdx.x - block * col_tiles) * STEP_COLS;
    const int t0 = blockIdx.y * STEP_ROWS, rows = min(STEP_ROWS, tokens - t0);
    const int tid = threadIdx.x, wave = tid / KIPP_WAVE, lane = tid & (KIPP_WAVE - 1), l16 = lane & 15, h = lane >> 4;
    const int gate = wave & 1, half = wave >> 1;
    const bf16_t* w_row = w + ((size_t)(block * 2 + gate) * size + min(c0 + l16, size - 1)) * size + 8 * h;
    f32x4 acc = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    for (int k0 = 0; k0 < size; k0 += STEP_KC) {
        Frag b[STEP_KC / 64];       // the weights are asked for first
#pragma unroll
        for (int s = 0; s < STEP_KC / 64; ++s) {
            const int k = k0 + 32 * (2 * s + half);
            b[s].u = k + 8 * h < size ? *(const u32x4*)(w_row + k) : (u32x4){0u, 0u, 0u, 0u};
        }
        __syncthreads();            // the numbers before have been multiplied
        {
            const int c = block * size + k0 + tid;
            const bool there = k0 + tid < size;
#pragma unroll 4
            for (int r = 0; r < STEP_ROWS; ++r) {
                float v = 0.0f;
                if (there && r < rows) {
                    const int t = t0 + r;
                    v = filter_at(f, t, t, positions[t], state + (size_t)slots[seq_of_token[t]] * state_stride + f.width, c);
                }
                bf16_t hi, mid, lo;
                split3(v, hi, mid, lo);
                a_s[0][r * STEP_PITCH + tid] = hi;
                a_s[1][r * STEP_PITCH + tid] = mid;
                a_s[2][r * STEP_PITCH + tid] = lo;
            }
        }
        __syncthreads();
#pragma unroll
        for (int s = 0; s < STEP_KC / 64; ++s) {
            const int k = 32 * (2 * s + half);
            if (k0 + k < size) {
#pragma unroll
                for (int p = 2; p >= 0; --p) {
                    Frag a;
                    a.u = *(const u32x4*)(a_s[p] + l16 * STEP_PITCH + k + 8 * h);
                    acc = __builtin_amdgcn_mfma_f32_16x16x32_bf16(a.v, b[s].v, acc, 0, 0, 0);
                }
            }
        }
    }
#pragma unroll
    for (int v = 0; v < 4; ++v) red[wave][(4 * h + v) * STEP_COLS + l16] = acc[v];
    __syncthreads();
    const int r = tid / STEP_COLS, col = c0 + (tid & (STEP_COLS - 1));
    if (r >= rows || col >= size) return;
    const int t = t0 + r, c = block * size + col, p = positions[t];
    float* slot = state + (size_t)slots[seq_of_token[t]] * state_stride;
    float* ring = slot + f.width;
    const float u = filter_at(f, t, t, p, ring, c);
    const float2 v = recurrence_terms(red[0][tid] + red[2][tid] + r_bias[c], red[1][tid] + red[3][tid] + i_bias[c], decay[c], u);
    const float S = fmaf(v.x, slot[c], v.y);
    slot[c] = S;
    const float* row = f.proj + (size_t)t * f.stride;
    ring[(size_t)(p % f.taps) * f.width + c] = row[f.x_at + c] + f.x_bias[c];
    store_f(out, (size_t)t * f.width + c, S * gelu_tanh_f(row[y_at + c] + y_bias[c]));
}

extern "C" {

// u [tokens][width] from proj's columns x_at .. x_at + width - 1; the slot's ring of inputs is then moved on by every entry.
int kipp_recurrence_filter(const float* proj, int stride, int x_at, const float* x_bias, const float* conv_w, const float* conv_b,
                           int taps, int width, float* state, size_t state_stride, const int32_t* positions,
                           const int32_t* seq_of_token, const int32_t* q_start, const int32_t* q_len, const int32_t* slots, float* u,
                           int tokens, int entries, hipStream_t stream) {
    if (tokens <= 0) return 0;
    if (taps < 1 || taps > MAX_TAPS || width <= 0 || stride < x_at + width || state_stride < (size_t)(1 + taps) * width) return -1;
    const Filter f = {proj, stride, x_at, x_bias, conv_w, conv_b, taps, width};
    const int cols = (width + THREADS - 1) / THREADS;
    hipLaunchKernelGGL(filter_kernel, dim3(tokens, cols), dim3(THREADS), 0, stream, f, (const float*)state, state_stride, positions,
                       seq_of_token, q_start, slots, u);
    hipLaunchKernelGGL(keep_kernel, dim3(cols, entries), dim3(THREADS), 0, stream, f, state, state_stride, positions, q_start, q_len, slots);
    return KIPP_LAUNCH_CHECK();
}

// terms [tokens][width] (a, sqrt(1 - a^2) i u).  `mfma`: w is bfloat16 [blocks][2][size out][size in], size a multiple of 8;
// else w is [blocks][size in][2 size out].
int kipp_recurrence_gates(const float* u, const void* w, int w_dtype, int mfma, const float* r_bias, const float* i_bias,
                          const float* decay, float* terms, int tokens, int width, int blocks, hipStream_t stream) {
    if (tokens <= 0) return 0;
    if (blocks <= 0 || width <= 0 || width % blocks) return -1;
    const int size = width / blocks;
    if (mfma) {
        if (w_dtype != KIPP_BF16 || size % 8) return -1;
        hipLaunchKernelGGL(gates_mfma_kernel, dim3((tokens + GT - 1) / GT, blocks, (size + GC - 1) / GC), dim3(THREADS), 0, stream, u,
                           (const bf16_t*)w, r_bias, i_bias, decay, (float2*)terms, tokens, width, size);
        return KIPP_LAUNCH_CHECK();
    }
    dim3 grid((tokens + PLAIN_TOKENS - 1) / PLAIN_TOKENS, blocks, (size + PLAIN_COLS - 1) / PLAIN_COLS);
    if (w_dtype == KIPP_F32)
        hipLaunchKernelGGL(gates_kernel<float>, grid, dim3(THREADS), 0, stream, u, (const float*)w, r_bias, i_bias, decay, (float2*)terms,
                           tokens, width, size);
    else if (w_dtype == KIPP_BF16)
        hipLaunchKernelGGL(gates_kernel<bf16_t>, grid, dim3(THREADS), 0, stream, u, (const bf16_t*)w, r_bias, i_bias, decay, (float2*)terms,
                           tokens, width, size);
    else
        return -2;
    return KIPP_LAUNCH_CHECK();
}

int kipp_recurrence_scan(const float* terms, const float* proj, int stride, int y_at, const float* y_bias, float* state,
                         size_t state_stride, const int32_t* q_start, const int32_t* q_len, const int32_t* slots, void* out, int out_dtype,
                         int entries, int width, hipStream_t stream) {
    if (entries <= 0) return 0;
    if (width <= 0 || stride < y_at + width || state_stride < (size_t)width) return -1;
    dim3 grid((width + SCAN_CH - 1) / SCAN_CH, entries);
    if (out_dtype == KIPP_F32)
        hipLaunchKernelGGL(scan_kernel<float>, grid, dim3(THREADS), 0, stream, (const float2*)terms, proj, stride, y_at, y_bias, state,
                           state_stride, q_start, q_len, slots, (float*)out, width);
    else if (out_dtype == KIPP_BF16)
        hipLaunchKernelGGL(scan_kernel<bf16_t>, grid, dim3(THREADS), 0, stream, (const float2*)terms, proj, stride, y_at, y_bias, state,
                           state_stride, q_start, q_len, slots, (bf16_t*)out, width);
    else
        return -2;
    return KIPP_LAUNCH_CHECK();
}

// Filter, gates, walk and output of a batch in which every entry brings one token; w as for `mfma` above.
int kipp_recurrence_step(const float* proj, int stride, int y_at, int x_at, const float* y_bias, const float* x_bias, const float* conv_w,
                         const float* conv_b, int taps, const void* w, const float* r_bias, const float* i_bias, const float* decay,
                         float* state, size_t state_stride, const int32_t* positions, const int32_t* seq_of_token, const int32_t* slots,
                         void* out, int out_dtype, int tokens, int width, int blocks, hipStream_t stream) {
    if (tokens <= 0) return 0;
    if (taps < 1 || taps > MAX_TAPS || width <= 0 || blocks <= 0 || width % blocks || (width / blocks) % 8) return -1;
    if (stride < x_at + width || stride < y_at + width || state_stride < (size_t)(1 + taps) * width) return -1;
    const int size = width / blocks, col_tiles = (size + STEP_COLS - 1) / STEP_COLS;
    const Filter f = {proj, stride, x_at, x_bias, conv_w, conv_b, taps, width};
    dim3 grid(blocks * col_tiles, (tokens + STEP_ROWS - 1) / STEP_ROWS);
    if (out_dtype == KIPP_F32)
        hipLaunchKernelGGL(step_kernel<float>, grid, dim3(THREADS), 0, stream, f, y_at, y_bias, (const bf16_t*)w, r_bias, i_bias, decay,
                           state, state_stride, positions, seq_of_token, slots, (float*)out, tokens, size, col_tiles);
    else if (out_dtype == KIPP_BF16)
        hipLaunchKernelGGL(step_kernel<bf16_t>, grid, dim3(THREADS), 0, stream, f, y_at, y_bias, (const bf16_t*)w, r_bias, i_bias, decay,
                           state, state_stride, positions, seq_of_token, slots, (bf16_t*)out, tokens, size, col_tiles);
    else
        return -2;
    return KIPP_LAUNCH_CHECK();
}

}  // extern "C"
