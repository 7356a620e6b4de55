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
    __bf16 e[8];
};

// The reciprocal and the root within an ulp, in one instruction each: enough for everything below.
__device__ __forceinline__ float sigmoid_f(float z) { return __builtin_amdgcn_rcpf(1.0f + expf(-z)); }
// 0.5 z (1 + tanh(w)) = z / (1 + e^(-2 w))
__device__ __forceinline__ float gelu_tanh_f(float z) {
    const float w = 0.79788456080286535588f * (z + 0.044715f * z * z * z);
    return z * __builtin_amdgcn_rcpf(1.0f + expf(-2.0f * w));
}

// 1 - e^x for x <= 0: near zero the power series of e^x - 1 (nine terms: below half an ulp for x > -1/2), else the difference.
__device__ __forceinline__ float one_minus_exp(float x, float exp_x) {
    float s = 1.0f + x * (1.0f / 9.0f);
#pragma unroll
    for (int k = 8; k >= 2; --k) s = fmaf(s * x, 1.0f / (float)k, 1.0f);
    return x > -0.5f ? -x * s : 1.0f - exp_x;
}

// (a, sqrt(1 - a^2) i u) from the two gates' sums (biases added).
__device__ __forceinline__ float2 recurrence_terms(float zr, float zi, float decay, float u) {
    const float log_a = -decay * sigmoid_f(zr);
    const float a = expf(log_a);
    return make_float2(a, __builtin_amdgcn_sqrtf(one_minus_exp(2.0f * log_a, a * a)) * (sigmoid_f(zi) * u));
}

struct Filter {
    const float* proj;          // [tokens][stride], the filter's inputs from column x_at on
    int stride, x_at;
    const float* x_bias;        // [width]
    const float* w;             // [taps][width], the last tap is the current token's
    const float* b;             // [width]
    int taps, width;
};

// One channel's filter in registers.  TAPS: the number of taps if the build knows it, 0: whatever `f.taps` says.
template <int TAPS>
struct Channel {
    static constexpr int MOST = TAPS > 0 ? TAPS : MAX_TAPS;
    float w[MOST], b, xb;
    int c, taps;
    __device__ __forceinline__ Channel(const Filter& f, int channel) {
        c = channel;
        taps = TAPS > 0 ? TAPS : f.taps;
        b = f.b[c];
        xb = f.x_bias[c];
#pragma unroll
        for (int j = 0; j < MOST; ++j) w[j] = j < taps ? f.w[(size_t)j * f.width + c] : 0.0f;
    }
    // u of token row t at position p; `first` is the row of its entry's first token, `ring` the slot's kept inputs.
    __device__ __forceinline__ float at(const Filter& f, int t, int first, int p, const float* __restrict__ ring) const {
        const int turn = p % taps;
        float in[MOST];
#pragma unroll
        for (int j = 0; j < MOST; ++j) {        // every load is asked for before the first is used
            const int back = taps - 1 - j;
            in[j] = 0.0f;
            if (j < taps) {
                if (t - back >= first) in[j] = f.proj[(size_t)(t - back) * f.stride + f.x_at + c] + xb;
                else if (p - back >= 0) in[j] = ring[(size_t)(turn - back + (turn < back ? taps : 0)) * f.width + c];
            }
        }
        float y = b;
#pragma unroll
        for (int j = 0; j < MOST; ++j)
            if (j < taps) y = fmaf(w[j], in[j], y);
        return y;
    }
};

#define FILTER_TOKENS 8     // tokens a thread takes: its channel's taps are read once for them

template <int TAPS>
__global__ void __launch_bounds__(THREADS)
filter_kernel(Filter f, const float* __restrict__ state, size_t state_stride, const int32_t* __restrict__ positions,
              const int32_t* __restrict__ seq_of_token, const int32_t* __restrict__ q_start, const int32_t* __restrict__ slots,
              float* __restrict__ u, int tokens) {
    const int c = blockIdx.y * THREADS + threadIdx.x;
    if (c >= f.width) return;
    const Channel<TAPS> channel(f, c);
    const int t0 = blockIdx.x * FILTER_TOKENS, t1 = min(t0 + FILTER_TOKENS, tokens);
#pragma unroll(TAPS > 0 ? 4 : 1)
    for (int t = t0; t < t1; ++t) {
        const int entry = seq_of_token[t];
        const float* ring = state + (size_t)slots[entry] * state_stride + f.width;
        u[(size_t)t * f.width + c] = channel.at(f, t, q_start[entry], positions[t], ring);
    }
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

// u as three bfloat16 numbers: the nearest, the nearest to what is left, and once more (the conversions of the hardware).
__device__ __forceinline__ void split3(float v, __bf16& hi, __bf16& mid, __bf16& lo) {
    hi = (__bf16)v;
    v -= (float)hi;
    mid = (__bf16)v;
    v -= (float)mid;
    lo = (__bf16)v;
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

// ---- the walk: a workgroup takes (entry, 16 channels).  Its first wave walks a run of 196 tokens out of LDS in order (16
// lanes, a channel each), while the other seven bring the next run from registers into LDS, ask memory for the one after it, and
// multiply the run before by the other branch and write it: one barrier a run.
#define SCAN_CH 16
#define SCAN_T 196
#define SCAN_WG 512
#define SCAN_MOVERS (SCAN_WG - KIPP_WAVE)
#define SCAN_STEP (SCAN_MOVERS / SCAN_CH)       // tokens the movers take side by side
#define SCAN_N (SCAN_T / SCAN_STEP)

// Eight tokens of a channel: their terms (read ahead) into the state, one after the other.
__device__ __forceinline__ void walk8(float& S, const float2 (&v)[8], float* to) {
    float s[8];
#pragma unroll
    for (int e = 0; e < 8; ++e) s[e] = S = fmaf(v[e].x, S, v[e].y);
#pragma unroll
    for (int e = 0; e < 8; ++e) to[e * SCAN_CH] = s[e];
}

template <typename TO>
__global__ void __launch_bounds__(SCAN_WG)
scan_kernel(const float2* __restrict__ terms, const float* __restrict__ proj, int stride, int y_at, const float* __restrict__ y_bias,
            float* __restrict__ state, size_t state_stride, const int32_t* __restrict__ q_start, const int32_t* __restrict__ q_len,
            const int32_t* __restrict__ slots, TO* __restrict__ out, int width) {
    __shared__ float2 in_s[2][SCAN_T * SCAN_CH];
    __shared__ float s_s[2][SCAN_T * SCAN_CH];
    const int entry = blockIdx.y;
    const bool walker = threadIdx.x < KIPP_WAVE;
    const int mover = threadIdx.x - KIPP_WAVE;
    const int ch = (walker ? threadIdx.x : mover) & (SCAN_CH - 1), tt = mover / SCAN_CH;
    const int c = min(blockIdx.x * SCAN_CH + ch, width - 1);
    const bool live = blockIdx.x * SCAN_CH + ch < width;
    const int first = q_start[entry], n = q_len[entry];
    float* s_at = state + (size_t)slots[entry] * state_stride + c;
    const bool walks = threadIdx.x < SCAN_CH;
    float S = walks ? *s_at : 0.0f;
    const float yb = y_bias[c];
    float2 in_r[SCAN_N];
    float y_r[SCAN_N];
    auto fetch = [&](int t0) {
#pragma unroll
        for (int j = 0; j < SCAN_N; ++j) {
            const int t = min(t0 + tt + j * SCAN_STEP, n - 1);      // (beyond the entry: its last token, dropped; no branch around a load)
            in_r[j] = terms[(size_t)(first + t) * width + c];
        }
    };
    auto store = [&](float2* to) {
#pragma unroll
        for (int j = 0; j < SCAN_N; ++j) to[(tt + j * SCAN_STEP) * SCAN_CH + ch] = in_r[j];
    };
    const int runs = (n + SCAN_T - 1) / SCAN_T;
    if (!walker) {
        fetch(0);
        store(in_s[0]);
        fetch(SCAN_T);
    }
    for (int run = 0; run <= runs; ++run) {
        __syncthreads();        // run `run` lies in LDS, run `run - 1` has been walked
        if (walker) {
            if (walks && run < runs) {
                const float2* in = in_s[run & 1] + ch;
                float* to = s_s[run & 1] + ch;
                const int m = min(SCAN_T, n - run * SCAN_T);
                float2 even[8], odd[8];
                auto read = [&](float2 (&v)[8], int t) {
                    const float2* at = in + min(t, SCAN_T - 8) * SCAN_CH;      // (beyond the run: read again and dropped)
#pragma unroll
                    for (int e = 0; e < 8; ++e) v[e] = at[e * SCAN_CH];
                };
                read(even, 0);
                int t = 0;
                for (; t + 16 <= m; t += 16) {
                    read(odd, t + 8);
                    walk8(S, even, to + t * SCAN_CH);
                    read(even, t + 16);
                    walk8(S, odd, to + (t + 8) * SCAN_CH);
                }
                for (; t < m; ++t) {
                    const float2 one = in[t * SCAN_CH];
                    S = fmaf(one.x, S, one.y);
                    to[t * SCAN_CH] = S;
                }
            }
        } else {
            if (run > 0) {      // the run before: its other branch was asked for a run ago
                const int t0 = (run - 1) * SCAN_T;
                const float* from = s_s[(run - 1) & 1];
                // every product ahead of the first store: a wait for a load behind a branch around a store waits for the store too
#pragma unroll
                for (int j = 0; j < SCAN_N; ++j) y_r[j] = from[(tt + j * SCAN_STEP) * SCAN_CH + ch] * gelu_tanh_f(y_r[j] + yb);
#pragma unroll
                for (int j = 0; j < SCAN_N; ++j) {
                    const int t = t0 + tt + j * SCAN_STEP;
                    if (t < n && live) store_f(out, (size_t)(first + t) * width + c, y_r[j]);
                }
            }
            if (run < runs) {
#pragma unroll
                for (int j = 0; j < SCAN_N; ++j) {
                    const int t = min(run * SCAN_T + tt + j * SCAN_STEP, n - 1);
                    y_r[j] = proj[(size_t)(first + t) * stride + y_at + c];
                }
                store(in_s[(run + 1) & 1]);
                fetch((run + 2) * SCAN_T);
            }
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

template <typename TO, int TAPS>
__global__ void __launch_bounds__(THREADS)
step_kernel(Filter f, int y_at, const float* __restrict__ y_bias, const bf16_t* __restrict__ w, const float* __restrict__ r_bias,
            const float* __restrict__ i_bias, const float* __restrict__ decay, float* __restrict__ state, size_t state_stride,
            const int32_t* __restrict__ positions, const int32_t* __restrict__ seq_of_token, const int32_t* __restrict__ slots,
            TO* __restrict__ out, int tokens, int size, int col_tiles) {
    __shared__ __attribute__((aligned(16))) bf16_t a_s[3][STEP_ROWS * STEP_PITCH];
    __shared__ float red[4][STEP_ROWS * STEP_COLS];
    __shared__ int p_s[STEP_ROWS], slot_s[STEP_ROWS];
    const int block = blockIdx.x / col_tiles, c0 = (blockIdx.x - block * col_tiles) * STEP_COLS;
    const int t0 = blockIdx.y * STEP_ROWS, rows = min(STEP_ROWS, tokens - t0);
    const int tid = threadIdx.x, wave = tid / KIPP_WAVE, lane = tid & (KIPP_WAVE - 1), l16 = lane & 15, h = lane >> 4;
    const int gate = wave & 1, half = wave >> 1;
    const bf16_t* w_row = w + ((size_t)(block * 2 + gate) * size + min(c0 + l16, size - 1)) * size + 8 * h;
    if (tid < rows) {
        p_s[tid] = positions[t0 + tid];
        slot_s[tid] = slots[seq_of_token[t0 + tid]];
    }
    f32x4 acc = (f32x4){0.0f, 0.0f, 0.0f, 0.0f};
    for (int k0 = 0; k0 < size; k0 += STEP_KC) {
        Frag b[STEP_KC / 64];       // the weights are asked for first
#pragma unroll
        for (int s = 0; s < STEP_KC / 64; ++s) {
            const int k = k0 + 32 * (2 * s + half);
            b[s].u = k + 8 * h < size ? *(const u32x4*)(w_row + k) : (u32x4){0u, 0u, 0u, 0u};
        }
        const bool there = k0 + tid < size;
        const Channel<TAPS> channel(f, block * size + (there ? k0 + tid : 0));
        __syncthreads();            // the numbers before have been multiplied (and the rows' places are known)
#pragma unroll(TAPS > 0 ? 8 : 1)
        for (int r = 0; r < STEP_ROWS; ++r) {
            float v = 0.0f;
            if (there && r < rows) v = channel.at(f, t0 + r, t0 + r, p_s[r], state + (size_t)slot_s[r] * state_stride + f.width);
            __bf16 hi, mid, lo;
            split3(v, hi, mid, lo);
            a_s[0][r * STEP_PITCH + tid] = __builtin_bit_cast(bf16_t, hi);
            a_s[1][r * STEP_PITCH + tid] = __builtin_bit_cast(bf16_t, mid);
            a_s[2][r * STEP_PITCH + tid] = __builtin_bit_cast(bf16_t, lo);
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
    const int t = t0 + r, c = block * size + col, p = p_s[r];
    float* slot = state + (size_t)slot_s[r] * state_stride;
    float* ring = slot + f.width;
    const float u = Channel<TAPS>(f, c).at(f, t, t, p, ring);
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
    dim3 grid((tokens + FILTER_TOKENS - 1) / FILTER_TOKENS, cols);
    if (taps == 4)
        hipLaunchKernelGGL(filter_kernel<4>, grid, dim3(THREADS), 0, stream, f, (const float*)state, state_stride, positions, seq_of_token,
                           q_start, slots, u, tokens);
    else
        hipLaunchKernelGGL(filter_kernel<0>, grid, dim3(THREADS), 0, stream, f, (const float*)state, state_stride, positions, seq_of_token,
                           q_start, slots, u, tokens);
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
        hipLaunchKernelGGL(scan_kernel<float>, grid, dim3(SCAN_WG), 0, stream, (const float2*)terms, proj, stride, y_at, y_bias, state,
                           state_stride, q_start, q_len, slots, (float*)out, width);
    else if (out_dtype == KIPP_BF16)
        hipLaunchKernelGGL(scan_kernel<bf16_t>, grid, dim3(SCAN_WG), 0, stream, (const float2*)terms, proj, stride, y_at, y_bias, state,
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
#define KIPP_RS(TO, TAPS)                                                                                                          \
    hipLaunchKernelGGL((step_kernel<TO, TAPS>), grid, dim3(THREADS), 0, stream, f, y_at, y_bias, (const bf16_t*)w, r_bias, i_bias, decay, \
                       state, state_stride, positions, seq_of_token, slots, (TO*)out, tokens, size, col_tiles)
    if (out_dtype == KIPP_F32) {
        if (taps == 4) KIPP_RS(float, 4);
        else KIPP_RS(float, 0);
    } else if (out_dtype == KIPP_BF16) {
        if (taps == 4) KIPP_RS(bf16_t, 4);
        else KIPP_RS(bf16_t, 0);
    } else {
        return -2;
    }
#undef KIPP_RS
    return KIPP_LAUNCH_CHECK();
}

}  // extern "C"
