// Kinds of the linear recurrences (recurrent.hip, recurrent_chunk.hip).
#pragma once

enum Kind { GLA, MLSTM, LIGHTNING };

constexpr float DEN_EPS = 1e-6f;     // floor of the matrix LSTM's denominator
