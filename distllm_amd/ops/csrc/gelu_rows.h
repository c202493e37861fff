// Which part of a table multiplies the rows of a product: row m gets
// columns col0 .. col0 + n - 1 of table row tokens[m].
#pragma once

struct RowsArgs {
  const long* tokens;
  const void* table;
  long ld;
  int col0, n;
};
